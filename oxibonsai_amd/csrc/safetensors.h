// safetensors.h — read-only view of a safetensors file (host only): an 8-byte little-endian header length, that many bytes
// of JSON (name -> dtype, shape, data_offsets), then the tensor data.  Memory-mapped; data is never copied.
#pragma once
#include <stddef.h>
#include <stdint.h>

#include <map>
#include <string>
#include <vector>

namespace oxb {

struct TensorView {
    int type = 0;                    // GGUF type ids: 0 F32, 1 F16, 30 BF16, 26 I32; -1: a type this tier does not read
    std::vector<uint64_t> shape;
    const uint8_t* data = nullptr;
    uint64_t bytes = 0;
    uint64_t elements() const {
        uint64_t n = 1;
        for (uint64_t d : shape) n *= d;
        return n;
    }
};
typedef std::map<std::string, TensorView> TensorMap;

class SafetensorsFile {
public:
    SafetensorsFile() = default;
    ~SafetensorsFile();
    SafetensorsFile(const SafetensorsFile&) = delete;
    SafetensorsFile& operator=(const SafetensorsFile&) = delete;
    bool open(const char* path, std::string* err);
    TensorMap tensors;

private:
    const uint8_t* base_ = nullptr;
    size_t size_ = 0;
    int fd_ = -1;
};

uint32_t tensor_type_bytes(int type);   // bytes per element, 0 for a type this tier does not read
bool read_text_file(const std::string& path, std::string* out, std::string* err);

}  // namespace oxb
