// safetensors.cpp — see safetensors.h.
#include "safetensors.h"

#include <errno.h>
#include <fcntl.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cstdio>

#include "gguf.h"
#include "json.h"

namespace oxb {

uint32_t tensor_type_bytes(int type) { return type == GGUF_F32 || type == GGUF_I32 ? 4u : type == GGUF_F16 || type == GGUF_BF16 ? 2u : 0u; }

SafetensorsFile::~SafetensorsFile() {
    if (base_) munmap(const_cast<uint8_t*>(base_), size_);
    if (fd_ >= 0) ::close(fd_);
}

bool SafetensorsFile::open(const char* path, std::string* err) {
    auto bad = [&](const std::string& why) {
        *err = why;
        return false;
    };
    fd_ = ::open(path, O_RDONLY | O_CLOEXEC);
    if (fd_ < 0) return bad(std::string("cannot open ") + path + ": " + strerror(errno));
    struct stat sb;
    if (fstat(fd_, &sb) != 0 || !S_ISREG(sb.st_mode)) return bad(std::string(path) + " is not a regular file");
    size_ = (size_t)sb.st_size;
    if (size_ < 8) return bad("unexpected end of file (no header length)");
    void* map = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd_, 0);
    if (map == MAP_FAILED) return bad(std::string("cannot map ") + path + ": " + strerror(errno));
    base_ = static_cast<const uint8_t*>(map);
    uint64_t hl;
    memcpy(&hl, base_, 8);   // little-endian hosts only
    if (hl > size_ - 8) return bad("header of " + std::to_string(hl) + " bytes does not fit the file");
    Json h;
    std::string why;
    if (!json_parse(reinterpret_cast<const char*>(base_) + 8, (size_t)hl, &h, &why)) return bad("header: " + why);
    if (h.type != Json::Object) return bad("header is not an object");
    const uint64_t data0 = 8 + hl, room = size_ - data0;
    for (const auto& kv : h.o) {
        if (kv.first == "__metadata__") continue;
        const Json *dt = kv.second.get("dtype"), *sh = kv.second.get("shape"), *off = kv.second.get("data_offsets");
        if (!dt || dt->type != Json::String || !sh || sh->type != Json::Array || !off || off->type != Json::Array || off->a.size() != 2 ||
            !off->a[0].integral || !off->a[1].integral)
            return bad("tensor " + kv.first + ": bad entry");
        TensorView t;
        t.type = dt->s == "F32" ? (int)GGUF_F32 : dt->s == "F16" ? (int)GGUF_F16 : dt->s == "BF16" ? (int)GGUF_BF16 : dt->s == "I32" ? (int)GGUF_I32 : -1;
        uint64_t n = 1;
        for (const Json& d : sh->a) {
            if (!d.integral || d.i < 0 || (d.i && n > (1ull << 48) / (uint64_t)d.i)) return bad("tensor " + kv.first + ": bad shape");
            n *= (uint64_t)d.i;
            t.shape.push_back((uint64_t)d.i);
        }
        const int64_t a = off->a[0].i, b = off->a[1].i;
        if (a < 0 || b < a || (uint64_t)b > room) return bad("tensor " + kv.first + ": data outside the file");
        t.bytes = (uint64_t)(b - a);
        if (t.type >= 0 && t.bytes != n * tensor_type_bytes(t.type)) return bad("tensor " + kv.first + ": size does not fit its shape");
        t.data = base_ + data0 + a;
        tensors[kv.first] = std::move(t);
    }
    return true;
}

bool read_text_file(const std::string& path, std::string* out, std::string* err) {
    FILE* f = fopen(path.c_str(), "rb");
    if (!f) {
        *err = "cannot open " + path + ": " + strerror(errno);
        return false;
    }
    char buf[65536];
    size_t n;
    out->clear();
    while ((n = fread(buf, 1, sizeof buf, f)) > 0 && out->size() < (64u << 20)) out->append(buf, n);
    fclose(f);
    return true;
}

}  // namespace oxb
