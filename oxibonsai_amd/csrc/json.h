// json.h — a small JSON reader (host only): what model configurations and safetensors headers need.
#pragma once
#include <stddef.h>
#include <stdint.h>

#include <map>
#include <string>
#include <vector>

namespace oxb {

struct Json {
    enum Type { Null, Bool, Number, String, Array, Object } type = Null;
    bool b = false;
    double num = 0.0;
    bool integral = false;   // written without fraction or exponent and within int64
    int64_t i = 0;
    std::string s;
    std::vector<Json> a;
    std::map<std::string, Json> o;

    const Json* get(const char* key) const {   // null: not an object, or no such key
        if (type != Object) return nullptr;
        auto it = o.find(key);
        return it == o.end() ? nullptr : &it->second;
    }
    bool is_null() const { return type == Null; }
};

// Parses the whole text (nothing but white space may follow the value); on failure returns false and leaves the reason
// and the byte offset in err.  Nesting is limited to 64 levels.
bool json_parse(const char* text, size_t len, Json* out, std::string* err);

}  // namespace oxb
