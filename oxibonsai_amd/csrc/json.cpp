// json.cpp — recursive-descent JSON reader (see json.h).
#include "json.h"

#include <stdlib.h>
#include <string.h>

namespace oxb {

namespace {

struct Parser {
    const char* p;
    const char* end;
    const char* begin;
    std::string why;

    bool bad(const char* what) {
        if (why.empty()) why = std::string(what) + " at byte " + std::to_string(p - begin);
        return false;
    }
    void space() {
        while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) p++;
    }
    bool word(const char* w) {
        const size_t n = strlen(w);
        if ((size_t)(end - p) < n || memcmp(p, w, n) != 0) return bad("unexpected character");
        p += n;
        return true;
    }
    static void utf8(std::string* s, uint32_t c) {
        if (c < 0x80) *s += (char)c;
        else if (c < 0x800) *s += (char)(0xC0 | c >> 6), *s += (char)(0x80 | (c & 63));
        else if (c < 0x10000) *s += (char)(0xE0 | c >> 12), *s += (char)(0x80 | (c >> 6 & 63)), *s += (char)(0x80 | (c & 63));
        else *s += (char)(0xF0 | c >> 18), *s += (char)(0x80 | (c >> 12 & 63)), *s += (char)(0x80 | (c >> 6 & 63)), *s += (char)(0x80 | (c & 63));
    }
    bool hex4(uint32_t* v) {
        if (end - p < 4) return bad("unfinished escape");
        *v = 0;
        for (int k = 0; k < 4; k++, p++) {
            const char c = *p;
            const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
            if (d < 0) return bad("bad escape");
            *v = *v * 16 + (uint32_t)d;
        }
        return true;
    }
    bool string(std::string* s) {
        p++;  // the opening quote
        while (p < end && *p != '"') {
            if ((unsigned char)*p < 0x20) return bad("control character in a string");
            if (*p != '\\') {
                *s += *p++;
                continue;
            }
            if (++p >= end) break;
            const char c = *p++;
            switch (c) {
                case '"': case '\\': case '/': *s += c; break;
                case 'b': *s += '\b'; break;
                case 'f': *s += '\f'; break;
                case 'n': *s += '\n'; break;
                case 'r': *s += '\r'; break;
                case 't': *s += '\t'; break;
                case 'u': {
                    uint32_t v, lo;
                    if (!hex4(&v)) return false;
                    if (v >= 0xD800 && v < 0xDC00) {
                        if (end - p < 6 || p[0] != '\\' || p[1] != 'u') return bad("lone surrogate");
                        p += 2;
                        if (!hex4(&lo)) return false;
                        if (lo < 0xDC00 || lo > 0xDFFF) return bad("lone surrogate");
                        v = 0x10000 + ((v - 0xD800) << 10) + (lo - 0xDC00);
                    }
                    utf8(s, v);
                    break;
                }
                default: return bad("bad escape");
            }
        }
        if (p >= end) return bad("unfinished string");
        p++;
        return true;
    }
    bool number(Json* j) {
        const char* s = p;
        bool whole = true;
        if (*p == '-') p++;
        if (p >= end || *p < '0' || *p > '9') return bad("bad number");
        while (p < end && ((*p >= '0' && *p <= '9') || *p == '.' || *p == 'e' || *p == 'E' || *p == '+' || *p == '-')) {
            if (*p == '.' || *p == 'e' || *p == 'E') whole = false;
            p++;
        }
        const std::string t(s, p);
        char* stop = nullptr;
        j->num = strtod(t.c_str(), &stop);
        if (*stop) return bad("bad number");
        j->integral = whole && t.size() <= 18;
        if (j->integral) j->i = strtoll(t.c_str(), nullptr, 10);
        j->type = Json::Number;
        return true;
    }
    bool value(Json* j, int depth) {
        if (depth > 64) return bad("nested too deeply");
        space();
        if (p >= end) return bad("unexpected end");
        switch (*p) {
            case '{': {
                j->type = Json::Object;
                p++;
                space();
                if (p < end && *p == '}') return p++, true;
                for (;;) {
                    space();
                    if (p >= end || *p != '"') return bad("expected a key");
                    std::string k;
                    if (!string(&k)) return false;
                    space();
                    if (p >= end || *p != ':') return bad("expected ':'");
                    p++;
                    if (!value(&j->o[k], depth + 1)) return false;
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == '}') return p++, true;
                    return bad("expected ',' or '}'");
                }
            }
            case '[': {
                j->type = Json::Array;
                p++;
                space();
                if (p < end && *p == ']') return p++, true;
                for (;;) {
                    j->a.emplace_back();
                    if (!value(&j->a.back(), depth + 1)) return false;
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == ']') return p++, true;
                    return bad("expected ',' or ']'");
                }
            }
            case '"': j->type = Json::String; return string(&j->s);
            case 't': j->type = Json::Bool, j->b = true; return word("true");
            case 'f': j->type = Json::Bool, j->b = false; return word("false");
            case 'n': j->type = Json::Null; return word("null");
            default: return number(j);
        }
    }
};

}  // namespace

bool json_parse(const char* text, size_t len, Json* out, std::string* err) {
    Parser q{text, text + len, text, {}};
    *out = Json();
    bool ok = q.value(out, 0);
    if (ok) {
        q.space();
        if (q.p != q.end) ok = q.bad("text after the value");
    }
    if (!ok && err) *err = q.why;
    return ok;
}

}  // namespace oxb
