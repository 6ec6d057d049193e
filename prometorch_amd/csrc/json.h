// A small JSON reader for model folders: config.json and the header of a safetensors file.  Host only.
#pragma once
#include <cstdint>
#include <cstdlib>
#include <cstring>
#include <string>
#include <utility>
#include <vector>

namespace ptm {

struct Json {
    enum Kind { Null, Bool, Number, String, Array, Object } kind = Null;
    bool b = false;
    double num = 0.0;
    std::string str;
    std::vector<Json> items;                            // Array
    std::vector<std::pair<std::string, Json>> members;  // Object, in file order

    const Json* find(const char* key) const {
        if (kind != Object) return nullptr;
        for (const auto& m : members)
            if (m.first == key) return &m.second;
        return nullptr;
    }
    bool is_null() const { return kind == Null; }
};

class JsonParser {
  public:
    JsonParser(const char* p, size_t n) : p_(p), end_(p + n) {}
    bool parse(Json* out) {
        if (!value(out, 0)) return false;
        ws();
        return p_ == end_ || *p_ == '\0';
    }

  private:
    const char *p_, *end_;
    void ws() {
        while (p_ < end_ && (*p_ == ' ' || *p_ == '\n' || *p_ == '\r' || *p_ == '\t')) ++p_;
    }
    bool lit(const char* s) {
        const size_t n = strlen(s);
        if ((size_t)(end_ - p_) < n || memcmp(p_, s, n) != 0) return false;
        p_ += n;
        return true;
    }
    static void utf8(std::string* s, uint32_t c) {
        if (c < 0x80) s->push_back((char)c);
        else if (c < 0x800) { s->push_back((char)(0xC0 | (c >> 6))); s->push_back((char)(0x80 | (c & 63))); }
        else { s->push_back((char)(0xE0 | (c >> 12))); s->push_back((char)(0x80 | ((c >> 6) & 63))); s->push_back((char)(0x80 | (c & 63))); }
    }
    bool string(std::string* out) {
        if (p_ >= end_ || *p_ != '"') return false;
        ++p_;
        while (p_ < end_ && *p_ != '"') {
            if (*p_ != '\\') { out->push_back(*p_++); continue; }
            if (++p_ >= end_) return false;
            switch (*p_++) {
                case '"': out->push_back('"'); break;
                case '\\': out->push_back('\\'); break;
                case '/': out->push_back('/'); break;
                case 'b': out->push_back('\b'); break;
                case 'f': out->push_back('\f'); break;
                case 'n': out->push_back('\n'); break;
                case 'r': out->push_back('\r'); break;
                case 't': out->push_back('\t'); break;
                case 'u': {
                    if (end_ - p_ < 4) return false;
                    uint32_t c = 0;
                    for (int i = 0; i < 4; ++i) {
                        const char ch = *p_++;
                        c = c * 16 + (ch >= '0' && ch <= '9' ? ch - '0' : ch >= 'a' && ch <= 'f' ? ch - 'a' + 10 : ch >= 'A' && ch <= 'F' ? ch - 'A' + 10 : 256);
                        if (c >= 0x10000) return false;
                    }
                    utf8(out, c);
                    break;
                }
                default: return false;
            }
        }
        if (p_ >= end_) return false;
        ++p_;
        return true;
    }
    bool value(Json* v, int depth) {
        if (depth > 64) return false;
        ws();
        if (p_ >= end_) return false;
        if (*p_ == '{') {
            ++p_;
            v->kind = Json::Object;
            ws();
            if (p_ < end_ && *p_ == '}') { ++p_; return true; }
            for (;;) {
                ws();
                std::string key;
                if (!string(&key)) return false;
                ws();
                if (p_ >= end_ || *p_++ != ':') return false;
                v->members.emplace_back(std::move(key), Json());
                if (!value(&v->members.back().second, depth + 1)) return false;
                ws();
                if (p_ >= end_) return false;
                const char c = *p_++;
                if (c == '}') return true;
                if (c != ',') return false;
            }
        }
        if (*p_ == '[') {
            ++p_;
            v->kind = Json::Array;
            ws();
            if (p_ < end_ && *p_ == ']') { ++p_; return true; }
            for (;;) {
                v->items.emplace_back();
                if (!value(&v->items.back(), depth + 1)) return false;
                ws();
                if (p_ >= end_) return false;
                const char c = *p_++;
                if (c == ']') return true;
                if (c != ',') return false;
            }
        }
        if (*p_ == '"') { v->kind = Json::String; return string(&v->str); }
        if (lit("true")) { v->kind = Json::Bool; v->b = true; return true; }
        if (lit("false")) { v->kind = Json::Bool; return true; }
        if (lit("null")) return true;
        // a number: copied out, because the buffer need not end with a terminator
        char tmp[64];
        size_t n = 0;
        while (p_ < end_ && n + 1 < sizeof tmp && (strchr("+-.eE", *p_) || (*p_ >= '0' && *p_ <= '9')) && *p_) tmp[n++] = *p_++;
        tmp[n] = '\0';
        char* stop = nullptr;
        v->kind = Json::Number;
        v->num = strtod(tmp, &stop);
        return n > 0 && stop == tmp + n;
    }
};

}  // namespace ptm
