// A small JSON reader for model folders (config.json and the header of a safetensors file).  Host only, not installed.
// Values are a tree of Json nodes; numbers are kept as double (every integer below 2^53 is exact).
#pragma once

#include <cstdint>
#include <cstdlib>
#include <string>
#include <utility>
#include <vector>

namespace wick_rocm {

struct Json {
    enum Kind { kNull, kBool, kNumber, kString, kArray, kObject };
    Kind kind = kNull;
    bool boolean = false;
    double number = 0.0;
    std::string string;
    std::vector<Json> items;                             // array
    std::vector<std::pair<std::string, Json>> members;   // object, in file order

    bool is_null() const { return kind == kNull; }
    const Json* find(const char* key) const {
        if (kind == kObject)
            for (const auto& m : members)
                if (m.first == key) return &m.second;
        return nullptr;
    }
};

// Parses one JSON document; false (with a message) on malformed text, trailing bytes or nesting deeper than 64.
class JsonParser {
  public:
    static bool parse(const char* text, size_t n, Json& out, std::string& error) {
        JsonParser p{text, text + n};
        bool ok = p.value(out, 0);
        if (ok) {
            p.space();
            if (p.at_ != p.end_) ok = p.fail("text behind the document");
        }
        if (!ok) error = p.error_ + " at byte " + std::to_string(p.at_ - text);
        return ok;
    }

  private:
    JsonParser(const char* at, const char* end) : at_(at), end_(end) {}
    const char *at_, *end_;
    std::string error_;

    bool fail(const char* what) {
        if (error_.empty()) error_ = what;
        return false;
    }
    void space() {
        while (at_ != end_ && (*at_ == ' ' || *at_ == '\t' || *at_ == '\n' || *at_ == '\r')) at_++;
    }
    bool word(const char* w) {
        for (; *w; w++, at_++)
            if (at_ == end_ || *at_ != *w) return fail("unknown word");
        return true;
    }
    static void utf8(uint32_t c, std::string& s) {
        if (c < 0x80) {
            s += (char)c;
        } else if (c < 0x800) {
            s += (char)(0xC0 | c >> 6), s += (char)(0x80 | (c & 63));
        } else if (c < 0x10000) {
            s += (char)(0xE0 | c >> 12), s += (char)(0x80 | (c >> 6 & 63)), s += (char)(0x80 | (c & 63));
        } else {
            s += (char)(0xF0 | c >> 18), s += (char)(0x80 | (c >> 12 & 63)), s += (char)(0x80 | (c >> 6 & 63)), s += (char)(0x80 | (c & 63));
        }
    }
    bool hex4(uint32_t& v) {
        v = 0;
        for (int i = 0; i < 4; i++, at_++) {
            if (at_ == end_) return fail("short \\u escape");
            const char c = *at_;
            const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
            if (d < 0) return fail("bad \\u escape");
            v = v * 16 + (uint32_t)d;
        }
        return true;
    }
    bool str(std::string& s) {
        at_++;  // the opening quote
        while (at_ != end_ && *at_ != '"') {
            if ((unsigned char)*at_ < 0x20) return fail("control character in a string");
            if (*at_ != '\\') {
                s += *at_++;
                continue;
            }
            if (++at_ == end_) break;
            const char c = *at_++;
            switch (c) {
                case '"': case '\\': case '/': s += c; break;
                case 'b': s += '\b'; break;
                case 'f': s += '\f'; break;
                case 'n': s += '\n'; break;
                case 'r': s += '\r'; break;
                case 't': s += '\t'; break;
                case 'u': {
                    uint32_t v = 0, lo = 0;
                    if (!hex4(v)) return false;
                    if (v >= 0xD800 && v < 0xDC00) {  // a surrogate pair
                        if (end_ - at_ < 2 || at_[0] != '\\' || at_[1] != 'u') return fail("lone surrogate");
                        at_ += 2;
                        if (!hex4(lo)) return false;
                        if (lo < 0xDC00 || lo > 0xDFFF) return fail("lone surrogate");
                        v = 0x10000 + ((v - 0xD800) << 10) + (lo - 0xDC00);
                    }
                    utf8(v, s);
                    break;
                }
                default: return fail("unknown escape");
            }
        }
        if (at_ == end_) return fail("unterminated string");
        at_++;
        return true;
    }
    bool number(Json& v) {
        const char* b = at_;
        while (at_ != end_ && ((*at_ >= '0' && *at_ <= '9') || *at_ == '-' || *at_ == '+' || *at_ == '.' || *at_ == 'e' || *at_ == 'E')) at_++;
        const std::string t(b, at_);
        char* e = nullptr;
        v.kind = Json::kNumber, v.number = strtod(t.c_str(), &e);
        return (!t.empty() && e == t.c_str() + t.size()) || fail("bad number");
    }
    bool value(Json& v, int depth) {
        if (depth > 64) return fail("nested too deeply");
        space();
        if (at_ == end_) return fail("unexpected end");
        switch (*at_) {
            case '{': {
                v.kind = Json::kObject, at_++, space();
                if (at_ != end_ && *at_ == '}') return at_++, true;
                for (;;) {
                    space();
                    if (at_ == end_ || *at_ != '"') return fail("expected a key");
                    v.members.emplace_back();
                    if (!str(v.members.back().first)) return false;
                    space();
                    if (at_ == end_ || *at_ != ':') return fail("expected ':'");
                    at_++;
                    if (!value(v.members.back().second, depth + 1)) return false;
                    space();
                    if (at_ != end_ && *at_ == ',') { at_++; continue; }
                    if (at_ != end_ && *at_ == '}') return at_++, true;
                    return fail("expected ',' or '}'");
                }
            }
            case '[': {
                v.kind = Json::kArray, at_++, space();
                if (at_ != end_ && *at_ == ']') return at_++, true;
                for (;;) {
                    v.items.emplace_back();
                    if (!value(v.items.back(), depth + 1)) return false;
                    space();
                    if (at_ != end_ && *at_ == ',') { at_++; continue; }
                    if (at_ != end_ && *at_ == ']') return at_++, true;
                    return fail("expected ',' or ']'");
                }
            }
            case '"': v.kind = Json::kString; return str(v.string);
            case 't': v.kind = Json::kBool, v.boolean = true; return word("true");
            case 'f': v.kind = Json::kBool; return word("false");
            case 'n': return word("null");
            default: return number(v);
        }
    }
};

}  // namespace wick_rocm
