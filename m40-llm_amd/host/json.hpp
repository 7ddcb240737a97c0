// A small JSON reader: what model folders need (config.json, the header of a safetensors file).
#pragma once

#include <cctype>
#include <cmath>
#include <cstdint>
#include <cstdlib>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

namespace m40host {
namespace json {

struct Error : std::runtime_error {
    using std::runtime_error::runtime_error;
};

class Value {
public:
    enum class Kind { Null, Bool, Number, String, Array, Object };
    Kind kind = Kind::Null;
    bool boolean = false;
    double number = 0.0;
    std::string string;
    std::vector<Value> items;
    std::vector<std::pair<std::string, Value>> members;

    bool is_null() const { return kind == Kind::Null; }
    // a member, or null where the object lacks it
    const Value* find(const std::string& key) const {
        if (kind != Kind::Object) return nullptr;
        for (const auto& m : members)
            if (m.first == key) return &m.second;
        return nullptr;
    }
    const Value& at(const std::string& key) const {
        const Value* v = find(key);
        if (!v) throw Error("missing key '" + key + "'");
        return *v;
    }
    double num(const std::string& key) const {
        const Value& v = at(key);
        if (v.kind != Kind::Number) throw Error("'" + key + "' is not a number");
        return v.number;
    }
    uint32_t u32(const std::string& key) const { return at(key).as_u32(key); }
    uint32_t as_u32(const std::string& what) const {
        if (kind != Kind::Number || number < 0.0 || number > 4294967295.0 || number != std::floor(number))
            throw Error("'" + what + "' is not a 32-bit count");
        return static_cast<uint32_t>(number);
    }
    const std::string& str(const std::string& key) const {
        const Value& v = at(key);
        if (v.kind != Kind::String) throw Error("'" + key + "' is not a string");
        return v.string;
    }
    // the same value, members in any order
    bool operator==(const Value& o) const {
        if (kind != o.kind || boolean != o.boolean || number != o.number || string != o.string || items != o.items || members.size() != o.members.size()) return false;
        for (const auto& m : members) {
            const Value* v = o.find(m.first);
            if (!v || !(m.second == *v)) return false;
        }
        return true;
    }
    bool operator!=(const Value& o) const { return !(*this == o); }
    const std::vector<Value>& array(const std::string& key) const {
        const Value& v = at(key);
        if (v.kind != Kind::Array) throw Error("'" + key + "' is not a list");
        return v.items;
    }
};

class Parser {
public:
    Parser(const char* p, size_t n) : p_(p), end_(p + n) {}
    Value document() {
        Value v = value(0);
        space();
        if (p_ != end_) throw Error("text after the JSON value");
        return v;
    }

private:
    void space() {
        while (p_ != end_ && (*p_ == ' ' || *p_ == '\t' || *p_ == '\n' || *p_ == '\r')) ++p_;
    }
    char peek() {
        space();
        if (p_ == end_) throw Error("JSON text ends early");
        return *p_;
    }
    void expect(char c) {
        if (peek() != c) throw Error(std::string("JSON: expected '") + c + "'");
        ++p_;
    }
    bool word(const char* w) {
        const char* q = p_;
        for (; *w; ++w, ++q)
            if (q == end_ || *q != *w) return false;
        p_ = q;
        return true;
    }
    static void utf8(std::string& out, uint32_t c) {
        if (c < 0x80) out += (char)c;
        else if (c < 0x800) { out += (char)(0xc0 | (c >> 6)); out += (char)(0x80 | (c & 63)); }
        else if (c < 0x10000) { out += (char)(0xe0 | (c >> 12)); out += (char)(0x80 | ((c >> 6) & 63)); out += (char)(0x80 | (c & 63)); }
        else { out += (char)(0xf0 | (c >> 18)); out += (char)(0x80 | ((c >> 12) & 63)); out += (char)(0x80 | ((c >> 6) & 63)); out += (char)(0x80 | (c & 63)); }
    }
    uint32_t hex4() {
        uint32_t v = 0;
        for (int i = 0; i < 4; ++i, ++p_) {
            if (p_ == end_) throw Error("JSON text ends early");
            const char c = *p_;
            const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
            if (d < 0) throw Error("JSON: bad \\u escape");
            v = v * 16 + (uint32_t)d;
        }
        return v;
    }
    std::string text() {
        expect('"');
        std::string out;
        for (;;) {
            if (p_ == end_) throw Error("JSON text ends early");
            const char c = *p_++;
            if (c == '"') return out;
            if (c != '\\') { out += c; continue; }
            if (p_ == end_) throw Error("JSON text ends early");
            const char e = *p_++;
            switch (e) {
                case '"': case '\\': case '/': out += e; break;
                case 'b': out += '\b'; break;
                case 'f': out += '\f'; break;
                case 'n': out += '\n'; break;
                case 'r': out += '\r'; break;
                case 't': out += '\t'; break;
                case 'u': {
                    uint32_t c32 = hex4();
                    if (c32 >= 0xd800 && c32 < 0xdc00 && word("\\u")) c32 = 0x10000 + ((c32 - 0xd800) << 10) + (hex4() - 0xdc00);
                    utf8(out, c32);
                    break;
                }
                default: throw Error("JSON: bad escape");
            }
        }
    }
    Value value(int depth) {
        if (depth > 64) throw Error("JSON nested too deeply");
        Value v;
        switch (peek()) {
            case '{':
                v.kind = Value::Kind::Object;
                ++p_;
                if (peek() == '}') { ++p_; return v; }
                for (;;) {
                    (void)peek();
                    std::string key = text();
                    expect(':');
                    v.members.emplace_back(std::move(key), value(depth + 1));
                    if (peek() == ',') { ++p_; continue; }
                    expect('}');
                    return v;
                }
            case '[':
                v.kind = Value::Kind::Array;
                ++p_;
                if (peek() == ']') { ++p_; return v; }
                for (;;) {
                    v.items.push_back(value(depth + 1));
                    if (peek() == ',') { ++p_; continue; }
                    expect(']');
                    return v;
                }
            case '"': v.kind = Value::Kind::String; v.string = text(); return v;
            case 't': if (word("true")) { v.kind = Value::Kind::Bool; v.boolean = true; return v; } break;
            case 'f': if (word("false")) { v.kind = Value::Kind::Bool; return v; } break;
            case 'n': if (word("null")) return v; break;
            default: break;
        }
        const char* q = p_;
        while (q != end_ && (std::isdigit((unsigned char)*q) || *q == '-' || *q == '+' || *q == '.' || *q == 'e' || *q == 'E')) ++q;
        if (q == p_) throw Error("JSON: unexpected character");
        const std::string num(p_, q);
        char* stop = nullptr;
        v.kind = Value::Kind::Number;
        v.number = std::strtod(num.c_str(), &stop);
        if (!stop || *stop) throw Error("JSON: bad number '" + num + "'");
        p_ = q;
        return v;
    }
    const char *p_, *end_;
};

inline Value parse(const char* p, size_t n) { return Parser(p, n).document(); }

}  // namespace json
}  // namespace m40host
