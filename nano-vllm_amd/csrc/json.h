// json.h -- a small JSON reader for config.json and safetensors headers: values, objects (members in
// file order), arrays, strings (escapes other than \uXXXX above 0x7f kept simple), numbers as double,
// true / false / null.  Malformed text ends the process with the place and the reason.
#pragma once

#include <cmath>
#include <cstdio>
#include <cstdlib>
#include <string>
#include <utility>
#include <vector>

namespace nvllm {

struct Json {
    enum Type { NUL, BOOL, NUMBER, STRING, ARRAY, OBJECT } type = NUL;
    bool boolean = false;
    double number = 0.0;
    std::string text;
    std::vector<Json> items;                               // ARRAY
    std::vector<std::pair<std::string, Json>> members;     // OBJECT

    const Json* find(const char* key) const {
        for (const auto& m : members)
            if (m.first == key) return &m.second;
        return nullptr;
    }
    bool is_null() const { return type == NUL; }
};

class JsonReader {
public:
    JsonReader(const char* text, size_t size, const char* what) : p_(text), begin_(text), end_(text + size), what_(what) {}
    Json document() {
        Json v = value(0);
        space();
        if (p_ != end_) fail("text after the end");
        return v;
    }

private:
    const char *p_, *begin_, *end_, *what_;

    [[noreturn]] void fail(const char* why) const {
        fprintf(stderr, "nvllm: %s is not valid JSON: %s at byte %zu\n", what_, why, (size_t)(p_ - begin_));
        exit(1);
    }
    void space() {
        while (p_ < end_ && (*p_ == ' ' || *p_ == '\t' || *p_ == '\n' || *p_ == '\r')) p_++;
    }
    bool take(char c) {
        space();
        if (p_ < end_ && *p_ == c) {
            p_++;
            return true;
        }
        return false;
    }
    bool word(const char* w) {
        const char* q = p_;
        while (*w && q < end_ && *q == *w) q++, w++;
        if (*w) return false;
        p_ = q;
        return true;
    }
    std::string string() {
        std::string s;
        if (!take('"')) fail("a string was expected");
        while (p_ < end_ && *p_ != '"') {
            char c = *p_++;
            if (c != '\\') {
                s.push_back(c);
                continue;
            }
            if (p_ == end_) break;
            c = *p_++;
            switch (c) {
                case 'n': s.push_back('\n'); break;
                case 't': s.push_back('\t'); break;
                case 'r': s.push_back('\r'); break;
                case 'b': s.push_back('\b'); break;
                case 'f': s.push_back('\f'); break;
                case 'u': {
                    unsigned u = 0;
                    for (int i = 0; i < 4; i++, p_++) {
                        if (p_ == end_) fail("a cut \\u escape");
                        const char h = *p_;
                        const int d = h >= '0' && h <= '9' ? h - '0' : h >= 'a' && h <= 'f' ? h - 'a' + 10 : h >= 'A' && h <= 'F' ? h - 'A' + 10 : -1;
                        if (d < 0) fail("a bad \\u escape");
                        u = u * 16 + (unsigned)d;
                    }
                    if (u < 0x80) s.push_back((char)u);
                    else if (u < 0x800) { s.push_back((char)(0xc0 | (u >> 6))); s.push_back((char)(0x80 | (u & 63))); }
                    else { s.push_back((char)(0xe0 | (u >> 12))); s.push_back((char)(0x80 | ((u >> 6) & 63))); s.push_back((char)(0x80 | (u & 63))); }
                    break;
                }
                default: s.push_back(c);
            }
        }
        if (p_ == end_) fail("an unterminated string");
        p_++;
        return s;
    }
    Json value(int depth) {
        if (depth > 64) fail("nested too deeply");
        space();
        if (p_ == end_) fail("a value was expected");
        Json v;
        if (*p_ == '{') {
            p_++;
            v.type = Json::OBJECT;
            if (take('}')) return v;
            do {
                space();
                std::string key = string();
                if (!take(':')) fail("':' was expected");
                v.members.emplace_back(std::move(key), value(depth + 1));
            } while (take(','));
            if (!take('}')) fail("'}' was expected");
        } else if (*p_ == '[') {
            p_++;
            v.type = Json::ARRAY;
            if (take(']')) return v;
            do v.items.push_back(value(depth + 1));
            while (take(','));
            if (!take(']')) fail("']' was expected");
        } else if (*p_ == '"') {
            v.type = Json::STRING;
            v.text = string();
        } else if (word("true")) {
            v.type = Json::BOOL;
            v.boolean = true;
        } else if (word("false")) {
            v.type = Json::BOOL;
        } else if (word("null")) {
        } else {
            std::string num;
            while (p_ < end_ && ((*p_ >= '0' && *p_ <= '9') || *p_ == '-' || *p_ == '+' || *p_ == '.' || *p_ == 'e' || *p_ == 'E')) num.push_back(*p_++);
            char* stop = nullptr;
            v.type = Json::NUMBER;
            v.number = strtod(num.c_str(), &stop);
            if (num.empty() || *stop) fail("a value was expected");
        }
        return v;
    }
};

// Typed access with the key's path in the message when something is missing or of the wrong type.
inline const Json& json_get(const Json& obj, const char* key, Json::Type type, const char* where) {
    const Json* v = obj.type == Json::OBJECT ? obj.find(key) : nullptr;
    if (!v || v->type != type) {
        fprintf(stderr, "nvllm: config.json: %s.%s is missing or of the wrong type\n", where, key);
        exit(1);
    }
    return *v;
}
inline int json_int(const Json& obj, const char* key, const char* where) {
    const double d = json_get(obj, key, Json::NUMBER, where).number;
    if (d != std::floor(d) || d < -2147483647.0 || d > 2147483647.0) {
        fprintf(stderr, "nvllm: config.json: %s.%s is not an integer\n", where, key);
        exit(1);
    }
    return (int)d;
}
inline double json_num(const Json& obj, const char* key, const char* where) { return json_get(obj, key, Json::NUMBER, where).number; }

}  // namespace nvllm
