// qm_json.hpp — JSON reader of the engine shell: safetensors headers and config.json.
#pragma once

#include <cctype>
#include <cstdlib>
#include <cstring>
#include <string>
#include <utility>
#include <vector>

#include "qm_safetensors.hpp"

namespace qm_engine {

// A JSON value: objects, arrays, strings, numbers, literals.
struct Json {
    enum Kind { Null, Bool, Number, String, Array, Object } kind = Null;
    bool boolean = false;
    double number = 0.0;
    std::string text;
    std::vector<Json> items;
    std::vector<std::pair<std::string, Json>> members;

    const Json* member(const std::string& key) const {
        for (const auto& m : members)
            if (m.first == key) return &m.second;
        return nullptr;
    }
};

class JsonReader {
public:
    JsonReader(const char* begin, size_t size, const char* what) : p_(begin), end_(begin + size), what_(what) {}
    Json document() {
        Json v = value(0);
        blanks();
        if (p_ != end_) fail("text after the document");
        return v;
    }

private:
    const char* p_;
    const char* end_;
    const char* what_;

    [[noreturn]] void fail(const char* what) const { throw IoError(std::string(what_) + ": " + what); }
    void blanks() {
        while (p_ != end_ && (*p_ == ' ' || *p_ == '\t' || *p_ == '\n' || *p_ == '\r')) ++p_;
    }
    bool take(char c) {
        blanks();
        if (p_ != end_ && *p_ == c) {
            ++p_;
            return true;
        }
        return false;
    }
    void expect(char c) {
        if (!take(c)) fail("unexpected character");
    }
    void word(const char* w) {
        const size_t n = std::strlen(w);
        if (static_cast<size_t>(end_ - p_) < n || std::memcmp(p_, w, n) != 0) fail("unknown literal");
        p_ += n;
    }
    static void utf8(std::string& out, unsigned cp) {
        if (cp < 0x80) {
            out.push_back(static_cast<char>(cp));
        } else if (cp < 0x800) {
            out.push_back(static_cast<char>(0xc0 | (cp >> 6)));
            out.push_back(static_cast<char>(0x80 | (cp & 0x3f)));
        } else if (cp < 0x10000) {
            out.push_back(static_cast<char>(0xe0 | (cp >> 12)));
            out.push_back(static_cast<char>(0x80 | ((cp >> 6) & 0x3f)));
            out.push_back(static_cast<char>(0x80 | (cp & 0x3f)));
        } else {
            out.push_back(static_cast<char>(0xf0 | (cp >> 18)));
            out.push_back(static_cast<char>(0x80 | ((cp >> 12) & 0x3f)));
            out.push_back(static_cast<char>(0x80 | ((cp >> 6) & 0x3f)));
            out.push_back(static_cast<char>(0x80 | (cp & 0x3f)));
        }
    }
    unsigned hex4() {
        if (end_ - p_ < 4) fail("short \\u escape");
        unsigned v = 0;
        for (int i = 0; i < 4; ++i) {
            const char c = *p_++;
            v <<= 4;
            if (c >= '0' && c <= '9') v |= static_cast<unsigned>(c - '0');
            else if (c >= 'a' && c <= 'f') v |= static_cast<unsigned>(c - 'a' + 10);
            else if (c >= 'A' && c <= 'F') v |= static_cast<unsigned>(c - 'A' + 10);
            else fail("bad \\u escape");
        }
        return v;
    }
    std::string string() {
        blanks();
        if (p_ == end_ || *p_ != '"') fail("string expected");
        ++p_;
        std::string out;
        while (p_ != end_) {
            const char c = *p_++;
            if (c == '"') return out;
            if (c != '\\') {
                out.push_back(c);
                continue;
            }
            if (p_ == end_) break;
            const char e = *p_++;
            switch (e) {
                case '"': out.push_back('"'); break;
                case '\\': out.push_back('\\'); break;
                case '/': out.push_back('/'); break;
                case 'b': out.push_back('\b'); break;
                case 'f': out.push_back('\f'); break;
                case 'n': out.push_back('\n'); break;
                case 'r': out.push_back('\r'); break;
                case 't': out.push_back('\t'); break;
                case 'u': {
                    unsigned cp = hex4();
                    if (cp >= 0xd800 && cp < 0xdc00 && end_ - p_ >= 6 && p_[0] == '\\' && p_[1] == 'u') {
                        p_ += 2;
                        const unsigned low = hex4();
                        cp = 0x10000 + ((cp - 0xd800) << 10) + (low - 0xdc00);
                    }
                    utf8(out, cp);
                    break;
                }
                default: fail("bad escape");
            }
        }
        fail("unterminated string");
    }
    Json value(int depth) {
        if (depth > 64) fail("nesting too deep");
        blanks();
        if (p_ == end_) fail("unexpected end");
        Json v;
        const char c = *p_;
        if (c == '{') {
            ++p_;
            v.kind = Json::Object;
            if (take('}')) return v;
            do {
                std::string key = string();
                expect(':');
                v.members.emplace_back(std::move(key), value(depth + 1));
            } while (take(','));
            expect('}');
        } else if (c == '[') {
            ++p_;
            v.kind = Json::Array;
            if (take(']')) return v;
            do {
                v.items.push_back(value(depth + 1));
            } while (take(','));
            expect(']');
        } else if (c == '"') {
            v.kind = Json::String;
            v.text = string();
        } else if (c == 't') {
            word("true");
            v.kind = Json::Bool;
            v.boolean = true;
        } else if (c == 'f') {
            word("false");
            v.kind = Json::Bool;
        } else if (c == 'n') {
            word("null");
        } else {
            const char* start = p_;
            while (p_ != end_ && (std::isdigit(static_cast<unsigned char>(*p_)) || *p_ == '-' || *p_ == '+' || *p_ == '.'
                                  || *p_ == 'e' || *p_ == 'E'))
                ++p_;
            if (p_ == start) fail("value expected");
            const std::string digits(start, p_);
            char* stop = nullptr;
            v.kind = Json::Number;
            v.number = std::strtod(digits.c_str(), &stop);
            if (stop == digits.c_str() || *stop != '\0') fail("bad number");
        }
        return v;
    }
};

}  // namespace qm_engine
