// A JSON reader for configuration files and safetensors headers: values are kept as a tree.
#pragma once
#include <cstdlib>
#include <map>
#include <stdexcept>
#include <string>
#include <vector>

namespace a81w41 {

class Json {
   public:
    enum Kind { kNull, kBool, kNumber, kString, kArray, kObject };

    static Json parse(const std::string& text) {
        Reader r{text.data(), text.data() + text.size()};
        Json v = r.value(0);
        r.space();
        if (r.p != r.end) throw std::runtime_error("JSON: text after the value");
        return v;
    }

    Kind kind() const { return kind_; }
    bool is_null() const { return kind_ == kNull; }
    bool has(const std::string& key) const { return kind_ == kObject && object_.count(key) && !object_.at(key).is_null(); }
    const Json& at(const std::string& key) const {
        if (!has(key)) throw std::runtime_error("missing key '" + key + "'");
        return object_.at(key);
    }
    const std::map<std::string, Json>& object() const { return expect(kObject, "an object").object_; }
    const std::vector<Json>& array() const { return expect(kArray, "an array").array_; }
    const std::string& string() const { return expect(kString, "a string").string_; }
    double number() const { return expect(kNumber, "a number").number_; }
    long long integer() const {
        const double v = number();
        const long long i = (long long)v;
        if ((double)i != v) throw std::runtime_error("a whole number is expected");
        return i;
    }
    // A size: 1 .. 2^30
    int size(const std::string& key) const {
        const long long v = at(key).integer();
        if (v < 1 || v > (1ll << 30)) throw std::runtime_error("'" + key + "' is out of range");
        return (int)v;
    }

   private:
    const Json& expect(Kind k, const char* what) const {
        if (kind_ != k) throw std::runtime_error(std::string(what) + " is expected");
        return *this;
    }

    struct Reader {
        const char *p, *end;
        [[noreturn]] void bad(const char* what) { throw std::runtime_error(std::string("JSON: ") + what); }
        void space() {
            while (p < end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) p++;
        }
        bool take(char c) {
            space();
            if (p < end && *p == c) {
                p++;
                return true;
            }
            return false;
        }
        void word(const char* w) {
            for (; *w; w++, p++)
                if (p >= end || *p != *w) bad("unknown word");
        }
        unsigned hex4() {
            unsigned v = 0;
            for (int i = 0; i < 4; i++, p++) {
                if (p >= end) bad("short escape");
                const char c = *p;
                v = v * 16 + (c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10
                                                                                                     : (bad("bad escape"), 0));
            }
            return v;
        }
        std::string text() {
            std::string s;
            for (p++; p < end && *p != '"';) {
                if (*p != '\\') {
                    s += *p++;
                    continue;
                }
                if (++p >= end) bad("short escape");
                const char c = *p++;
                switch (c) {
                    case 'n': s += '\n'; break;
                    case 't': s += '\t'; break;
                    case 'r': s += '\r'; break;
                    case 'b': s += '\b'; break;
                    case 'f': s += '\f'; break;
                    case 'u': {
                        unsigned u = hex4();
                        if (u >= 0xD800 && u < 0xDC00 && end - p >= 6 && p[0] == '\\' && p[1] == 'u') {
                            p += 2;
                            u = 0x10000 + ((u - 0xD800) << 10) + (hex4() - 0xDC00);
                        }
                        if (u < 0x80) s += (char)u;
                        else if (u < 0x800) s += (char)(0xC0 | u >> 6), s += (char)(0x80 | (u & 63));
                        else if (u < 0x10000) s += (char)(0xE0 | u >> 12), s += (char)(0x80 | (u >> 6 & 63)), s += (char)(0x80 | (u & 63));
                        else s += (char)(0xF0 | u >> 18), s += (char)(0x80 | (u >> 12 & 63)), s += (char)(0x80 | (u >> 6 & 63)), s += (char)(0x80 | (u & 63));
                        break;
                    }
                    default: s += c;
                }
            }
            if (p >= end) bad("string without an end");
            p++;
            return s;
        }
        Json value(int depth) {
            if (depth > 64) bad("nested too deeply");
            space();
            if (p >= end) bad("short text");
            Json v;
            switch (*p) {
                case '{':
                    p++;
                    v.kind_ = kObject;
                    if (take('}')) return v;
                    do {
                        space();
                        if (p >= end || *p != '"') bad("a key is expected");
                        std::string k = text();
                        if (!take(':')) bad("':' is expected");
                        v.object_[k] = value(depth + 1);
                    } while (take(','));
                    if (!take('}')) bad("'}' is expected");
                    return v;
                case '[':
                    p++;
                    v.kind_ = kArray;
                    if (take(']')) return v;
                    do v.array_.push_back(value(depth + 1));
                    while (take(','));
                    if (!take(']')) bad("']' is expected");
                    return v;
                case '"':
                    v.kind_ = kString;
                    v.string_ = text();
                    return v;
                case 't': word("true"); v.kind_ = kBool; v.number_ = 1; return v;
                case 'f': word("false"); v.kind_ = kBool; return v;
                case 'n': word("null"); return v;
                default: {
                    std::string digits;  // the text need not end with a zero byte
                    while (p < end && ((*p >= '0' && *p <= '9') || *p == '-' || *p == '+' || *p == '.' || *p == 'e' || *p == 'E'))
                        digits += *p++;
                    char* stop = nullptr;
                    v.number_ = std::strtod(digits.c_str(), &stop);
                    if (digits.empty() || *stop) bad("a value is expected");
                    v.kind_ = kNumber;
                    return v;
                }
            }
        }
    };

    Kind kind_ = kNull;
    double number_ = 0;
    std::string string_;
    std::vector<Json> array_;
    std::map<std::string, Json> object_;
};

}  // namespace a81w41
