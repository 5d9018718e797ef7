// A small JSON reader for configurations and safetensors headers (host code).
#pragma once
#include <cmath>
#include <cstdint>
#include <cstdlib>
#include <cstring>
#include <string>
#include <utility>
#include <vector>

struct FhJson {
    enum Kind { NUL, BOOL, NUMBER, STRING, ARRAY, OBJECT } kind = NUL;
    double num = 0;
    bool flag = false;
    std::string str;
    std::vector<FhJson> items;                            // ARRAY
    std::vector<std::pair<std::string, FhJson>> members;  // OBJECT, in file order

    bool is_null() const { return kind == NUL; }
    bool is_number() const { return kind == NUMBER; }
    bool is_string() const { return kind == STRING; }
    bool is_object() const { return kind == OBJECT; }
    bool is_array() const { return kind == ARRAY; }
    // a member that is there and not null; the last one of a repeated name
    const FhJson *find(const char *name) const {
        for (size_t i = members.size(); i-- > 0;)
            if (members[i].first == name) return members[i].second.is_null() ? nullptr : &members[i].second;
        return nullptr;
    }

    static bool parse(const char *text, size_t len, FhJson &out, std::string &err) {
        Reader r{text, text + len, text, err};
        if (!r.value(out, 0)) return false;
        r.space();
        return r.p == r.end || r.fail("text after the value");
    }

  private:
    struct Reader {
        const char *p, *end, *start;
        std::string &err;
        bool fail(const char *what) {
            err = std::string(what) + " at byte " + std::to_string(p - start);
            return false;
        }
        void space() {
            while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) p++;
        }
        bool word(const char *w) {
            const size_t n = strlen(w);
            if ((size_t)(end - p) < n || memcmp(p, w, n)) return fail("unknown word");
            p += n;
            return true;
        }
        static void utf8(std::string &s, uint32_t c) {
            if (c < 0x80) s += (char)c;
            else if (c < 0x800) s += (char)(0xC0 | c >> 6), s += (char)(0x80 | (c & 63));
            else if (c < 0x10000) s += (char)(0xE0 | c >> 12), s += (char)(0x80 | (c >> 6 & 63)), s += (char)(0x80 | (c & 63));
            else s += (char)(0xF0 | c >> 18), s += (char)(0x80 | (c >> 12 & 63)), s += (char)(0x80 | (c >> 6 & 63)), s += (char)(0x80 | (c & 63));
        }
        bool hex4(uint32_t &c) {
            if (end - p < 4) return fail("short escape");
            c = 0;
            for (int i = 0; i < 4; i++, p++) {
                const char d = *p;
                const int v = d >= '0' && d <= '9' ? d - '0' : d >= 'a' && d <= 'f' ? d - 'a' + 10 : d >= 'A' && d <= 'F' ? d - 'A' + 10 : -1;
                if (v < 0) return fail("bad escape");
                c = c * 16 + (uint32_t)v;
            }
            return true;
        }
        bool string(std::string &s) {
            p++; // the quote
            while (p < end && *p != '"') {
                if (*p != '\\') { s += *p++; continue; }
                if (++p >= end) break;
                const char e = *p++;
                uint32_t c;
                switch (e) {
                case 'b': s += '\b'; break;
                case 'f': s += '\f'; break;
                case 'n': s += '\n'; break;
                case 'r': s += '\r'; break;
                case 't': s += '\t'; break;
                case 'u':
                    if (!hex4(c)) return false;
                    if (c >= 0xD800 && c < 0xDC00 && end - p >= 6 && p[0] == '\\' && p[1] == 'u') {
                        uint32_t lo;
                        p += 2;
                        if (!hex4(lo)) return false;
                        c = 0x10000 + ((c - 0xD800) << 10) + (lo - 0xDC00);
                    }
                    utf8(s, c);
                    break;
                default: s += e;
                }
            }
            if (p >= end) return fail("string without an end");
            p++;
            return true;
        }
        bool value(FhJson &v, int depth) {
            if (depth > 64) return fail("nested too deep");
            space();
            if (p >= end) return fail("value expected");
            switch (*p) {
            case '{':
                v.kind = OBJECT;
                p++;
                space();
                if (p < end && *p == '}') { p++; return true; }
                while (true) {
                    space();
                    if (p >= end || *p != '"') return fail("name expected");
                    v.members.emplace_back();
                    if (!string(v.members.back().first)) return false;
                    space();
                    if (p >= end || *p != ':') return fail("':' expected");
                    p++;
                    if (!value(v.members.back().second, depth + 1)) return false;
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == '}') { p++; return true; }
                    return fail("',' or '}' expected");
                }
            case '[':
                v.kind = ARRAY;
                p++;
                space();
                if (p < end && *p == ']') { p++; return true; }
                while (true) {
                    v.items.emplace_back();
                    if (!value(v.items.back(), depth + 1)) return false;
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == ']') { p++; return true; }
                    return fail("',' or ']' expected");
                }
            case '"': v.kind = STRING; return string(v.str);
            case 't': v.kind = BOOL; v.flag = true; return word("true");
            case 'f': v.kind = BOOL; return word("false");
            case 'n': return word("null");
            default: {
                const std::string t(p, (size_t)(end - p < 64 ? end - p : 64)); // strtod needs a terminator
                char *e = nullptr;
                v.num = strtod(t.c_str(), &e);
                if (e == t.c_str() || !std::isfinite(v.num)) return fail("number expected");
                v.kind = NUMBER;
                p += e - t.c_str();
                return true;
            }
            }
        }
    };
};
