// A small JSON reader for the files a model folder holds (config.json, the header of a safetensors file).
#pragma once

#include <cstdint>
#include <cstdlib>
#include <string>
#include <utility>
#include <vector>

struct RmiJson {
    enum Type { kNull, kBool, kNumber, kString, kArray, kObject } type = kNull;
    double number = 0;
    bool boolean = false;
    std::string text;
    std::vector<RmiJson> items;
    std::vector<std::pair<std::string, RmiJson>> members;

    const RmiJson *get(const char *key) const {  // nullptr when absent or not an object
        for (const auto &m : members)
            if (m.first == key) return &m.second;
        return nullptr;
    }
    bool is_null() const { return type == kNull; }

    // the whole text as one value; on failure false and a message
    static bool parse(const char *p, size_t n, RmiJson *out, std::string *error) {
        Reader r{p, p + n, error};
        r.space();
        if (!r.value(out, 0)) return false;
        r.space();
        return r.p == r.end || r.fail("text behind the JSON value");
    }

  private:
    struct Reader {
        const char *p, *end;
        std::string *error;
        bool fail(const char *what) {
            if (error) *error = what;
            return false;
        }
        void space() {
            while (p < end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) p++;
        }
        bool word(const char *w) {
            const char *q = p;
            for (; *w; w++, q++)
                if (q >= end || *q != *w) return false;
            p = q;
            return true;
        }
        static void utf8(std::string *s, uint32_t c) {
            if (c < 0x80) {
                s->push_back(char(c));
            } else if (c < 0x800) {
                s->push_back(char(0xc0 | (c >> 6)));
                s->push_back(char(0x80 | (c & 63)));
            } else if (c < 0x10000) {
                s->push_back(char(0xe0 | (c >> 12)));
                s->push_back(char(0x80 | ((c >> 6) & 63)));
                s->push_back(char(0x80 | (c & 63)));
            } else {
                s->push_back(char(0xf0 | (c >> 18)));
                s->push_back(char(0x80 | ((c >> 12) & 63)));
                s->push_back(char(0x80 | ((c >> 6) & 63)));
                s->push_back(char(0x80 | (c & 63)));
            }
        }
        bool hex4(uint32_t *c) {
            *c = 0;
            for (int i = 0; i < 4; i++, p++) {
                if (p >= end) return false;
                const char ch = *p;
                const int v = ch >= '0' && ch <= '9' ? ch - '0' : ch >= 'a' && ch <= 'f' ? ch - 'a' + 10 : ch >= 'A' && ch <= 'F' ? ch - 'A' + 10 : -1;
                if (v < 0) return false;
                *c = *c * 16 + uint32_t(v);
            }
            return true;
        }
        bool string(std::string *s) {
            if (p >= end || *p != '"') return fail("expected a string");
            for (p++; p < end && *p != '"';) {
                if (*p != '\\') {
                    s->push_back(*p++);
                    continue;
                }
                if (++p >= end) break;
                const char c = *p++;
                switch (c) {
                    case 'n': s->push_back('\n'); break;
                    case 't': s->push_back('\t'); break;
                    case 'r': s->push_back('\r'); break;
                    case 'b': s->push_back('\b'); break;
                    case 'f': s->push_back('\f'); break;
                    case 'u': {
                        uint32_t u, lo;
                        if (!hex4(&u)) return fail("bad \\u escape");
                        if (u >= 0xd800 && u < 0xdc00 && end - p >= 6 && p[0] == '\\' && p[1] == 'u') {
                            p += 2;
                            if (!hex4(&lo)) return fail("bad \\u escape");
                            u = 0x10000 + ((u - 0xd800) << 10) + (lo - 0xdc00);
                        }
                        utf8(s, u);
                        break;
                    }
                    default: s->push_back(c);
                }
            }
            if (p >= end) return fail("unterminated string");
            p++;
            return true;
        }
        bool value(RmiJson *out, int depth) {
            if (depth > 64) return fail("nested too deep");
            if (p >= end) return fail("unexpected end");
            if (*p == '{') {
                out->type = kObject;
                p++;
                space();
                if (p < end && *p == '}') return ++p, true;
                while (true) {
                    std::string key;
                    space();
                    if (!string(&key)) return false;
                    space();
                    if (p >= end || *p != ':') return fail("expected ':'");
                    p++;
                    space();
                    out->members.emplace_back(std::move(key), RmiJson());
                    if (!value(&out->members.back().second, depth + 1)) return false;
                    space();
                    if (p < end && *p == ',') {
                        p++;
                        continue;
                    }
                    if (p < end && *p == '}') return ++p, true;
                    return fail("expected ',' or '}'");
                }
            }
            if (*p == '[') {
                out->type = kArray;
                p++;
                space();
                if (p < end && *p == ']') return ++p, true;
                while (true) {
                    space();
                    out->items.emplace_back();
                    if (!value(&out->items.back(), depth + 1)) return false;
                    space();
                    if (p < end && *p == ',') {
                        p++;
                        continue;
                    }
                    if (p < end && *p == ']') return ++p, true;
                    return fail("expected ',' or ']'");
                }
            }
            if (*p == '"') {
                out->type = kString;
                return string(&out->text);
            }
            if (word("true")) return out->type = kBool, out->boolean = true, true;
            if (word("false")) return out->type = kBool, true;
            if (word("null")) return true;
            const char *q = p;
            while (q < end && ((*q >= '0' && *q <= '9') || *q == '-' || *q == '+' || *q == '.' || *q == 'e' || *q == 'E')) q++;
            if (q == p || q - p > 60) return fail("expected a value");
            const std::string num(p, q);
            char *stop = nullptr;
            out->type = kNumber;
            out->number = strtod(num.c_str(), &stop);
            if (*stop) return fail("bad number");
            p = q;
            return true;
        }
    };
};
