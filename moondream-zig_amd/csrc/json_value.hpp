// A JSON reader for model folders (config.json, the header of a safetensors file).  Host code only.
#pragma once
#include <cmath>
#include <cstdint>
#include <cstdlib>
#include <cstring>
#include <string>
#include <utility>
#include <vector>

struct Json {
    enum Type { NIL, BOOL, NUMBER, STRING, ARRAY, OBJECT } type = NIL;
    bool b = false;
    double num = 0.0;
    std::string str;
    std::vector<Json> items;                            // ARRAY
    std::vector<std::pair<std::string, Json>> members;  // OBJECT

    const Json *find(const char *key) const {
        if (type == OBJECT)
            for (const auto &m : members)
                if (m.first == key) return &m.second;
        return nullptr;
    }
    bool is_size() const { return type == NUMBER && num >= 0 && num <= 9007199254740992.0 && num == std::floor(num); }

    static bool parse(const char *text, size_t len, Json *out, std::string *err) {
        Reader r{text, text + len, 0};
        if (!r.value(out) || (r.space(), r.p != r.end)) {
            *err = "not JSON near byte " + std::to_string(r.p - text);
            return false;
        }
        return true;
    }

  private:
    struct Reader {
        const char *p, *end;
        int depth;
        void space() {
            while (p < end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) p++;
        }
        bool word(const char *w) {
            const size_t n = strlen(w);
            if (size_t(end - p) < n || memcmp(p, w, n)) return false;
            p += n;
            return true;
        }
        bool hex4(uint32_t *v) {
            if (end - p < 4) return false;
            *v = 0;
            for (int i = 0; i < 4; i++, p++) {
                const char c = *p;
                *v = *v * 16 + (c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : 0x10000);
                if (*v > 0xffff) return false;
            }
            return true;
        }
        bool string(std::string *s) {
            if (p >= end || *p != '"') return false;
            for (p++; p < end && *p != '"';) {
                if (*p != '\\') {
                    s->push_back(*p++);
                    continue;
                }
                if (++p >= end) return false;
                const char c = *p++;
                const char *from = "\"\\/bfnrt", *to = "\"\\/\b\f\n\r\t", *at = strchr(from, c);
                if (at && c) {
                    s->push_back(to[at - from]);
                    continue;
                }
                uint32_t u, lo;
                if (c != 'u' || !hex4(&u)) return false;
                if (u >= 0xd800 && u < 0xdc00) { // the first half of a pair
                    if (!word("\\u") || !hex4(&lo) || lo < 0xdc00 || lo > 0xdfff) return false;
                    u = 0x10000 + ((u - 0xd800) << 10) + (lo - 0xdc00);
                }
                if (u < 0x80) s->push_back((char)u);
                else {
                    const int more = u < 0x800 ? 1 : u < 0x10000 ? 2 : 3;
                    s->push_back((char)((more == 1 ? 0xc0 : more == 2 ? 0xe0 : 0xf0) | (u >> (6 * more))));
                    for (int i = more - 1; i >= 0; i--) s->push_back((char)(0x80 | ((u >> (6 * i)) & 0x3f)));
                }
            }
            if (p >= end) return false;
            p++;
            return true;
        }
        bool value(Json *v) {
            space();
            if (p >= end || ++depth > 64) return false;
            bool ok = true;
            if (*p == '{' || *p == '[') {
                const bool object = *p == '{';
                const char close = object ? '}' : ']';
                v->type = object ? OBJECT : ARRAY;
                p++;
                space();
                if (p < end && *p == close) p++;
                else
                    for (;;) {
                        space();
                        Json *slot;
                        if (object) {
                            std::string key;
                            if (!string(&key)) return false;
                            space();
                            if (p >= end || *p++ != ':') return false;
                            v->members.emplace_back(std::move(key), Json());
                            slot = &v->members.back().second;
                        } else {
                            v->items.emplace_back();
                            slot = &v->items.back();
                        }
                        if (!value(slot)) return false;
                        space();
                        if (p >= end) return false;
                        if (*p == close) {
                            p++;
                            break;
                        }
                        if (*p++ != ',') return false;
                    }
            } else if (*p == '"') {
                v->type = STRING;
                ok = string(&v->str);
            } else if (word("true")) {
                v->type = BOOL;
                v->b = true;
            } else if (word("false")) v->type = BOOL;
            else if (word("null")) v->type = NIL;
            else {
                const char *q = p;
                while (q < end && strchr("+-0123456789.eE", *q) && *q) q++;
                const std::string n(p, q);
                char *stop = nullptr;
                v->type = NUMBER;
                v->num = strtod(n.c_str(), &stop);
                ok = !n.empty() && *stop == 0;
                p = q;
            }
            depth--;
            return ok;
        }
    };
};
