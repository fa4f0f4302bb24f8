// A small JSON reader (RFC 8259) for model configurations and safetensors headers.  Host only.
#pragma once
#include <cerrno>
#include <cstdint>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <string>
#include <utility>
#include <vector>

namespace jq {

struct Json {
    enum Kind { NUL, BOOL, NUMBER, STRING, ARRAY, OBJECT };
    Kind kind = NUL;
    bool b = false;
    double num = 0.0;
    std::string str;
    std::vector<Json> items;                            // ARRAY
    std::vector<std::pair<std::string, Json>> members;  // OBJECT, in file order

    const Json *find(const char *key) const {
        if (kind == OBJECT)
            for (const auto &m : members)
                if (m.first == key) return &m.second;
        return nullptr;
    }
};

struct JsonParser {
    const char *p, *end;
    const char *what = nullptr;
    static constexpr int MAX_DEPTH = 64;

    bool bad(const char *w) {
        if (!what) what = w;
        return false;
    }
    void space() {
        while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) p++;
    }
    bool word(const char *w) {
        const size_t n = strlen(w);
        if ((size_t)(end - p) < n || memcmp(p, w, n) != 0) return bad("unexpected character");
        p += n;
        return true;
    }
    static void utf8(unsigned c, std::string *s) {
        if (c < 0x80) {
            s->push_back((char)c);
        } else if (c < 0x800) {
            s->push_back((char)(0xC0 | c >> 6)), s->push_back((char)(0x80 | (c & 63)));
        } else if (c < 0x10000) {
            s->push_back((char)(0xE0 | c >> 12)), s->push_back((char)(0x80 | (c >> 6 & 63))), s->push_back((char)(0x80 | (c & 63)));
        } else {
            s->push_back((char)(0xF0 | c >> 18)), s->push_back((char)(0x80 | (c >> 12 & 63)));
            s->push_back((char)(0x80 | (c >> 6 & 63))), s->push_back((char)(0x80 | (c & 63)));
        }
    }
    bool hex4(unsigned *out) {
        if (end - p < 4) return bad("truncated \\u escape");
        unsigned v = 0;
        for (int i = 0; i < 4; i++) {
            const char c = *p++;
            const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
            if (d < 0) return bad("bad \\u escape");
            v = v * 16 + (unsigned)d;
        }
        *out = v;
        return true;
    }
    bool string(std::string *s) {
        if (p >= end || *p != '"') return bad("expected a string");
        for (p++; p < end && *p != '"';) {
            if (*p != '\\') {
                s->push_back(*p++);
                continue;
            }
            if (++p >= end) break;
            const char c = *p++;
            unsigned u, v;
            switch (c) {
            case '"': case '\\': case '/': s->push_back(c); break;
            case 'b': s->push_back('\b'); break;
            case 'f': s->push_back('\f'); break;
            case 'n': s->push_back('\n'); break;
            case 'r': s->push_back('\r'); break;
            case 't': s->push_back('\t'); break;
            case 'u':
                if (!hex4(&u)) return false;
                if (u >= 0xD800 && u < 0xDC00 && end - p >= 2 && p[0] == '\\' && p[1] == 'u') {
                    p += 2;
                    if (!hex4(&v)) return false;
                    u = 0x10000 + ((u - 0xD800) << 10) + ((v - 0xDC00) & 0x3FF);
                }
                utf8(u, s);
                break;
            default: return bad("bad escape in a string");
            }
        }
        if (p >= end) return bad("unterminated string");
        p++;
        return true;
    }
    bool value(Json *v, int depth) {
        if (depth > MAX_DEPTH) return bad("nested too deeply");
        space();
        if (p >= end) return bad("unexpected end");
        switch (*p) {
        case 'n': return word("null");
        case 't': v->kind = Json::BOOL, v->b = true; return word("true");
        case 'f': v->kind = Json::BOOL; return word("false");
        case '"': v->kind = Json::STRING; return string(&v->str);
        case '[':
            v->kind = Json::ARRAY;
            p++, space();
            if (p < end && *p == ']') { p++; return true; }
            for (;;) {
                v->items.emplace_back();
                if (!value(&v->items.back(), depth + 1)) return false;
                space();
                if (p < end && *p == ',') { p++; continue; }
                if (p < end && *p == ']') { p++; return true; }
                return bad("expected , or ]");
            }
        case '{':
            v->kind = Json::OBJECT;
            p++, space();
            if (p < end && *p == '}') { p++; return true; }
            for (;;) {
                space();
                std::string key;
                if (!string(&key)) return false;
                space();
                if (p >= end || *p != ':') return bad("expected :");
                p++;
                v->members.emplace_back(std::move(key), Json());
                if (!value(&v->members.back().second, depth + 1)) return false;
                space();
                if (p < end && *p == ',') { p++; continue; }
                if (p < end && *p == '}') { p++; return true; }
                return bad("expected , or }");
            }
        default: break;
        }
        std::string text;
        while (p < end && (strchr("+-.eE", *p) || (*p >= '0' && *p <= '9')) && *p) text.push_back(*p++);
        char *stop = nullptr;
        v->kind = Json::NUMBER;
        v->num = strtod(text.c_str(), &stop);
        return !text.empty() && *stop == 0 ? true : bad("unexpected character");
    }
};

inline bool json_parse(const char *text, size_t len, Json *out, std::string *err) {
    JsonParser ps{text, text + len};
    bool ok = ps.value(out, 0);
    if (ok) {
        ps.space();
        if (ps.p != ps.end) ok = ps.bad("text behind the value");
    }
    if (!ok) *err = std::string("JSON: ") + ps.what + " at byte " + std::to_string(ps.p - text);
    return ok;
}

inline bool json_read_file(const std::string &path, Json *out, std::string *err) {
    FILE *f = fopen(path.c_str(), "rb");
    if (!f) {
        *err = "cannot open `" + path + "`: " + strerror(errno);
        return false;
    }
    std::string text;
    char buf[65536];
    for (size_t n; (n = fread(buf, 1, sizeof buf, f)) > 0;) text.append(buf, n);
    fclose(f);
    if (json_parse(text.data(), text.size(), out, err)) return true;
    *err = path + ": " + *err;
    return false;
}

}  // namespace jq
