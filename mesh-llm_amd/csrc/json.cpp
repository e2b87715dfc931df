// See json.hpp.  Host-only; every read is bounded by the text's length.
#include "json.hpp"

#include <cerrno>
#include <cmath>
#include <cstdlib>
#include <cstring>

namespace mesh {

namespace {

constexpr int MAX_DEPTH = 64;

struct Parser {
    const char *p, *end, *begin;
    std::string &err;

    bool bad(const char *what) {
        if (err.empty()) err = std::string(what) + " at byte " + std::to_string(p - begin);
        return false;
    }
    void space() { while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) ++p; }
    bool take(char c) {
        if (p < end && *p == c) { ++p; return true; }
        return false;
    }
    bool word(const char *w) {
        const size_t n = strlen(w);
        if ((size_t)(end - p) < n || memcmp(p, w, n)) return bad("unknown word");
        p += n;
        return true;
    }
    static void utf8(std::string &s, uint32_t c) {
        if (c < 0x80) s += (char)c;
        else if (c < 0x800) { s += (char)(0xC0 | (c >> 6)); s += (char)(0x80 | (c & 63)); }
        else if (c < 0x10000) { s += (char)(0xE0 | (c >> 12)); s += (char)(0x80 | ((c >> 6) & 63)); s += (char)(0x80 | (c & 63)); }
        else { s += (char)(0xF0 | (c >> 18)); s += (char)(0x80 | ((c >> 12) & 63)); s += (char)(0x80 | ((c >> 6) & 63)); s += (char)(0x80 | (c & 63)); }
    }
    bool hex4(uint32_t &v) {
        if (end - p < 4) return bad("short escape");
        v = 0;
        for (int i = 0; i < 4; ++i, ++p) {
            const char c = *p;
            const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
            if (d < 0) return bad("bad escape");
            v = v * 16 + (uint32_t)d;
        }
        return true;
    }
    bool string(std::string &s) {
        if (!take('"')) return bad("string expected");
        for (;;) {
            if (p >= end) return bad("unterminated string");
            const char c = *p++;
            if (c == '"') return true;
            if ((unsigned char)c < 0x20) return bad("control character in a string");
            if (c != '\\') { s += c; continue; }
            if (p >= end) return bad("unterminated string");
            const char e = *p++;
            switch (e) {
                case '"': case '\\': case '/': s += e; break;
                case 'b': s += '\b'; break;
                case 'f': s += '\f'; break;
                case 'n': s += '\n'; break;
                case 'r': s += '\r'; break;
                case 't': s += '\t'; break;
                case 'u': {
                    uint32_t v = 0, lo = 0;
                    if (!hex4(v)) return false;
                    if (v >= 0xD800 && v < 0xDC00) {
                        if (!take('\\') || !take('u') || !hex4(lo) || lo < 0xDC00 || lo > 0xDFFF) return bad("bad surrogate pair");
                        v = 0x10000 + ((v - 0xD800) << 10) + (lo - 0xDC00);
                    }
                    utf8(s, v);
                    break;
                }
                default: return bad("bad escape");
            }
        }
    }
    bool number(double &out) {
        const char *q = p;
        if (q < end && *q == '-') ++q;
        const char *digits = q;
        while (q < end && *q >= '0' && *q <= '9') ++q;
        if (q == digits) return bad("value expected");
        if (q < end && *q == '.') { ++q; while (q < end && *q >= '0' && *q <= '9') ++q; }
        if (q < end && (*q == 'e' || *q == 'E')) {
            ++q;
            if (q < end && (*q == '+' || *q == '-')) ++q;
            while (q < end && *q >= '0' && *q <= '9') ++q;
        }
        const std::string t(p, q);
        char *stop = nullptr;
        out = strtod(t.c_str(), &stop);
        if (*stop || !std::isfinite(out)) return bad("bad number");
        p = q;
        return true;
    }
    bool value(JsonValue &v, int depth) {
        if (depth > MAX_DEPTH) return bad("nested too deep");
        space();
        if (p >= end) return bad("value expected");
        if (*p == '{') {
            ++p;
            v.kind = JsonValue::OBJECT;
            space();
            if (take('}')) return true;
            for (;;) {
                std::string key;
                space();
                if (!string(key)) return false;
                space();
                if (!take(':')) return bad("':' expected");
                if (!value(v.fields[key], depth + 1)) return false;
                space();
                if (take('}')) return true;
                if (!take(',')) return bad("',' expected");
            }
        }
        if (*p == '[') {
            ++p;
            v.kind = JsonValue::ARRAY;
            space();
            if (take(']')) return true;
            for (;;) {
                v.items.emplace_back();
                if (!value(v.items.back(), depth + 1)) return false;
                space();
                if (take(']')) return true;
                if (!take(',')) return bad("',' expected");
            }
        }
        if (*p == '"') { v.kind = JsonValue::STRING; return string(v.str); }
        if (*p == 't') { v.kind = JsonValue::BOOL; v.b = true; return word("true"); }
        if (*p == 'f') { v.kind = JsonValue::BOOL; return word("false"); }
        if (*p == 'n') return word("null");
        v.kind = JsonValue::NUMBER;
        return number(v.num);
    }
};

}  // namespace

const JsonValue *JsonValue::get(const char *name) const {
    if (kind != OBJECT) return nullptr;
    auto it = fields.find(name);
    return it == fields.end() ? nullptr : &it->second;
}

bool JsonValue::as_count(uint64_t max, uint64_t &out) const {
    if (kind != NUMBER || num < 0 || num > (double)max || num != std::floor(num)) return false;
    out = (uint64_t)num;
    return true;
}

bool json_parse(const char *text, size_t n, JsonValue &out, std::string &err) {
    err.clear();
    Parser ps{text, text + n, text, err};
    if (!ps.value(out, 0)) return false;
    ps.space();
    return ps.p == ps.end || ps.bad("text after the value");
}

}  // namespace mesh
