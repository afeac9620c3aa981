#include "json.h"

#include <cmath>
#include <cstdlib>
#include <cstring>

namespace itj {
namespace {

struct Reader {
    const char *p, *begin, *end;
    std::string err;
    bool bad(const char* what) {
        if (err.empty()) err = std::string(what) + " at byte " + std::to_string(p - begin);
        return false;
    }
    void space() {
        while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) p++;
    }
    bool word(const char* w) {
        const size_t n = strlen(w);
        if ((size_t)(end - p) < n || memcmp(p, w, n)) return bad("unknown word");
        p += n;
        return true;
    }
    bool hex4(unsigned* out) {
        if (end - p < 4) return bad("short \\u escape");
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
    static void utf8(unsigned c, std::string* s) {
        if (c < 0x80) s->push_back((char)c);
        else if (c < 0x800) { s->push_back((char)(0xc0 | c >> 6)); s->push_back((char)(0x80 | (c & 63))); }
        else if (c < 0x10000) { s->push_back((char)(0xe0 | c >> 12)); s->push_back((char)(0x80 | ((c >> 6) & 63))); s->push_back((char)(0x80 | (c & 63))); }
        else { s->push_back((char)(0xf0 | c >> 18)); s->push_back((char)(0x80 | ((c >> 12) & 63))); s->push_back((char)(0x80 | ((c >> 6) & 63))); s->push_back((char)(0x80 | (c & 63))); }
    }
    bool string(std::string* out) {
        if (p >= end || *p != '"') return bad("expected a string");
        p++;
        out->clear();
        while (p < end && *p != '"') {
            if ((unsigned char)*p < 0x20) return bad("control character in a string");
            if (*p != '\\') {
                out->push_back(*p++);
                continue;
            }
            if (++p >= end) return bad("unfinished escape");
            const char c = *p++;
            switch (c) {
                case '"': case '\\': case '/': out->push_back(c); break;
                case 'b': out->push_back('\b'); break;
                case 'f': out->push_back('\f'); break;
                case 'n': out->push_back('\n'); break;
                case 'r': out->push_back('\r'); break;
                case 't': out->push_back('\t'); break;
                case 'u': {
                    unsigned v = 0, lo = 0;
                    if (!hex4(&v)) return false;
                    if (v >= 0xd800 && v < 0xdc00) {
                        if (end - p < 2 || p[0] != '\\' || p[1] != 'u') return bad("lone surrogate");
                        p += 2;
                        if (!hex4(&lo)) return false;
                        if (lo < 0xdc00 || lo > 0xdfff) return bad("lone surrogate");
                        v = 0x10000 + ((v - 0xd800) << 10) + (lo - 0xdc00);
                    }
                    utf8(v, out);
                    break;
                }
                default: return bad("unknown escape");
            }
        }
        if (p >= end) return bad("unfinished string");
        p++;
        return true;
    }
    bool number(double* out) {
        const char* q = p;
        while (q < end && (strchr("+-.eE", *q) || (*q >= '0' && *q <= '9'))) q++;
        const std::string s(p, q);
        char* stop = nullptr;
        *out = strtod(s.c_str(), &stop);
        if (s.empty() || *stop || !std::isfinite(*out)) return bad("bad number");
        p = q;
        return true;
    }
    bool value(Value* v, int depth) {
        if (depth > 64) return bad("nested too deep");
        space();
        if (p >= end) return bad("unexpected end");
        switch (*p) {
            case 'n': return word("null");
            case 't': v->kind = Value::Bool; v->b = true; return word("true");
            case 'f': v->kind = Value::Bool; return word("false");
            case '"': v->kind = Value::String; return string(&v->str);
            case '[':
                v->kind = Value::Array;
                p++;
                space();
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
                v->kind = Value::Object;
                p++;
                space();
                if (p < end && *p == '}') { p++; return true; }
                for (;;) {
                    std::string key;
                    space();
                    if (!string(&key)) return false;
                    space();
                    if (p >= end || *p != ':') return bad("expected :");
                    p++;
                    Value item;
                    if (!value(&item, depth + 1)) return false;
                    if (!v->members.emplace(key, std::move(item)).second) return bad("a key appears twice");
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == '}') { p++; return true; }
                    return bad("expected , or }");
                }
            default: v->kind = Value::Number; return number(&v->num);
        }
    }
};

}  // namespace

bool parse(const char* text, size_t len, Value* out, std::string* err) {
    Reader r{text, text, text + len, {}};
    *out = Value{};
    bool ok = r.value(out, 0);
    if (ok) {
        r.space();
        if (r.p != r.end) ok = r.bad("text after the document");
    }
    if (!ok && err) *err = r.err;
    return ok;
}

}  // namespace itj
