/*
 * tk_json.h — a JSON document as a tree: what the decision parser (cJSON's reading of an LLM's answer) and the model configuration and
 * safetensors readers need.  Host only.
 */
#ifndef TK_JSON_H
#define TK_JSON_H

#include <stdlib.h>
#include <string.h>

#include <string>
#include <utility>
#include <vector>

namespace tk_json {

struct JVal {
    enum Kind { JNULL, JBOOL, JNUM, JSTR, JARR, JOBJ } kind = JNULL;
    bool b = false;
    double num = 0.0;
    std::string str;
    std::vector<JVal> arr;
    std::vector<std::pair<std::string, JVal>> obj;
    const JVal* get(const char* key) const { /* cJSON_GetObjectItemCaseSensitive: first member of that name */
        if (kind != JOBJ) return nullptr;
        for (const auto& kv : obj)
            if (kv.first == key) return &kv.second;
        return nullptr;
    }
};

struct JParser {
    const char* p;
    const char* end;
    int depth = 0;
    void ws() { while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) ++p; }
    static void utf8(std::string& s, unsigned cp) {
        if (cp < 0x80) s += (char)cp;
        else if (cp < 0x800) { s += (char)(0xC0 | (cp >> 6)); s += (char)(0x80 | (cp & 63)); }
        else if (cp < 0x10000) { s += (char)(0xE0 | (cp >> 12)); s += (char)(0x80 | ((cp >> 6) & 63)); s += (char)(0x80 | (cp & 63)); }
        else { s += (char)(0xF0 | (cp >> 18)); s += (char)(0x80 | ((cp >> 12) & 63)); s += (char)(0x80 | ((cp >> 6) & 63)); s += (char)(0x80 | (cp & 63)); }
    }
    bool hex4(unsigned* v) {
        if (end - p < 4) return false;
        unsigned x = 0;
        for (int i = 0; i < 4; ++i) {
            char c = p[i];
            x <<= 4;
            if (c >= '0' && c <= '9') x |= (unsigned)(c - '0');
            else if (c >= 'a' && c <= 'f') x |= (unsigned)(c - 'a' + 10);
            else if (c >= 'A' && c <= 'F') x |= (unsigned)(c - 'A' + 10);
            else return false;
        }
        p += 4;
        *v = x;
        return true;
    }
    bool string(std::string* out) {
        if (p >= end || *p != '"') return false;
        ++p;
        out->clear();
        while (p < end && *p != '"') {
            if ((unsigned char)*p < 0x20) return false;
            if (*p != '\\') { *out += *p++; continue; }
            if (++p >= end) return false;
            switch (*p++) {
                case '"': *out += '"'; break;
                case '\\': *out += '\\'; break;
                case '/': *out += '/'; break;
                case 'b': *out += '\b'; break;
                case 'f': *out += '\f'; break;
                case 'n': *out += '\n'; break;
                case 'r': *out += '\r'; break;
                case 't': *out += '\t'; break;
                case 'u': {
                    unsigned cp;
                    if (!hex4(&cp)) return false;
                    if (cp >= 0xD800 && cp <= 0xDBFF) { /* surrogate pair */
                        unsigned lo;
                        if (end - p < 6 || p[0] != '\\' || p[1] != 'u') return false;
                        p += 2;
                        if (!hex4(&lo) || lo < 0xDC00 || lo > 0xDFFF) return false;
                        cp = 0x10000 + ((cp - 0xD800) << 10) + (lo - 0xDC00);
                    } else if (cp >= 0xDC00 && cp <= 0xDFFF) return false;
                    utf8(*out, cp);
                    break;
                }
                default: return false;
            }
        }
        if (p >= end) return false;
        ++p;
        return true;
    }
    bool value(JVal* v) {
        if (++depth > 64) return false;
        ws();
        if (p >= end) return false;
        bool ok = false;
        if (*p == '{') {
            ++p;
            v->kind = JVal::JOBJ;
            ws();
            if (p < end && *p == '}') { ++p; ok = true; }
            else
                for (;;) {
                    ws();
                    std::string key;
                    if (!string(&key)) break;
                    ws();
                    if (p >= end || *p != ':') break;
                    ++p;
                    JVal child;
                    if (!value(&child)) break;
                    v->obj.emplace_back(std::move(key), std::move(child));
                    ws();
                    if (p < end && *p == ',') { ++p; continue; }
                    if (p < end && *p == '}') { ++p; ok = true; }
                    break;
                }
        } else if (*p == '[') {
            ++p;
            v->kind = JVal::JARR;
            ws();
            if (p < end && *p == ']') { ++p; ok = true; }
            else
                for (;;) {
                    JVal child;
                    if (!value(&child)) break;
                    v->arr.push_back(std::move(child));
                    ws();
                    if (p < end && *p == ',') { ++p; continue; }
                    if (p < end && *p == ']') { ++p; ok = true; }
                    break;
                }
        } else if (*p == '"') {
            v->kind = JVal::JSTR;
            ok = string(&v->str);
        } else if (end - p >= 4 && !strncmp(p, "true", 4)) { v->kind = JVal::JBOOL; v->b = true; p += 4; ok = true; }
        else if (end - p >= 5 && !strncmp(p, "false", 5)) { v->kind = JVal::JBOOL; v->b = false; p += 5; ok = true; }
        else if (end - p >= 4 && !strncmp(p, "null", 4)) { v->kind = JVal::JNULL; p += 4; ok = true; }
        else if (*p == '-' || (*p >= '0' && *p <= '9')) {
            char tmp[64];
            size_t n = 0;
            while (p + n < end && n < sizeof tmp - 1 && (strchr("+-0123456789.eE", p[n]) != nullptr) && p[n] != 0) ++n;
            memcpy(tmp, p, n);
            tmp[n] = 0;
            char* e = nullptr;
            v->num = strtod(tmp, &e);
            if (e != tmp) { v->kind = JVal::JNUM; p += (e - tmp); ok = true; }
        }
        --depth;
        return ok;
    }
};

} // namespace tk_json

#endif
