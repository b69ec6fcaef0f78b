// A JSON reader just large enough for a safetensors header, model.safetensors.index.json and a model's config.json.
#pragma once
#include <cstdint>
#include <cstdlib>
#include <cstring>
#include <string>
#include <utility>
#include <vector>

namespace mynn {

struct Json {
    enum Kind { NUL, NUM, STR, ARR, OBJ, BOOL } kind = NUL;
    double num = 0;
    std::string str;
    std::vector<Json> arr;
    std::vector<std::pair<std::string, Json>> obj;  // insertion order
    const Json *get(const char *key) const {
        for (auto &kv : obj)
            if (kv.first == key) return &kv.second;
        return nullptr;
    }
};
struct JsonParser {
    const char *p, *end;  // [p, end) is followed by a NUL (parse_json copies the text), so strtod cannot run past it
    bool ok = true;
    int depth = 0;
    static constexpr int kMaxDepth = 32;  // a safetensors header nests 3 deep, a config.json a little deeper
    void ws() {
        while (p < end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) p++;
    }
    bool eat(char c) {
        ws();
        if (p < end && *p == c) {
            p++;
            return true;
        }
        return false;
    }
    std::string string() {
        std::string s;
        if (!eat('"')) {
            ok = false;
            return s;
        }
        while (p < end && *p != '"') {
            if (*p == '\\' && p + 1 < end) {
                p++;
                switch (*p) {
                case 'n': s += '\n'; break;
                case 't': s += '\t'; break;
                case 'u':  // tensor names are ASCII; keep the escape verbatim
                    s += "\\u";
                    break;
                default: s += *p;
                }
                p++;
            } else s += *p++;
        }
        if (p >= end) ok = false;
        else p++;
        return s;
    }
    Json value() {
        Json j;
        ws();
        if (p >= end) {
            ok = false;
            return j;
        }
        if ((*p == '{' || *p == '[') && ++depth > kMaxDepth) {
            ok = false;
            return j;
        }
        if (*p == '{') {
            p++;
            j.kind = Json::OBJ;
            if (eat('}')) {
                depth--;
                return j;
            }
            do {
                std::string k = string();
                if (!ok || !eat(':')) {
                    ok = false;
                    return j;
                }
                j.obj.emplace_back(std::move(k), value());
                if (!ok) return j;
            } while (eat(','));
            if (!eat('}')) ok = false;
            depth--;
        } else if (*p == '[') {
            p++;
            j.kind = Json::ARR;
            if (eat(']')) {
                depth--;
                return j;
            }
            do {
                j.arr.push_back(value());
                if (!ok) return j;
            } while (eat(','));
            if (!eat(']')) ok = false;
            depth--;
        } else if (*p == '"') {
            j.kind = Json::STR;
            j.str = string();
        } else if ((end - p >= 4 && (!strncmp(p, "true", 4) || !strncmp(p, "null", 4))) || (end - p >= 5 && !strncmp(p, "false", 5))) {
            j.kind = *p == 'n' ? Json::NUL : Json::BOOL;
            j.num = *p == 't';
            p += *p == 'f' ? 5 : 4;
        } else {
            char *q = nullptr;
            j.kind = Json::NUM;
            j.num = strtod(p, &q);
            if (q == p || q > end) ok = false;
            p = q;
        }
        return j;
    }
};
inline bool parse_json(const char *data, size_t n, Json &out) {
    const std::string text(data, n);  // NUL-terminated copy: the mapped header may end exactly at the end of the file
    JsonParser ps{text.c_str(), text.c_str() + n};
    out = ps.value();
    return ps.ok;
}

// a JSON number that must be a non-negative integer below 2^53 (offsets, extents): false otherwise
inline bool as_size(const Json &j, size_t *out) {
    if (j.kind != Json::NUM || !(j.num >= 0.0) || j.num > 9007199254740992.0 || j.num != (double)(uint64_t)j.num) return false;
    *out = (size_t)j.num;
    return true;
}

}  // namespace mynn
