// json.hpp -- a small JSON reader (RFC 8259 subset: no surrogate pairs) for model configurations, safetensors headers and the
// trace runner's steps.
#pragma once

#include <cstdint>
#include <cstdlib>
#include <cstring>
#include <map>
#include <string>
#include <vector>

namespace bitnet_host {

struct Json {
    enum Kind { Null, Bool, Number, String, Array, Object } kind = Null;
    bool b = false;
    double num = 0.0;
    std::string str;
    std::vector<Json> items;
    std::vector<std::pair<std::string, Json>> members;

    const Json *find(const std::string &key) const {
        for (const auto &m : members)
            if (m.first == key) return &m.second;
        return nullptr;
    }
    bool is_null() const { return kind == Null; }

    static bool parse(const char *text, size_t len, Json &out, std::string &err) {
        Reader r{text, text + len, 0};
        if (!r.value(out)) {
            err = "JSON: " + (r.err.empty() ? std::string("syntax error") : r.err) + " at byte " + std::to_string(r.p - text);
            return false;
        }
        r.space();
        if (r.p != r.end) {
            err = "JSON: text after the value";
            return false;
        }
        return true;
    }

  private:
    struct Reader {
        const char *p, *end;
        int depth;
        std::string err;
        void space() {
            while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) ++p;
        }
        bool lit(const char *s) {
            const size_t n = strlen(s);
            if ((size_t)(end - p) < n || memcmp(p, s, n) != 0) return false;
            p += n;
            return true;
        }
        bool string(std::string &out) {
            if (p >= end || *p != '"') return false;
            for (++p; p < end && *p != '"'; ++p) {
                if (*p != '\\') {
                    out.push_back(*p);
                    continue;
                }
                if (++p >= end) return false;
                switch (*p) {
                    case 'n': out.push_back('\n'); break;
                    case 't': out.push_back('\t'); break;
                    case 'r': out.push_back('\r'); break;
                    case 'b': out.push_back('\b'); break;
                    case 'f': out.push_back('\f'); break;
                    case 'u': {
                        if (end - p < 5) return false;
                        const unsigned u = (unsigned)strtoul(std::string(p + 1, 4).c_str(), nullptr, 16);
                        p += 4;
                        if (u < 0x80) {
                            out.push_back((char)u);
                        } else if (u < 0x800) {
                            out.push_back((char)(0xc0 | u >> 6));
                            out.push_back((char)(0x80 | (u & 63)));
                        } else {
                            out.push_back((char)(0xe0 | u >> 12));
                            out.push_back((char)(0x80 | (u >> 6 & 63)));
                            out.push_back((char)(0x80 | (u & 63)));
                        }
                        break;
                    }
                    default: out.push_back(*p);
                }
            }
            if (p >= end) return false;
            ++p;
            return true;
        }
        bool value(Json &v) {
            space();
            if (p >= end || depth > 64) return false;
            if (*p == '{') {
                ++depth, ++p, v.kind = Object;
                space();
                if (p < end && *p == '}') return --depth, ++p, true;
                for (;;) {
                    space();
                    std::string key;
                    if (!string(key)) return false;
                    space();
                    if (p >= end || *p++ != ':') return false;
                    v.members.emplace_back(key, Json());
                    if (!value(v.members.back().second)) return false;
                    space();
                    if (p >= end) return false;
                    if (*p == '}') return --depth, ++p, true;
                    if (*p++ != ',') return false;
                }
            }
            if (*p == '[') {
                ++depth, ++p, v.kind = Array;
                space();
                if (p < end && *p == ']') return --depth, ++p, true;
                for (;;) {
                    v.items.emplace_back();
                    if (!value(v.items.back())) return false;
                    space();
                    if (p >= end) return false;
                    if (*p == ']') return --depth, ++p, true;
                    if (*p++ != ',') return false;
                }
            }
            if (*p == '"') return v.kind = String, string(v.str);
            if (lit("true")) return v.kind = Bool, v.b = true;
            if (lit("false")) return v.kind = Bool, true;
            if (lit("null")) return true;
            std::string n;
            while (p < end && (strchr("+-.eE", *p) || (*p >= '0' && *p <= '9')) && *p) n.push_back(*p++);
            char *e = nullptr;
            v.num = strtod(n.c_str(), &e);
            v.kind = Number;
            return !n.empty() && *e == 0;
        }
    };
};

// Typed reads that remember the first problem ("layers[2].mixer.dim: missing").
struct JsonView {
    const Json *j;
    std::string path;
    std::string *err;
    void bad(const std::string &key, const char *what) const {
        if (err->empty()) *err = "config: " + path + key + ": " + what;
    }
    bool has(const std::string &key) const {
        const Json *v = j ? j->find(key) : nullptr;
        return v && !v->is_null();
    }
    JsonView at(const std::string &key) const {
        const Json *v = j ? j->find(key) : nullptr;
        if (!v || v->kind != Json::Object) bad(key, "missing object"), v = nullptr;
        return {v, path + key + ".", err};
    }
    double number(const std::string &key) const {
        const Json *v = j ? j->find(key) : nullptr;
        if (!v || v->kind != Json::Number) return bad(key, "missing number"), 0.0;
        return v->num;
    }
    int integer(const std::string &key, int lo = 1, int hi = 1 << 28) const {
        const double v = number(key);
        if (v != (double)(int64_t)v || v < lo || v > hi) return bad(key, "not an integer in range"), lo;
        return (int)v;
    }
    std::string text(const std::string &key) const {
        const Json *v = j ? j->find(key) : nullptr;
        if (!v || v->kind != Json::String) return bad(key, "missing string"), std::string();
        return v->str;
    }
    std::vector<double> numbers(const std::string &key) const {
        std::vector<double> out;
        const Json *v = j ? j->find(key) : nullptr;
        if (!v || v->kind != Json::Array) return bad(key, "missing array"), out;
        for (const Json &i : v->items) {
            if (i.kind != Json::Number) bad(key, "not an array of numbers");
            out.push_back(i.num);
        }
        return out;
    }
};

}  // namespace bitnet_host
