// JSON text: a cursor for the safetensors header and a small value tree for config.json.  Host code only.
#pragma once
#include <stdint.h>
#include <stdlib.h>
#include <string>
#include <utility>
#include <vector>

namespace lmhip {

// A cursor over JSON text.
struct Json {
    const char *p, *end;
    void ws() { while (p < end && (*p == ' ' || *p == '\n' || *p == '\r' || *p == '\t')) p++; }
    bool eat(char c) { ws(); if (p < end && *p == c) { p++; return true; } return false; }
    bool string(std::string &out)
    {
        ws();
        if (p >= end || *p != '"') return false;
        out.clear();
        for (p++; p < end && *p != '"'; p++) {
            if (*p == '\\' && p + 1 < end) p++;
            out.push_back(*p);
        }
        if (p >= end) return false;
        p++;
        return true;
    }
    bool number(uint64_t &v)
    {
        ws();
        if (p >= end || *p < '0' || *p > '9') return false;
        v = 0;
        while (p < end && *p >= '0' && *p <= '9') v = v * 10 + (uint64_t)(*p++ - '0');
        return true;
    }
    bool skip()                    // any value
    {
        ws();
        if (p >= end) return false;
        if (*p == '"') { std::string s; return string(s); }
        if (*p == '{' || *p == '[') {
            const char open = *p, close = open == '{' ? '}' : ']';
            p++;
            if (eat(close)) return true;
            do {
                if (open == '{') { std::string k; if (!string(k) || !eat(':')) return false; }
                if (!skip()) return false;
            } while (eat(','));
            return eat(close);
        }
        while (p < end && *p != ',' && *p != '}' && *p != ']') p++;
        return true;
    }
};

// A parsed value.  Members keep the order of the text; a lookup of a missing member gives the null value.
struct JsonValue {
    enum Kind { NUL, BOOL, NUMBER, STRING, ARRAY, OBJECT } kind = NUL;
    double num = 0.0;
    std::string str;
    std::vector<JsonValue> items;
    std::vector<std::pair<std::string, JsonValue>> members;

    const JsonValue &operator[](const char *key) const
    {
        static const JsonValue none;
        for (const auto &m : members) if (m.first == key) return m.second;
        return none;
    }
    bool is_null() const { return kind == NUL; }
    bool is_number() const { return kind == NUMBER; }

    static bool parse(Json &j, JsonValue &v, int depth = 0)
    {
        j.ws();
        if (j.p >= j.end || depth > 64) return false;
        if (*j.p == '"') { v.kind = STRING; return j.string(v.str); }
        if (*j.p == '[') {
            v.kind = ARRAY; j.p++;
            if (j.eat(']')) return true;
            do { v.items.emplace_back(); if (!parse(j, v.items.back(), depth + 1)) return false; } while (j.eat(','));
            return j.eat(']');
        }
        if (*j.p == '{') {
            v.kind = OBJECT; j.p++;
            if (j.eat('}')) return true;
            do {
                v.members.emplace_back();
                if (!j.string(v.members.back().first) || !j.eat(':') || !parse(j, v.members.back().second, depth + 1)) return false;
            } while (j.eat(','));
            return j.eat('}');
        }
        std::string word;
        while (j.p < j.end && *j.p != ',' && *j.p != '}' && *j.p != ']' && *j.p > ' ') word.push_back(*j.p++);
        if (word == "null") { v.kind = NUL; return true; }
        if (word == "true" || word == "false") { v.kind = BOOL; v.num = word == "true"; return true; }
        char *e = nullptr;
        v.kind = NUMBER; v.num = strtod(word.c_str(), &e);
        return !word.empty() && *e == 0;
    }
    static bool parse_text(const std::string &text, JsonValue &v)
    {
        Json j{text.data(), text.data() + text.size()};
        if (!parse(j, v)) return false;
        j.ws();
        return j.p == j.end;
    }
};

}  // namespace lmhip
