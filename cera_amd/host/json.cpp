#include "json.h"

#include <charconv>
#include <cmath>
#include <cstdlib>

namespace cera {
namespace {

struct Parser {
    std::string_view s;
    size_t at = 0;
    std::string err;

    bool fail(const char* what) {
        if (err.empty()) err = std::string(what) + " at byte " + std::to_string(at);
        return false;
    }
    void space() {
        while (at < s.size() && (s[at] == ' ' || s[at] == '\t' || s[at] == '\n' || s[at] == '\r')) ++at;
    }
    bool word(const char* w, size_t n) {
        if (s.compare(at, n, w) != 0) return fail("unexpected character");
        at += n;
        return true;
    }
    static void utf8(std::string& o, uint32_t c) {
        if (c < 0x80) o += static_cast<char>(c);
        else if (c < 0x800) { o += static_cast<char>(0xC0 | (c >> 6)); o += static_cast<char>(0x80 | (c & 63)); }
        else if (c < 0x10000) { o += static_cast<char>(0xE0 | (c >> 12)); o += static_cast<char>(0x80 | ((c >> 6) & 63)); o += static_cast<char>(0x80 | (c & 63)); }
        else { o += static_cast<char>(0xF0 | (c >> 18)); o += static_cast<char>(0x80 | ((c >> 12) & 63)); o += static_cast<char>(0x80 | ((c >> 6) & 63)); o += static_cast<char>(0x80 | (c & 63)); }
    }
    bool hex4(uint32_t* v) {
        if (at + 4 > s.size()) return fail("short \\u escape");
        const auto r = std::from_chars(s.data() + at, s.data() + at + 4, *v, 16);
        if (r.ptr != s.data() + at + 4) return fail("bad \\u escape");
        at += 4;
        return true;
    }
    bool string(std::string* o) {
        ++at;   // opening quote
        for (;;) {
            if (at >= s.size()) return fail("unterminated string");
            const char c = s[at++];
            if (c == '"') return true;
            if (static_cast<unsigned char>(c) < 0x20) return fail("control character in string");
            if (c != '\\') { *o += c; continue; }
            if (at >= s.size()) return fail("unterminated string");
            const char e = s[at++];
            switch (e) {
                case '"': case '\\': case '/': *o += e; break;
                case 'b': *o += '\b'; break;
                case 'f': *o += '\f'; break;
                case 'n': *o += '\n'; break;
                case 'r': *o += '\r'; break;
                case 't': *o += '\t'; break;
                case 'u': {
                    uint32_t u, lo;
                    if (!hex4(&u)) return false;
                    if (u >= 0xD800 && u < 0xDC00) {
                        if (s.compare(at, 2, "\\u") != 0) return fail("lone surrogate");
                        at += 2;
                        if (!hex4(&lo)) return false;
                        if (lo < 0xDC00 || lo > 0xDFFF) return fail("lone surrogate");
                        u = 0x10000 + ((u - 0xD800) << 10) + (lo - 0xDC00);
                    }
                    utf8(*o, u);
                    break;
                }
                default: return fail("bad escape");
            }
        }
    }
    bool number(Json* o) {
        const size_t b = at;
        bool integral = true;
        if (at < s.size() && s[at] == '-') ++at;
        const size_t d0 = at;
        while (at < s.size() && s[at] >= '0' && s[at] <= '9') ++at;
        if (at == d0 || (s[d0] == '0' && at > d0 + 1)) return fail("bad number");
        if (at < s.size() && s[at] == '.') {
            integral = false;
            const size_t f0 = ++at;
            while (at < s.size() && s[at] >= '0' && s[at] <= '9') ++at;
            if (at == f0) return fail("bad number");
        }
        if (at < s.size() && (s[at] == 'e' || s[at] == 'E')) {
            integral = false;
            ++at;
            if (at < s.size() && (s[at] == '+' || s[at] == '-')) ++at;
            const size_t e0 = at;
            while (at < s.size() && s[at] >= '0' && s[at] <= '9') ++at;
            if (at == e0) return fail("bad number");
        }
        o->type = Json::Number;
        o->num = std::strtod(std::string(s.substr(b, at - b)).c_str(), nullptr);
        if (integral) {
            const auto r = std::from_chars(s.data() + b, s.data() + at, o->integer);
            o->is_int = r.ec == std::errc();
        } else if (std::fabs(o->num) < 9007199254740992.0 && o->num == std::floor(o->num)) {   // 1e3, 2.0
            o->is_int = true;
            o->integer = static_cast<int64_t>(o->num);
        }
        return true;
    }
    bool value(Json* o, int depth) {
        if (depth > 200) return fail("nested too deeply");
        space();
        if (at >= s.size()) return fail("unexpected end");
        switch (s[at]) {
            case '{':
                o->type = Json::Object;
                ++at;
                space();
                if (at < s.size() && s[at] == '}') { ++at; return true; }
                for (;;) {
                    space();
                    if (at >= s.size() || s[at] != '"') return fail("expected a key");
                    std::string k;
                    if (!string(&k)) return false;
                    space();
                    if (at >= s.size() || s[at++] != ':') return fail("expected ':'");
                    o->obj.emplace_back(std::move(k), Json());
                    if (!value(&o->obj.back().second, depth + 1)) return false;
                    space();
                    if (at < s.size() && s[at] == ',') { ++at; continue; }
                    if (at < s.size() && s[at] == '}') { ++at; return true; }
                    return fail("expected ',' or '}'");
                }
            case '[':
                o->type = Json::Array;
                ++at;
                space();
                if (at < s.size() && s[at] == ']') { ++at; return true; }
                for (;;) {
                    o->arr.emplace_back();
                    if (!value(&o->arr.back(), depth + 1)) return false;
                    space();
                    if (at < s.size() && s[at] == ',') { ++at; continue; }
                    if (at < s.size() && s[at] == ']') { ++at; return true; }
                    return fail("expected ',' or ']'");
                }
            case '"': o->type = Json::String; return string(&o->str);
            case 't': o->type = Json::Bool; o->b = true; return word("true", 4);
            case 'f': o->type = Json::Bool; return word("false", 5);
            case 'n': return word("null", 4);
            default: return number(o);
        }
    }
};

}  // namespace

bool Json::parse(std::string_view text, Json* out, std::string* err) {
    Parser p{text, 0, {}};
    *out = Json();
    bool ok = p.value(out, 0);
    if (ok) {
        p.space();
        if (p.at != text.size()) ok = p.fail("trailing characters");
    }
    if (!ok && err) *err = "JSON: " + p.err;
    return ok;
}

const Json* Json::find(const std::string& key) const {
    if (type != Object) return nullptr;
    for (const auto& kv : obj)
        if (kv.first == key) return &kv.second;
    return nullptr;
}

}  // namespace cera
