// A small JSON reader for configuration files: objects, arrays, strings, numbers, true / false / null.
#pragma once

#include <cstdlib>
#include <map>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

namespace cgh {

struct ConfigError : std::runtime_error {
    using std::runtime_error::runtime_error;
};

class Json {
  public:
    enum Kind { NIL, BOOL, NUMBER, STRING, ARRAY, OBJECT } kind = NIL;
    bool boolean = false;
    double number = 0.0;
    std::string string;
    std::vector<Json> array;
    std::map<std::string, Json> object;

    static Json parse(const std::string &text) {
        Reader r{text.data(), text.data() + text.size()};
        Json v = r.value(0);
        r.space();
        if (r.p != r.end) throw ConfigError("json: text after the value");
        return v;
    }

    bool is_null() const { return kind == NIL; }
    // a member that may be absent (or null)
    const Json *find(const std::string &key) const {
        if (kind != OBJECT) return nullptr;
        auto it = object.find(key);
        return it == object.end() || it->second.is_null() ? nullptr : &it->second;
    }
    const Json &at(const std::string &key) const {
        const Json *v = find(key);
        if (!v) throw ConfigError("config: '" + key + "' is missing");
        return *v;
    }
    double real() const {
        if (kind != NUMBER) throw ConfigError("config: expected a number");
        return number;
    }
    size_t nat() const {
        const double d = real();
        if (!(d >= 0.0) || d > 9007199254740992.0 || d != (double)(size_t)d) throw ConfigError("config: expected a non-negative integer");
        return (size_t)d;
    }
    const std::string &str() const {
        if (kind != STRING) throw ConfigError("config: expected a string");
        return string;
    }
    bool flag() const {
        if (kind != BOOL) throw ConfigError("config: expected true or false");
        return boolean;
    }
    const std::vector<Json> &list() const {
        if (kind != ARRAY) throw ConfigError("config: expected a list");
        return array;
    }

  private:
    struct Reader {
        const char *p, *end;
        void space() {
            while (p < end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) p++;
        }
        char peek() {
            space();
            if (p >= end) throw ConfigError("json: unexpected end");
            return *p;
        }
        void expect(char c) {
            if (peek() != c) throw ConfigError(std::string("json: expected '") + c + "'");
            p++;
        }
        bool word(const char *w, size_t n) {
            if ((size_t)(end - p) < n || std::string(p, n) != w) return false;
            p += n;
            return true;
        }
        std::string text() {
            expect('"');
            std::string s;
            for (;;) {
                if (p >= end) throw ConfigError("json: unexpected end");
                char c = *p++;
                if (c == '"') return s;
                if (c != '\\') {
                    s += c;
                    continue;
                }
                if (p >= end) throw ConfigError("json: unexpected end");
                c = *p++;
                switch (c) {
                case 'n': s += '\n'; break;
                case 't': s += '\t'; break;
                case 'r': s += '\r'; break;
                case 'b': s += '\b'; break;
                case 'f': s += '\f'; break;
                case 'u': s += "\\u"; break; // kept as written: keys and names are plain ASCII
                default: s += c;
                }
            }
        }
        Json value(int depth) {
            if (depth > 64) throw ConfigError("json: nested too deeply");
            Json v;
            const char c = peek();
            if (c == '{') {
                v.kind = OBJECT;
                p++;
                if (peek() == '}') {
                    p++;
                    return v;
                }
                for (;;) {
                    space();
                    std::string key = text();
                    expect(':');
                    v.object[key] = value(depth + 1);
                    if (peek() != ',') break;
                    p++;
                }
                expect('}');
            } else if (c == '[') {
                v.kind = ARRAY;
                p++;
                if (peek() == ']') {
                    p++;
                    return v;
                }
                for (;;) {
                    v.array.push_back(value(depth + 1));
                    if (peek() != ',') break;
                    p++;
                }
                expect(']');
            } else if (c == '"') {
                v.kind = STRING;
                v.string = text();
            } else if (word("true", 4)) {
                v.kind = BOOL;
                v.boolean = true;
            } else if (word("false", 5)) {
                v.kind = BOOL;
            } else if (word("null", 4)) {
                v.kind = NIL;
            } else {
                const char *q = p;
                while (q < end && ((*q >= '0' && *q <= '9') || *q == '-' || *q == '+' || *q == '.' || *q == 'e' || *q == 'E')) q++;
                if (q == p) throw ConfigError("json: unexpected character");
                const std::string n(p, q);
                char *stop = nullptr;
                v.kind = NUMBER;
                v.number = std::strtod(n.c_str(), &stop);
                if (stop != n.c_str() + n.size()) throw ConfigError("json: malformed number");
                p = q;
            }
            return v;
        }
    };
};

} // namespace cgh
