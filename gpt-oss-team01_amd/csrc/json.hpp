// A small JSON reader for model configurations and safetensors headers.
#pragma once
#include <stdlib.h>
#include <string.h>

#include <string>
#include <utility>
#include <vector>

namespace gptoss {

struct Json {
  enum Type { NUL, BOOL, NUMBER, STRING, ARRAY, OBJECT } type = NUL;
  bool boolean = false;
  double number = 0.0;
  std::string text;
  std::vector<Json> items;                            // ARRAY
  std::vector<std::pair<std::string, Json>> fields;   // OBJECT

  const Json *find(const char *key) const {
    for (const auto &f : fields)
      if (f.first == key) return &f.second;
    return nullptr;
  }
  bool is(Type t) const { return type == t; }

  // false: not JSON, or nested deeper than any document read here
  static bool parse(const char *s, size_t n, Json *out) {
    Reader r{s, s + n};
    if (!r.value(out, 0)) return false;
    r.space();
    return r.p == r.end;
  }

 private:
  struct Reader {
    const char *p, *end;
    void space() {
      while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) p++;
    }
    bool word(const char *w) {
      const size_t n = strlen(w);
      if ((size_t)(end - p) < n || memcmp(p, w, n)) return false;
      p += n;
      return true;
    }
    bool string(std::string *out) {
      if (p >= end || *p != '"') return false;
      for (p++; p < end && *p != '"'; p++) {
        if (*p != '\\') {
          out->push_back(*p);
          continue;
        }
        if (++p >= end) return false;
        switch (*p) {
          case 'n': out->push_back('\n'); break;
          case 't': out->push_back('\t'); break;
          case 'r': out->push_back('\r'); break;
          case 'b': out->push_back('\b'); break;
          case 'f': out->push_back('\f'); break;
          case 'u': {
            if (end - p < 5) return false;
            const std::string hex(p + 1, p + 5);
            const unsigned c = (unsigned)strtoul(hex.c_str(), nullptr, 16);
            if (c < 0x80) {
              out->push_back((char)c);
            } else if (c < 0x800) {
              out->push_back((char)(0xC0 | (c >> 6)));
              out->push_back((char)(0x80 | (c & 0x3F)));
            } else {
              out->push_back((char)(0xE0 | (c >> 12)));
              out->push_back((char)(0x80 | ((c >> 6) & 0x3F)));
              out->push_back((char)(0x80 | (c & 0x3F)));
            }
            p += 4;
            break;
          }
          default: out->push_back(*p);
        }
      }
      if (p >= end) return false;
      p++;
      return true;
    }
    bool value(Json *v, int depth) {
      if (depth > 64) return false;
      space();
      if (p >= end) return false;
      if (*p == '{') {
        v->type = OBJECT;
        p++;
        space();
        if (p < end && *p == '}') return p++, true;
        while (true) {
          space();
          v->fields.emplace_back();
          if (!string(&v->fields.back().first)) return false;
          space();
          if (p >= end || *p++ != ':') return false;
          if (!value(&v->fields.back().second, depth + 1)) return false;
          space();
          if (p >= end) return false;
          if (*p == ',') { p++; continue; }
          return *p++ == '}';
        }
      }
      if (*p == '[') {
        v->type = ARRAY;
        p++;
        space();
        if (p < end && *p == ']') return p++, true;
        while (true) {
          v->items.emplace_back();
          if (!value(&v->items.back(), depth + 1)) return false;
          space();
          if (p >= end) return false;
          if (*p == ',') { p++; continue; }
          return *p++ == ']';
        }
      }
      if (*p == '"') {
        v->type = STRING;
        return string(&v->text);
      }
      if (word("true")) return v->type = BOOL, v->boolean = true, true;
      if (word("false")) return v->type = BOOL, true;
      if (word("null")) return true;
      const char *q = p;
      while (q < end && (strchr("+-.eE", *q) || (*q >= '0' && *q <= '9'))) q++;
      if (q == p) return false;
      const std::string num(p, q);
      char *stop = nullptr;
      v->type = NUMBER;
      v->number = strtod(num.c_str(), &stop);
      p = q;
      return stop && *stop == 0;
    }
  };
};

}  // namespace gptoss
