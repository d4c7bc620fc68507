// json.h -- a small JSON reader for config.json and safetensors headers.
#pragma once
#include <stdint.h>
#include <stdlib.h>
#include <string.h>

#include <map>
#include <memory>
#include <string>
#include <vector>

namespace ffmi {

class Json {
 public:
  enum Type { NUL, BOOL, NUM, STR, ARR, OBJ };
  Type type = NUL;
  bool b = false;
  double num = 0;
  std::string str;
  std::vector<Json> arr;
  std::map<std::string, Json> obj;

  bool is_null() const { return type == NUL; }
  const Json *find(const std::string &k) const {
    if (type != OBJ) return nullptr;
    auto it = obj.find(k);
    return it == obj.end() ? nullptr : &it->second;
  }
  // the number at key k; false when absent or not a number
  bool get(const char *k, double *v) const {
    const Json *j = find(k);
    if (!j || j->type != NUM) return false;
    *v = j->num;
    return true;
  }
  bool get(const char *k, int *v) const {
    double d;
    if (!get(k, &d) || d != (double)(int)d) return false;
    *v = (int)d;
    return true;
  }
  bool get(const char *k, float *v) const {
    double d;
    if (!get(k, &d)) return false;
    *v = (float)d;
    return true;
  }
  std::string text(const char *k) const {
    const Json *j = find(k);
    return j && j->type == STR ? j->str : std::string();
  }

  static bool parse(const char *p, size_t n, Json *out) {
    Parser q{p, p + n};
    return q.value(out, 0) && (q.space(), q.p == q.e);
  }

 private:
  struct Parser {
    const char *p, *e;
    void space() {
      while (p < e && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) ++p;
    }
    bool lit(const char *s) {
      const size_t n = strlen(s);
      if ((size_t)(e - p) < n || memcmp(p, s, n)) return false;
      p += n;
      return true;
    }
    bool string(std::string *o) {
      if (p >= e || *p != '"') return false;
      for (++p; p < e && *p != '"'; ++p) {
        if (*p != '\\') {
          o->push_back(*p);
          continue;
        }
        if (++p >= e) return false;
        switch (*p) {
          case 'n': o->push_back('\n'); break;
          case 't': o->push_back('\t'); break;
          case 'r': o->push_back('\r'); break;
          case 'b': o->push_back('\b'); break;
          case 'f': o->push_back('\f'); break;
          case 'u': {
            if (e - p < 5) return false;
            const unsigned c = (unsigned)strtoul(std::string(p + 1, 4).c_str(), nullptr, 16);
            if (c < 0x80) o->push_back((char)c);
            else if (c < 0x800) o->push_back((char)(0xc0 | c >> 6)), o->push_back((char)(0x80 | (c & 63)));
            else
              o->push_back((char)(0xe0 | c >> 12)), o->push_back((char)(0x80 | (c >> 6 & 63))),
                  o->push_back((char)(0x80 | (c & 63)));
            p += 4;
            break;
          }
          default: o->push_back(*p);
        }
      }
      if (p >= e) return false;
      ++p;
      return true;
    }
    bool value(Json *v, int depth) {
      if (depth > 64) return false;
      space();
      if (p >= e) return false;
      if (*p == '{') {
        v->type = OBJ;
        ++p;
        space();
        if (p < e && *p == '}') return ++p, true;
        for (;;) {
          std::string k;
          space();
          if (!string(&k)) return false;
          space();
          if (p >= e || *p++ != ':') return false;
          if (!value(&v->obj[k], depth + 1)) return false;
          space();
          if (p >= e) return false;
          if (*p == ',') { ++p; continue; }
          return *p++ == '}';
        }
      }
      if (*p == '[') {
        v->type = ARR;
        ++p;
        space();
        if (p < e && *p == ']') return ++p, true;
        for (;;) {
          v->arr.emplace_back();
          if (!value(&v->arr.back(), depth + 1)) return false;
          space();
          if (p >= e) return false;
          if (*p == ',') { ++p; continue; }
          return *p++ == ']';
        }
      }
      if (*p == '"') return v->type = STR, string(&v->str);
      if (lit("true")) return v->type = BOOL, v->b = true, true;
      if (lit("false")) return v->type = BOOL, true;
      if (lit("null")) return true;
      const char *q = p;
      while (p < e && (strchr("+-.eE", *p) || (*p >= '0' && *p <= '9'))) ++p;
      if (p == q) return false;
      const std::string t(q, p - q);
      char *end = nullptr;
      v->type = NUM, v->num = strtod(t.c_str(), &end);
      return *end == 0;
    }
  };
};

}  // namespace ffmi
