// json.hpp -- a small JSON reader: what config.json and a safetensors header need (RFC 8259 values, UTF-8 passed through).
#pragma once
#include <cmath>
#include <cstdint>
#include <cstdlib>
#include <map>
#include <memory>
#include <string>
#include <utility>
#include <vector>

#include "strider.hpp"  // Error

namespace crabml_host {

class Json {
 public:
  enum class Kind { Null, Bool, Number, String, Array, Object };
  Json() = default;

  static Json parse(const char* text, size_t n) {
    Reader r{text, text + n};
    Json v = r.value(0);
    r.space();
    if (r.p != r.end) r.fail("something follows the value");
    return v;
  }
  static Json parse(const std::string& s) { return parse(s.data(), s.size()); }

  Kind kind() const { return kind_; }
  bool is_null() const { return kind_ == Kind::Null; }
  bool is_object() const { return kind_ == Kind::Object; }
  const std::vector<Json>& items() const {
    need(Kind::Array, "an array");
    return items_;
  }
  const std::vector<std::pair<std::string, Json>>& fields() const {
    need(Kind::Object, "an object");
    return fields_;
  }
  // the field of an object, null if absent
  const Json& operator[](const std::string& key) const {
    static const Json none;
    need(Kind::Object, "an object");
    for (const auto& f : fields_)
      if (f.first == key) return f.second;
    return none;
  }
  const Json& at(const std::string& key) const {
    const Json& v = (*this)[key];
    if (v.is_null()) throw Error(ErrorKind::ModelError, "missing `" + key + "`");
    return v;
  }
  double number() const {
    need(Kind::Number, "a number");
    return num_;
  }
  size_t size() const {
    const double v = number();
    if (v < 0 || v != std::floor(v) || v > 9007199254740992.0) throw Error(ErrorKind::ModelError, "expected a whole number");
    return (size_t)v;
  }
  bool truth() const {
    need(Kind::Bool, "true or false");
    return num_ != 0;
  }
  const std::string& str() const {
    need(Kind::String, "a string");
    return str_;
  }

 private:
  void need(Kind k, const char* what) const {
    if (kind_ != k) throw Error(ErrorKind::ModelError, std::string("json: expected ") + what);
  }

  struct Reader {
    const char* p;
    const char* end;
    [[noreturn]] void fail(const char* what) const { throw Error(ErrorKind::FormatError, std::string("json: ") + what); }
    void space() {
      while (p != end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) p++;
    }
    bool take(char c) {
      space();
      if (p == end || *p != c) return false;
      p++;
      return true;
    }
    void word(const char* w) {
      for (; *w; w++, p++)
        if (p == end || *p != *w) fail("unknown word");
    }
    Json value(int depth) {
      if (depth > 64) fail("nested too deeply");
      space();
      if (p == end) fail("ends early");
      Json v;
      switch (*p) {
        case '{':
          p++;
          v.kind_ = Kind::Object;
          if (take('}')) return v;
          do {
            space();
            if (p == end || *p != '"') fail("a field needs a name");
            std::string key = string();
            if (!take(':')) fail("a field needs a colon");
            v.fields_.emplace_back(std::move(key), value(depth + 1));
          } while (take(','));
          if (!take('}')) fail("an object does not end");
          return v;
        case '[':
          p++;
          v.kind_ = Kind::Array;
          if (take(']')) return v;
          do v.items_.push_back(value(depth + 1));
          while (take(','));
          if (!take(']')) fail("an array does not end");
          return v;
        case '"':
          v.kind_ = Kind::String;
          v.str_ = string();
          return v;
        case 't': word("true"); v.kind_ = Kind::Bool; v.num_ = 1; return v;
        case 'f': word("false"); v.kind_ = Kind::Bool; return v;
        case 'n': word("null"); return v;
        default: break;
      }
      const char* q = p;
      while (q != end && (*q == '-' || *q == '+' || *q == '.' || *q == 'e' || *q == 'E' || (*q >= '0' && *q <= '9'))) q++;
      const std::string t(p, q);
      char* stop = nullptr;
      v.num_ = std::strtod(t.c_str(), &stop);
      if (t.empty() || stop != t.c_str() + t.size()) fail("not a number");
      v.kind_ = Kind::Number;
      p = q;
      return v;
    }
    std::string string() {
      std::string s;
      for (p++; p != end && *p != '"'; p++) {
        if (*p != '\\') {
          s += *p;
          continue;
        }
        if (++p == end) break;
        switch (*p) {
          case 'b': s += '\b'; break;
          case 'f': s += '\f'; break;
          case 'n': s += '\n'; break;
          case 'r': s += '\r'; break;
          case 't': s += '\t'; break;
          case 'u': {
            unsigned c = hex4();
            if (c >= 0xD800 && c < 0xDC00 && end - p > 2 && p[1] == '\\' && p[2] == 'u') {
              p += 2;
              c = 0x10000 + ((c - 0xD800) << 10) + (hex4() - 0xDC00);
            }
            if (c < 0x80) {
              s += (char)c;
            } else if (c < 0x800) {
              s += (char)(0xC0 | c >> 6);
              s += (char)(0x80 | (c & 63));
            } else if (c < 0x10000) {
              s += (char)(0xE0 | c >> 12);
              s += (char)(0x80 | (c >> 6 & 63));
              s += (char)(0x80 | (c & 63));
            } else {
              s += (char)(0xF0 | c >> 18);
              s += (char)(0x80 | (c >> 12 & 63));
              s += (char)(0x80 | (c >> 6 & 63));
              s += (char)(0x80 | (c & 63));
            }
            break;
          }
          default: s += *p;
        }
      }
      if (p == end) fail("a string does not end");
      p++;
      return s;
    }
    unsigned hex4() {  // leaves p on the last digit
      unsigned v = 0;
      for (int i = 0; i < 4; i++) {
        if (++p == end) fail("a string does not end");
        const char c = *p;
        const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
        if (d < 0) fail("not a hex digit");
        v = v * 16 + (unsigned)d;
      }
      return v;
    }
  };

  Kind kind_ = Kind::Null;
  double num_ = 0;
  std::string str_;
  std::vector<Json> items_;
  std::vector<std::pair<std::string, Json>> fields_;
};

}  // namespace crabml_host
