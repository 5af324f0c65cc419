// json.h -- a small JSON reader (RFC 8259) for model configurations, safetensors
// headers and traces.  Throws std::runtime_error on malformed text or on a value of
// another type than asked for.
#pragma once

#include <cmath>
#include <cstdint>
#include <cstdlib>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

namespace bh {

class Json {
public:
  enum Type { kNull, kBool, kNumber, kString, kArray, kObject };

  static Json parse(const char *text, size_t size) {
    Reader r{text, text + size};
    Json v = r.value(0);
    r.space();
    if (r.p != r.end)
      throw std::runtime_error("JSON: text after the value");
    return v;
  }
  static Json parse(const std::string &s) { return parse(s.data(), s.size()); }

  Type type() const { return type_; }
  bool is_null() const { return type_ == kNull; }
  bool boolean() const { return want(kBool, "a truth value").num_ != 0; }
  double number() const { return want(kNumber, "a number").num_; }
  int64_t integer() const {
    const double d = number();
    if (d != std::floor(d) || std::fabs(d) > 9007199254740992.0)
      throw std::runtime_error("JSON: expected an integer");
    return (int64_t)d;
  }
  const std::string &string() const { return want(kString, "a string").str_; }
  const std::vector<Json> &array() const { return want(kArray, "an array").items_; }
  const std::vector<std::pair<std::string, Json>> &object() const {
    return want(kObject, "an object").members_;
  }
  // member of an object: null when missing
  const Json *find(const std::string &key) const {
    for (const auto &m : object())
      if (m.first == key)
        return &m.second;
    return nullptr;
  }
  const Json &at(const std::string &key) const {
    const Json *v = find(key);
    if (!v)
      throw std::runtime_error("JSON: no \"" + key + "\"");
    return *v;
  }

private:
  const Json &want(Type t, const char *what) const {
    if (type_ != t)
      throw std::runtime_error(std::string("JSON: expected ") + what);
    return *this;
  }

  struct Reader {
    const char *p, *end;
    [[noreturn]] void bad(const char *what) const {
      throw std::runtime_error(std::string("JSON: ") + what);
    }
    void space() {
      while (p != end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r'))
        ++p;
    }
    bool take(char c) {
      space();
      if (p == end || *p != c)
        return false;
      ++p;
      return true;
    }
    void need(char c) {
      if (!take(c))
        bad("unexpected character");
    }
    bool word(const char *w) {
      const char *q = p;
      while (*w && q != end && *q == *w) {
        ++q;
        ++w;
      }
      if (*w)
        return false;
      p = q;
      return true;
    }
    Json value(int depth) {
      if (depth > 64)
        bad("nested too deeply");
      space();
      if (p == end)
        bad("text ends early");
      Json v;
      switch (*p) {
      case '{':
        ++p;
        v.type_ = kObject;
        if (take('}'))
          return v;
        do {
          space();
          std::string key = text();
          need(':');
          Json member = value(depth + 1);
          v.members_.emplace_back(std::move(key), std::move(member));
        } while (take(','));
        need('}');
        return v;
      case '[':
        ++p;
        v.type_ = kArray;
        if (take(']'))
          return v;
        do
          v.items_.push_back(value(depth + 1));
        while (take(','));
        need(']');
        return v;
      case '"':
        v.type_ = kString;
        v.str_ = text();
        return v;
      case 't':
      case 'f':
        v.type_ = kBool;
        v.num_ = *p == 't';
        if (!word(*p == 't' ? "true" : "false"))
          bad("unknown word");
        return v;
      case 'n':
        if (!word("null"))
          bad("unknown word");
        return v;
      default:
        break;
      }
      const char *q = p;
      while (q != end && ((*q >= '0' && *q <= '9') || *q == '-' || *q == '+' || *q == '.' ||
                          *q == 'e' || *q == 'E'))
        ++q;
      if (q == p)
        bad("unexpected character");
      const std::string digits(p, q);
      char *stop = nullptr;
      v.type_ = kNumber;
      v.num_ = std::strtod(digits.c_str(), &stop);
      if (*stop)
        bad("not a number");
      p = q;
      return v;
    }
    unsigned hex4() {
      unsigned v = 0;
      for (int i = 0; i < 4; ++i, ++p) {
        if (p == end)
          bad("text ends early");
        const char c = *p;
        const int d = c >= '0' && c <= '9'   ? c - '0'
                      : c >= 'a' && c <= 'f' ? c - 'a' + 10
                      : c >= 'A' && c <= 'F' ? c - 'A' + 10
                                             : -1;
        if (d < 0)
          bad("bad escape");
        v = v * 16 + (unsigned)d;
      }
      return v;
    }
    std::string text() {
      if (p == end || *p != '"')
        bad("expected a string");
      ++p;
      std::string s;
      while (true) {
        if (p == end)
          bad("text ends early");
        const char c = *p++;
        if (c == '"')
          return s;
        if (c != '\\') {
          s += c;
          continue;
        }
        if (p == end)
          bad("text ends early");
        const char e = *p++;
        switch (e) {
        case 'n': s += '\n'; break;
        case 't': s += '\t'; break;
        case 'r': s += '\r'; break;
        case 'b': s += '\b'; break;
        case 'f': s += '\f'; break;
        case 'u': {
          unsigned u = hex4();
          if (u >= 0xd800 && u < 0xdc00) { // the first half of a pair
            if (!word("\\u"))
              bad("half a surrogate pair");
            u = 0x10000 + ((u - 0xd800) << 10) + ((hex4() - 0xdc00) & 0x3ff);
          }
          if (u < 0x80) {
            s += (char)u;
          } else if (u < 0x800) {
            s += (char)(0xc0 | u >> 6);
            s += (char)(0x80 | (u & 63));
          } else if (u < 0x10000) {
            s += (char)(0xe0 | u >> 12);
            s += (char)(0x80 | (u >> 6 & 63));
            s += (char)(0x80 | (u & 63));
          } else {
            s += (char)(0xf0 | u >> 18);
            s += (char)(0x80 | (u >> 12 & 63));
            s += (char)(0x80 | (u >> 6 & 63));
            s += (char)(0x80 | (u & 63));
          }
          break;
        }
        default:
          if (e != '"' && e != '\\' && e != '/')
            bad("bad escape");
          s += e;
        }
      }
    }
  };

  Type type_ = kNull;
  double num_ = 0;
  std::string str_;
  std::vector<Json> items_;
  std::vector<std::pair<std::string, Json>> members_;
};

} // namespace bh
