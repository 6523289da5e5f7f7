// A small JSON reader for config.json files and safetensors headers.
#pragma once

#include <cctype>
#include <cmath>
#include <cstdlib>
#include <map>
#include <stdexcept>
#include <string>
#include <vector>

namespace lightseq {
namespace hip {

class Json {
 public:
  enum Type { kNull, kBool, kNumber, kString, kArray, kObject };

  static Json parse(const char* begin, const char* end) {
    Parser p{begin, end};
    Json v = p.value(0);
    p.space();
    if (p.at != p.end) throw std::runtime_error("json: text after the value");
    return v;
  }
  static Json parse(const std::string& s) { return parse(s.data(), s.data() + s.size()); }

  Type type() const { return type_; }
  bool is_null() const { return type_ == kNull; }
  // a member that is absent and one that is null are the same: a null value
  const Json& operator[](const std::string& key) const {
    static const Json none;
    if (type_ == kNull) return none;
    need(kObject, "an object");
    auto it = members_.find(key);
    return it == members_.end() ? none : it->second;
  }
  const Json& at(const std::string& key) const {
    const Json& v = (*this)[key];
    if (v.is_null()) throw std::runtime_error("config: '" + key + "' is missing");
    return v;
  }
  const std::map<std::string, Json>& members() const {
    need(kObject, "an object");
    return members_;
  }
  const std::vector<Json>& items() const {
    need(kArray, "an array");
    return items_;
  }
  double number() const {
    need(kNumber, "a number");
    return number_;
  }
  long integer() const {
    need(kNumber, "a number");
    if (number_ != std::floor(number_) || std::fabs(number_) > 9007199254740992.0)
      throw std::runtime_error("json: an integer was expected");
    return (long)number_;
  }
  // the member `key`, a size or a count
  int positive(const char* key) const {
    const long v = at(key).integer();
    if (v <= 0 || v > (1L << 30))
      throw std::runtime_error(std::string("config: '") + key + "' must be a positive integer");
    return (int)v;
  }
  const std::string& string() const {
    need(kString, "a string");
    return string_;
  }

 private:
  void need(Type t, const char* what) const {
    if (type_ != t) throw std::runtime_error(std::string("json: ") + what + " was expected");
  }
  struct Parser {
    const char *at, *end;
    [[noreturn]] void fail(const char* what) { throw std::runtime_error(std::string("json: ") + what); }
    void space() {
      while (at != end && (*at == ' ' || *at == '\t' || *at == '\n' || *at == '\r')) ++at;
    }
    char peek() {
      space();
      if (at == end) fail("unexpected end");
      return *at;
    }
    void expect(char c) {
      if (peek() != c) fail("unexpected character");
      ++at;
    }
    bool word(const char* w) {
      const char* p = at;
      for (; *w; ++w, ++p)
        if (p == end || *p != *w) return false;
      at = p;
      return true;
    }
    void utf8(std::string& s, unsigned c) {
      if (c < 0x80) {
        s += (char)c;
      } else if (c < 0x800) {
        s += (char)(0xc0 | c >> 6);
        s += (char)(0x80 | (c & 0x3f));
      } else if (c < 0x10000) {
        s += (char)(0xe0 | c >> 12);
        s += (char)(0x80 | (c >> 6 & 0x3f));
        s += (char)(0x80 | (c & 0x3f));
      } else {
        s += (char)(0xf0 | c >> 18);
        s += (char)(0x80 | (c >> 12 & 0x3f));
        s += (char)(0x80 | (c >> 6 & 0x3f));
        s += (char)(0x80 | (c & 0x3f));
      }
    }
    unsigned hex4() {
      if (end - at < 4) fail("bad escape");
      unsigned v = 0;
      for (int i = 0; i < 4; ++i, ++at) {
        if (!isxdigit((unsigned char)*at)) fail("bad escape");
        v = v * 16 + (isdigit((unsigned char)*at) ? *at - '0' : (*at | 0x20) - 'a' + 10);
      }
      return v;
    }
    std::string text() {
      expect('"');
      std::string s;
      for (;;) {
        if (at == end) fail("unterminated string");
        const char c = *at++;
        if (c == '"') return s;
        if (c != '\\') {
          s += c;
          continue;
        }
        if (at == end) fail("bad escape");
        const char e = *at++;
        switch (e) {
          case 'n': s += '\n'; break;
          case 't': s += '\t'; break;
          case 'r': s += '\r'; break;
          case 'b': s += '\b'; break;
          case 'f': s += '\f'; break;
          case 'u': {
            unsigned v = hex4();
            if (v >= 0xd800 && v < 0xdc00 && end - at >= 6 && at[0] == '\\' && at[1] == 'u') {
              at += 2;
              v = 0x10000 + ((v - 0xd800) << 10) + (hex4() - 0xdc00);
            }
            utf8(s, v);
            break;
          }
          case '"': case '\\': case '/': s += e; break;
          default: fail("bad escape");
        }
      }
    }
    Json value(int depth) {
      if (depth > 64) fail("nested too deeply");
      Json v;
      const char c = peek();
      if (c == '{') {
        ++at;
        v.type_ = kObject;
        if (peek() == '}') {
          ++at;
          return v;
        }
        for (;;) {
          space();
          std::string key = text();
          expect(':');
          v.members_[key] = value(depth + 1);
          if (peek() == ',') {
            ++at;
            continue;
          }
          expect('}');
          return v;
        }
      }
      if (c == '[') {
        ++at;
        v.type_ = kArray;
        if (peek() == ']') {
          ++at;
          return v;
        }
        for (;;) {
          v.items_.push_back(value(depth + 1));
          if (peek() == ',') {
            ++at;
            continue;
          }
          expect(']');
          return v;
        }
      }
      if (c == '"') {
        v.type_ = kString;
        v.string_ = text();
        return v;
      }
      if (word("null")) return v;
      if (word("true")) {
        v.type_ = kBool;
        v.number_ = 1;
        return v;
      }
      if (word("false")) {
        v.type_ = kBool;
        return v;
      }
      const char* p = at;
      while (p != end && (isdigit((unsigned char)*p) || *p == '-' || *p == '+' || *p == '.' ||
                          *p == 'e' || *p == 'E'))
        ++p;
      const std::string num(at, p);
      char* stop = nullptr;
      v.number_ = strtod(num.c_str(), &stop);
      if (num.empty() || *stop) fail("unexpected character");
      v.type_ = kNumber;
      at = p;
      return v;
    }
  };

  Type type_ = kNull;
  double number_ = 0;
  std::string string_;
  std::vector<Json> items_;
  std::map<std::string, Json> members_;
};

}  // namespace hip
}  // namespace lightseq
