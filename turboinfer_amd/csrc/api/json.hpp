// json.hpp -- a small JSON reader for model configurations and safetensors headers (not installed).
#pragma once

#include <cstdlib>
#include <map>
#include <stdexcept>
#include <string>
#include <vector>

namespace turboinfer {
namespace api {

class Json {
 public:
  enum Kind { kNull, kBool, kNumber, kString, kArray, kObject };

  static Json parse(const std::string& text) {
    Parser p{text, 0, 0};
    Json v = p.value();
    p.space();
    if (p.at != text.size()) p.fail("trailing characters");
    return v;
  }

  Kind kind() const { return kind_; }
  bool is_null() const { return kind_ == kNull; }
  double number() const { return need(kNumber, "a number"), num_; }
  const std::string& string() const { return need(kString, "a string"), str_; }
  const std::vector<Json>& array() const { return need(kArray, "an array"), arr_; }
  const std::map<std::string, Json>& object() const { return need(kObject, "an object"), obj_; }
  bool has(const std::string& key) const { return kind_ == kObject && obj_.count(key) != 0; }
  /// Member `key`; std::runtime_error when missing.
  const Json& operator[](const std::string& key) const {
    const auto it = object().find(key);
    if (it == obj_.end()) throw std::runtime_error("JSON: missing key \"" + key + "\"");
    return it->second;
  }
  /// The number as an integer that fits int.
  int integer() const {
    const double d = number();
    if (!(d >= -2147483648.0 && d <= 2147483647.0) || d != (double)(int)d)
      throw std::runtime_error("JSON: expected an integer");
    return (int)d;
  }

 private:
  struct Parser {
    const std::string& s;
    size_t at;
    int depth;
    [[noreturn]] void fail(const char* what) const {
      throw std::runtime_error("JSON: " + std::string(what) + " at byte " + std::to_string(at));
    }
    void space() {
      while (at < s.size() && (s[at] == ' ' || s[at] == '\t' || s[at] == '\n' || s[at] == '\r')) ++at;
    }
    bool take(char c) {
      space();
      if (at < s.size() && s[at] == c) return ++at, true;
      return false;
    }
    bool word(const char* w) {
      const std::string t(w);
      if (s.compare(at, t.size(), t) != 0) return false;
      at += t.size();
      return true;
    }
    std::string quoted() {
      if (!take('"')) fail("expected a string");
      std::string o;
      while (at < s.size() && s[at] != '"') {
        char c = s[at++];
        if (c == '\\') {
          if (at >= s.size()) break;
          c = s[at++];
          switch (c) {
            case 'n': o += '\n'; break;
            case 't': o += '\t'; break;
            case 'r': o += '\r'; break;
            case 'b': o += '\b'; break;
            case 'f': o += '\f'; break;
            case 'u': {
              if (at + 4 > s.size()) fail("short \\u escape");
              const unsigned u = (unsigned)std::strtoul(s.substr(at, 4).c_str(), nullptr, 16);
              at += 4;
              if (u < 0x80) o += (char)u;
              else if (u < 0x800) o += {(char)(0xC0 | (u >> 6)), (char)(0x80 | (u & 63))};
              else o += {(char)(0xE0 | (u >> 12)), (char)(0x80 | ((u >> 6) & 63)), (char)(0x80 | (u & 63))};
              break;
            }
            default: o += c;
          }
        } else {
          o += c;
        }
      }
      if (at >= s.size()) fail("unterminated string");
      ++at;
      return o;
    }
    Json value() {
      if (++depth > 64) fail("nested too deeply");
      space();
      if (at >= s.size()) fail("unexpected end");
      Json v;
      if (s[at] == '{') {
        ++at;
        v.kind_ = kObject;
        if (!take('}')) do {
            std::string k = quoted();
            if (!take(':')) fail("expected ':'");
            v.obj_[std::move(k)] = value();
          } while (take(',') || (take('}') ? false : (fail("expected ',' or '}'"), false)));
      } else if (s[at] == '[') {
        ++at;
        v.kind_ = kArray;
        if (!take(']')) do {
            v.arr_.push_back(value());
          } while (take(',') || (take(']') ? false : (fail("expected ',' or ']'"), false)));
      } else if (s[at] == '"') {
        v.kind_ = kString;
        v.str_ = quoted();
      } else if (word("null")) {
      } else if (word("true")) {
        v.kind_ = kBool;
        v.num_ = 1;
      } else if (word("false")) {
        v.kind_ = kBool;
      } else {
        char* end = nullptr;
        v.kind_ = kNumber;
        v.num_ = std::strtod(s.c_str() + at, &end);
        if (end == s.c_str() + at) fail("unexpected character");
        at = (size_t)(end - s.c_str());
      }
      --depth;
      return v;
    }
  };

  void need(Kind k, const char* what) const {
    if (kind_ != k) throw std::runtime_error(std::string("JSON: expected ") + what);
  }
  Kind kind_ = kNull;
  double num_ = 0;
  std::string str_;
  std::vector<Json> arr_;
  std::map<std::string, Json> obj_;
};

}  // namespace api
}  // namespace turboinfer
