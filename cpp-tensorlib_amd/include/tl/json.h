#pragma once

// A small JSON reader for model configurations and safetensors headers: the whole text into a tree,
// strict about syntax, throws std::runtime_error with the offset. Numbers are doubles (integers up to
// 2^53 exactly); \u escapes become UTF-8.

#include <cmath>
#include <cstdint>
#include <cstdlib>
#include <cstring>
#include <map>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

namespace tl {
namespace json {

class value {
 public:
  enum class kind { null, boolean, number, string, array, object };
  kind k = kind::null;
  bool b = false;
  double n = 0;
  std::string s;
  std::vector<value> a;
  std::vector<std::pair<std::string, value>> o;   // in file order

  bool is_null() const { return k == kind::null; }
  bool is_object() const { return k == kind::object; }
  const value* find(const std::string& key) const {
    for (const auto& e : o)
      if (e.first == key) return &e.second;
    return nullptr;
  }
  const value& at(const std::string& key) const {
    const value* v = k == kind::object ? find(key) : nullptr;
    if (!v) throw std::runtime_error("missing key \"" + key + "\"");
    return *v;
  }
  double num() const {
    if (k != kind::number) throw std::runtime_error("number expected");
    return n;
  }
  int64_t integer() const {
    const double d = num();
    if (d != std::floor(d) || std::fabs(d) > 9007199254740992.0) throw std::runtime_error("integer expected");
    return static_cast<int64_t>(d);
  }
  const std::string& str() const {
    if (k != kind::string) throw std::runtime_error("string expected");
    return s;
  }
  const std::vector<value>& items() const {
    if (k != kind::array) throw std::runtime_error("array expected");
    return a;
  }
};

namespace detail {
class parser {
  const char *p_, *begin_, *end_;
  int depth_ = 0;

  [[noreturn]] void bad(const char* what) const {
    throw std::runtime_error(std::string("JSON: ") + what + " at byte " + std::to_string(p_ - begin_));
  }
  void space() {
    while (p_ < end_ && (*p_ == ' ' || *p_ == '\t' || *p_ == '\n' || *p_ == '\r')) p_++;
  }
  bool take(char c) {
    if (p_ < end_ && *p_ == c) { p_++; return true; }
    return false;
  }
  void word(const char* w) {
    const size_t n = std::strlen(w);
    if (static_cast<size_t>(end_ - p_) < n || std::memcmp(p_, w, n) != 0) bad("unknown word");
    p_ += n;
  }
  unsigned hex4() {
    if (end_ - p_ < 4) bad("short escape");
    unsigned v = 0;
    for (int i = 0; i < 4; i++, p_++) {
      const char c = *p_;
      if (c >= '0' && c <= '9') v = v * 16 + static_cast<unsigned>(c - '0');
      else if (c >= 'a' && c <= 'f') v = v * 16 + static_cast<unsigned>(c - 'a' + 10);
      else if (c >= 'A' && c <= 'F') v = v * 16 + static_cast<unsigned>(c - 'A' + 10);
      else bad("bad escape");
    }
    return v;
  }
  static void utf8(std::string& s, unsigned c) {
    const auto put = [&s](unsigned b) { s.push_back(static_cast<char>(b)); };
    if (c < 0x80) put(c);
    else if (c < 0x800) { put(0xC0 | c >> 6); put(0x80 | (c & 63)); }
    else if (c < 0x10000) { put(0xE0 | c >> 12); put(0x80 | (c >> 6 & 63)); put(0x80 | (c & 63)); }
    else { put(0xF0 | c >> 18); put(0x80 | (c >> 12 & 63)); put(0x80 | (c >> 6 & 63)); put(0x80 | (c & 63)); }
  }
  std::string string() {
    std::string s;
    if (!take('"')) bad("string expected");
    while (p_ < end_ && *p_ != '"') {
      if (static_cast<unsigned char>(*p_) < 0x20) bad("control character in a string");
      if (*p_ != '\\') { s.push_back(*p_++); continue; }
      if (++p_ >= end_) bad("short escape");
      switch (*p_++) {
        case '"': s.push_back('"'); break;
        case '\\': s.push_back('\\'); break;
        case '/': s.push_back('/'); break;
        case 'b': s.push_back('\b'); break;
        case 'f': s.push_back('\f'); break;
        case 'n': s.push_back('\n'); break;
        case 'r': s.push_back('\r'); break;
        case 't': s.push_back('\t'); break;
        case 'u': {
          unsigned c = hex4();
          if (c >= 0xD800 && c < 0xDC00 && end_ - p_ >= 6 && p_[0] == '\\' && p_[1] == 'u') {
            p_ += 2;
            c = 0x10000 + ((c - 0xD800) << 10) + ((hex4() - 0xDC00) & 0x3FF);
          }
          utf8(s, c);
          break;
        }
        default: bad("bad escape");
      }
    }
    if (!take('"')) bad("unterminated string");
    return s;
  }
  value any() {
    if (++depth_ > 200) bad("nested too deeply");
    value v;
    space();
    if (p_ >= end_) bad("unexpected end");
    if (*p_ == '{') {
      p_++;
      v.k = value::kind::object;
      space();
      for (bool more = !take('}'); more;) {
        space();
        std::string key = string();
        space();
        if (!take(':')) bad("':' expected");
        v.o.emplace_back(std::move(key), any());
        space();
        more = take(',');
        if (!more && !take('}')) bad("',' or '}' expected");
      }
    } else if (*p_ == '[') {
      p_++;
      v.k = value::kind::array;
      space();
      for (bool more = !take(']'); more;) {
        v.a.push_back(any());
        space();
        more = take(',');
        if (!more && !take(']')) bad("',' or ']' expected");
      }
    } else if (*p_ == '"') {
      v.k = value::kind::string;
      v.s = string();
    } else if (*p_ == 't') {
      word("true");
      v.k = value::kind::boolean;
      v.b = true;
    } else if (*p_ == 'f') {
      word("false");
      v.k = value::kind::boolean;
    } else if (*p_ == 'n') {
      word("null");
    } else {
      const char* q = p_;
      while (q < end_ && (std::strchr("+-.eE", *q) || (*q >= '0' && *q <= '9'))) q++;
      const std::string t(p_, q);
      char* stop = nullptr;
      v.n = std::strtod(t.c_str(), &stop);
      if (t.empty() || *stop) bad("value expected");
      v.k = value::kind::number;
      p_ = q;
    }
    depth_--;
    return v;
  }

 public:
  parser(const char* p, size_t n) : p_(p), begin_(p), end_(p + n) {}
  value all() {
    value v = any();
    space();
    if (p_ != end_) bad("text after the value");
    return v;
  }
};
}  // namespace detail

inline value parse(const char* text, size_t n) { return detail::parser(text, n).all(); }
inline value parse(const std::string& text) { return parse(text.data(), text.size()); }

}  // namespace json
}  // namespace tl
