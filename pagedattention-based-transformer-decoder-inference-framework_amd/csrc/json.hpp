// A small JSON reader for model configurations and safetensors headers.
#pragma once

#include <cstdlib>
#include <cstring>
#include <map>
#include <string>
#include <vector>

namespace llm {

struct Json {
  enum Kind { Null, Bool, Number, String, Array, Object };
  Kind kind = Null;
  bool b = false;
  double num = 0.0;
  std::string str;
  std::vector<Json> arr;
  std::map<std::string, Json> obj;

  bool is_null() const { return kind == Null; }
  bool is_object() const { return kind == Object; }
  bool is_array() const { return kind == Array; }
  // member of an object, or a null value
  const Json& operator[](const std::string& key) const {
    static const Json none;
    const auto it = obj.find(key);
    return it == obj.end() ? none : it->second;
  }
  bool has(const std::string& key) const { return !(*this)[key].is_null(); }
};

class JsonReader {
 public:
  JsonReader(const char* p, size_t n) : p_(p), end_(p + n) {}
  // false: not one well-formed JSON value
  bool parse(Json& out) {
    if (!value(out, 0)) return false;
    space();
    return p_ == end_;
  }

 private:
  static constexpr int kMaxDepth = 64;
  const char* p_;
  const char* end_;

  void space() {
    while (p_ < end_ && (*p_ == ' ' || *p_ == '\n' || *p_ == '\t' || *p_ == '\r')) ++p_;
  }
  bool word(const char* w) {
    const size_t n = std::strlen(w);
    if ((size_t)(end_ - p_) < n || std::strncmp(p_, w, n) != 0) return false;
    p_ += n;
    return true;
  }
  static void utf8(unsigned c, std::string& s) {
    if (c < 0x80) { s += (char)c; return; }
    if (c < 0x800) { s += (char)(0xC0 | c >> 6); s += (char)(0x80 | (c & 63)); return; }
    s += (char)(0xE0 | c >> 12);
    s += (char)(0x80 | ((c >> 6) & 63));
    s += (char)(0x80 | (c & 63));
  }
  bool string(std::string& s) {
    if (p_ >= end_ || *p_ != '"') return false;
    for (++p_; p_ < end_ && *p_ != '"'; ++p_) {
      if (*p_ != '\\') { s += *p_; continue; }
      if (++p_ >= end_) return false;
      switch (*p_) {
        case 'n': s += '\n'; break;
        case 't': s += '\t'; break;
        case 'r': s += '\r'; break;
        case 'b': s += '\b'; break;
        case 'f': s += '\f'; break;
        case 'u': {
          if (end_ - p_ < 5) return false;
          utf8((unsigned)std::strtoul(std::string(p_ + 1, 4).c_str(), nullptr, 16), s);
          p_ += 4;
          break;
        }
        default: s += *p_;
      }
    }
    if (p_ >= end_) return false;
    ++p_;
    return true;
  }
  bool value(Json& v, int depth) {
    if (depth > kMaxDepth) return false;
    space();
    if (p_ >= end_) return false;
    if (*p_ == '{') {
      v.kind = Json::Object;
      ++p_;
      space();
      if (p_ < end_ && *p_ == '}') { ++p_; return true; }
      for (;;) {
        std::string key;
        space();
        if (!string(key)) return false;
        space();
        if (p_ >= end_ || *p_++ != ':') return false;
        if (!value(v.obj[key], depth + 1)) return false;
        space();
        if (p_ >= end_) return false;
        if (*p_ == ',') { ++p_; continue; }
        return *p_++ == '}';
      }
    }
    if (*p_ == '[') {
      v.kind = Json::Array;
      ++p_;
      space();
      if (p_ < end_ && *p_ == ']') { ++p_; return true; }
      for (;;) {
        v.arr.emplace_back();
        if (!value(v.arr.back(), depth + 1)) return false;
        space();
        if (p_ >= end_) return false;
        if (*p_ == ',') { ++p_; continue; }
        return *p_++ == ']';
      }
    }
    if (*p_ == '"') { v.kind = Json::String; return string(v.str); }
    if (*p_ == 't') { v.kind = Json::Bool; v.b = true; return word("true"); }
    if (*p_ == 'f') { v.kind = Json::Bool; return word("false"); }
    if (*p_ == 'n') return word("null");
    const char* q = p_;
    while (q < end_ && std::strchr("+-.eE0123456789", *q)) ++q;
    if (q == p_) return false;
    const std::string t(p_, q);
    char* stop = nullptr;
    v.num = std::strtod(t.c_str(), &stop);
    v.kind = Json::Number;
    p_ = q;
    return *stop == '\0';
  }
};

}  // namespace llm
