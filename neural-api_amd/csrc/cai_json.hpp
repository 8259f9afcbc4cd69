// A small JSON reader for model configurations and container headers (host code only).
#pragma once
#include <ctype.h>
#include <math.h>
#include <stdint.h>
#include <stdlib.h>
#include <string>
#include <utility>
#include <vector>

namespace cai {

struct Json {
  enum Kind { NUL, BOOL, NUM, STR, ARR, OBJ } kind = NUL;
  bool b = false; double num = 0.0; std::string str;
  std::vector<Json> arr;
  std::vector<std::pair<std::string, Json>> obj;

  const Json* get(const char* key) const
  {
    for (auto& kv : obj) if (kv.first == key) return &kv.second;
    return nullptr;
  }
  bool is_int() const { return kind == NUM && num == floor(num) && fabs(num) < 9.0e15; }
};

class JsonReader {
 public:
  // false: malformed (error() says where)
  static bool parse(const char* text, size_t n, Json& out, std::string& err)
  {
    JsonReader r(text, n);
    if (!r.value(out, 0)) { err = "malformed JSON near byte " + std::to_string(r.p_); return false; }
    r.space();
    if (r.p_ != n) { err = "text after the JSON value at byte " + std::to_string(r.p_); return false; }
    return true;
  }

 private:
  JsonReader(const char* t, size_t n) : t_(t), n_(n) {}
  void space() { while (p_ < n_ && (t_[p_] == ' ' || t_[p_] == '\n' || t_[p_] == '\t' || t_[p_] == '\r')) p_++; }
  bool eat(char c) { space(); if (p_ < n_ && t_[p_] == c) { p_++; return true; } return false; }
  bool word(const char* w) { size_t k = 0; while (w[k]) { if (p_ + k >= n_ || t_[p_ + k] != w[k]) return false; k++; } p_ += k; return true; }
  static void utf8(std::string& s, uint32_t c)
  {
    if (c < 0x80) s += (char)c;
    else if (c < 0x800) { s += (char)(0xc0 | c >> 6); s += (char)(0x80 | (c & 63)); }
    else if (c < 0x10000) { s += (char)(0xe0 | c >> 12); s += (char)(0x80 | (c >> 6 & 63)); s += (char)(0x80 | (c & 63)); }
    else { s += (char)(0xf0 | c >> 18); s += (char)(0x80 | (c >> 12 & 63)); s += (char)(0x80 | (c >> 6 & 63)); s += (char)(0x80 | (c & 63)); }
  }
  bool hex4(uint32_t& v)
  {
    v = 0;
    for (int i = 0; i < 4; i++) {
      if (p_ >= n_ || !isxdigit((unsigned char)t_[p_])) return false;
      const char c = t_[p_++];
      v = v * 16 + (uint32_t)(c <= '9' ? c - '0' : (c | 32) - 'a' + 10);
    }
    return true;
  }
  bool string(std::string& s)
  {
    if (!eat('"')) return false;
    while (p_ < n_) {
      const char c = t_[p_++];
      if (c == '"') return true;
      if (c != '\\') { s += c; continue; }
      if (p_ >= n_) return false;
      const char e = t_[p_++];
      switch (e) {
        case '"': case '\\': case '/': s += e; break;
        case 'b': s += '\b'; break; case 'f': s += '\f'; break; case 'n': s += '\n'; break;
        case 'r': s += '\r'; break; case 't': s += '\t'; break;
        case 'u': {
          uint32_t v, lo;
          if (!hex4(v)) return false;
          if (v >= 0xd800 && v < 0xdc00) {
            if (!(p_ + 1 < n_ && t_[p_] == '\\' && t_[p_ + 1] == 'u')) return false;
            p_ += 2;
            if (!hex4(lo) || lo < 0xdc00 || lo > 0xdfff) return false;
            v = 0x10000 + ((v - 0xd800) << 10) + (lo - 0xdc00);
          }
          utf8(s, v);
          break;
        }
        default: return false;
      }
    }
    return false;
  }
  bool value(Json& v, int depth)
  {
    if (depth > 64) return false;
    space();
    if (p_ >= n_) return false;
    const char c = t_[p_];
    if (c == '{') {
      p_++; v.kind = Json::OBJ;
      if (eat('}')) return true;
      do {
        v.obj.emplace_back();
        if (!string(v.obj.back().first) || !eat(':') || !value(v.obj.back().second, depth + 1)) return false;
      } while (eat(','));
      return eat('}');
    }
    if (c == '[') {
      p_++; v.kind = Json::ARR;
      if (eat(']')) return true;
      do { v.arr.emplace_back(); if (!value(v.arr.back(), depth + 1)) return false; } while (eat(','));
      return eat(']');
    }
    if (c == '"') { v.kind = Json::STR; return string(v.str); }
    if (c == 't') { v.kind = Json::BOOL; v.b = true; return word("true"); }
    if (c == 'f') { v.kind = Json::BOOL; return word("false"); }
    if (c == 'n') return word("null");
    size_t e = p_;
    while (e < n_ && (isdigit((unsigned char)t_[e]) || t_[e] == '-' || t_[e] == '+' || t_[e] == '.' || t_[e] == 'e' || t_[e] == 'E')) e++;
    if (e == p_) return false;
    const std::string num(t_ + p_, e - p_);
    char* end = nullptr;
    v.kind = Json::NUM; v.num = strtod(num.c_str(), &end);
    p_ = e;
    return end && *end == 0;
  }
  const char* t_; size_t n_, p_ = 0;
};

}  // namespace cai
