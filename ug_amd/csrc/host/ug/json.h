// A JSON reader for what this library reads: safetensors headers and model configurations.
#pragma once
#include <cstdint>
#include <cstdlib>
#include <cstring>
#include <limits>
#include <string>
#include <utility>
#include <vector>

#include "core.h"

namespace ug {

struct Json {
  enum Kind { Null, Bool, Num, Str, Arr, Obj } kind = Null;
  double num = 0;
  bool is_uint = false;
  uint64_t uint = 0;
  std::string str;
  std::vector<Json> arr;
  std::vector<std::pair<std::string, Json>> obj;

  bool is_null() const { return kind == Null; }
  // A member of an object, or nullptr (absent members and null are alike to a configuration).
  const Json* find(const std::string& key) const {
    for (const auto& kv : obj)
      if (kv.first == key) return kv.second.is_null() ? nullptr : &kv.second;
    return nullptr;
  }
  const Json& at(const std::string& key) const {
    const Json* j = find(key);
    if (!j) bail("configuration: '" + key + "' is missing");
    return *j;
  }
  size_t size_at(const std::string& key) const {
    const Json& j = at(key);
    if (j.kind != Num || !j.is_uint) bail("configuration: '" + key + "' is not a non-negative integer");
    return (size_t)j.uint;
  }
  size_t size_or(const std::string& key, size_t dflt) const { return find(key) ? size_at(key) : dflt; }
  double num_at(const std::string& key) const {
    const Json& j = at(key);
    if (j.kind != Num) bail("configuration: '" + key + "' is not a number");
    return j.num;
  }
  double num_or(const std::string& key, double dflt) const { return find(key) ? num_at(key) : dflt; }
  const std::string& str_at(const std::string& key) const {
    const Json& j = at(key);
    if (j.kind != Str) bail("configuration: '" + key + "' is not a string");
    return j.str;
  }
};

struct JsonParser {
  const char* p;
  const char* end;
  std::string what;  // starts every error message
  [[noreturn]] void fail(const std::string& why) const { bail(what + ": " + why); }
  void ws() {
    while (p < end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) ++p;
  }
  char peek() {
    ws();
    if (p >= end) fail("unexpected end");
    return *p;
  }
  void expect(char c) {
    if (peek() != c) fail(std::string("expected '") + c + "'");
    ++p;
  }
  std::string string() {
    expect('"');
    std::string out;
    while (true) {
      if (p >= end) fail("unterminated string");
      char c = *p++;
      if (c == '"') break;
      if (c != '\\') {
        out.push_back(c);
        continue;
      }
      if (p >= end) fail("unterminated escape");
      char e = *p++;
      switch (e) {
        case '"': out.push_back('"'); break;
        case '\\': out.push_back('\\'); break;
        case '/': out.push_back('/'); break;
        case 'b': out.push_back('\b'); break;
        case 'f': out.push_back('\f'); break;
        case 'n': out.push_back('\n'); break;
        case 'r': out.push_back('\r'); break;
        case 't': out.push_back('\t'); break;
        case 'u': {
          if (end - p < 4) fail("short \\u escape");
          unsigned cp = 0;
          for (int i = 0; i < 4; ++i) {
            char h = *p++;
            cp <<= 4;
            if (h >= '0' && h <= '9') cp |= (unsigned)(h - '0');
            else if (h >= 'a' && h <= 'f') cp |= (unsigned)(h - 'a' + 10);
            else if (h >= 'A' && h <= 'F') cp |= (unsigned)(h - 'A' + 10);
            else fail("bad \\u escape");
          }
          // UTF-8 encode the BMP code point (surrogate pairs are kept as two 3-byte sequences)
          if (cp < 0x80) out.push_back((char)cp);
          else if (cp < 0x800) {
            out.push_back((char)(0xC0 | (cp >> 6)));
            out.push_back((char)(0x80 | (cp & 0x3F)));
          } else {
            out.push_back((char)(0xE0 | (cp >> 12)));
            out.push_back((char)(0x80 | ((cp >> 6) & 0x3F)));
            out.push_back((char)(0x80 | (cp & 0x3F)));
          }
          break;
        }
        default: fail("bad escape");
      }
    }
    return out;
  }
  Json value(int depth) {
    if (depth > 16) fail("nesting too deep");
    Json j;
    char c = peek();
    if (c == '{') {
      ++p;
      j.kind = Json::Obj;
      if (peek() == '}') {
        ++p;
        return j;
      }
      while (true) {
        std::string k = string();
        expect(':');
        j.obj.emplace_back(std::move(k), value(depth + 1));
        char d = peek();
        ++p;
        if (d == '}') break;
        if (d != ',') fail("expected ',' or '}'");
        ws();
      }
    } else if (c == '[') {
      ++p;
      j.kind = Json::Arr;
      if (peek() == ']') {
        ++p;
        return j;
      }
      while (true) {
        j.arr.push_back(value(depth + 1));
        char d = peek();
        ++p;
        if (d == ']') break;
        if (d != ',') fail("expected ',' or ']'");
      }
    } else if (c == '"') {
      j.kind = Json::Str;
      j.str = string();
    } else if (c == 't' && end - p >= 4 && !strncmp(p, "true", 4)) {
      p += 4;
      j.kind = Json::Bool;
      j.num = 1;
    } else if (c == 'f' && end - p >= 5 && !strncmp(p, "false", 5)) {
      p += 5;
      j.kind = Json::Bool;
    } else if (c == 'n' && end - p >= 4 && !strncmp(p, "null", 4)) {
      p += 4;
    } else if (c == '-' || (c >= '0' && c <= '9')) {
      const char* s = p;
      bool all_digits = true;
      uint64_t u = 0;
      bool overflow = false;
      while (p < end && (*p == '-' || *p == '+' || *p == '.' || *p == 'e' || *p == 'E' || (*p >= '0' && *p <= '9'))) {
        if (*p >= '0' && *p <= '9') {
          if (u > (std::numeric_limits<uint64_t>::max() - (uint64_t)(*p - '0')) / 10) overflow = true;
          u = u * 10 + (uint64_t)(*p - '0');
        } else {
          all_digits = false;
        }
        ++p;
      }
      j.kind = Json::Num;
      j.num = strtod(std::string(s, p).c_str(), nullptr);
      j.is_uint = all_digits && !overflow;
      j.uint = u;
    } else {
      fail(std::string("unexpected character '") + c + "'");
    }
    return j;
  }
};

}  // namespace ug
