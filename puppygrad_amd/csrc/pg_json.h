// The JSON reader of the host-side translation units (safetensors headers, config.json,
// puppygrad-tune.json).
#pragma once

#include <cstdint>
#include <cstdlib>
#include <cstring>
#include <string>
#include <utility>
#include <vector>

#include "pg_internal.h"

namespace pgh {

// ---------------------------------------------------------------------------
// A small JSON reader (RFC 8259): enough for a safetensors header and config.json.
// ---------------------------------------------------------------------------
struct Json {
  enum Kind { Null, Bool, Num, Str, Arr, Obj } kind = Null;
  bool b = false;
  double num = 0.0;
  bool integral = false;  // written without fraction or exponent, and not negative
  uint64_t u = 0;         // its value when integral
  std::string str;
  std::vector<Json> arr;
  std::vector<std::pair<std::string, Json>> obj;  // file order; a later duplicate wins in find()

  const Json* find(const std::string& key) const {
    const Json* hit = nullptr;
    for (const auto& kv : obj)
      if (kv.first == key) hit = &kv.second;
    return hit;
  }
};

class JsonParser {
 public:
  JsonParser(const char* b, const char* e) : begin_(b), p_(b), e_(e) {}

  bool parse(Json& out, std::string& err) {
    bool ok = value(out, 0);
    if (ok) {
      ws();
      if (p_ != e_) ok = bad("trailing characters");
    }
    if (!ok) err = err_ + " at " + where();
    return ok;
  }

 private:
  const char* begin_;
  const char* p_;
  const char* e_;
  std::string err_;

  std::string where() const {
    size_t line = 1, col = 1;
    for (const char* q = begin_; q < p_; ++q) {
      if (*q == '\n') {
        ++line;
        col = 1;
      } else {
        ++col;
      }
    }
    return "line " + std::to_string(line) + " column " + std::to_string(col);
  }
  void ws() {
    while (p_ < e_ && (*p_ == ' ' || *p_ == '\t' || *p_ == '\n' || *p_ == '\r')) ++p_;
  }
  bool bad(const char* what) {
    err_ = what;
    return false;
  }
  bool literal(const char* word) {
    const size_t n = std::strlen(word);
    if ((size_t)(e_ - p_) < n || std::memcmp(p_, word, n) != 0) return bad("expected value");
    p_ += n;
    return true;
  }
  static void utf8(std::string& s, uint32_t cp) {
    if (cp < 0x80) {
      s += (char)cp;
    } else if (cp < 0x800) {
      s += (char)(0xC0 | (cp >> 6));
      s += (char)(0x80 | (cp & 0x3F));
    } else if (cp < 0x10000) {
      s += (char)(0xE0 | (cp >> 12));
      s += (char)(0x80 | ((cp >> 6) & 0x3F));
      s += (char)(0x80 | (cp & 0x3F));
    } else {
      s += (char)(0xF0 | (cp >> 18));
      s += (char)(0x80 | ((cp >> 12) & 0x3F));
      s += (char)(0x80 | ((cp >> 6) & 0x3F));
      s += (char)(0x80 | (cp & 0x3F));
    }
  }
  bool hex4(uint32_t& v) {
    if (e_ - p_ < 4) return bad("EOF while parsing a string");
    v = 0;
    for (int i = 0; i < 4; ++i) {
      const char c = *p_++;
      v <<= 4;
      if (c >= '0' && c <= '9') v |= (uint32_t)(c - '0');
      else if (c >= 'a' && c <= 'f') v |= (uint32_t)(c - 'a' + 10);
      else if (c >= 'A' && c <= 'F') v |= (uint32_t)(c - 'A' + 10);
      else return bad("invalid escape");
    }
    return true;
  }
  bool string(std::string& out) {
    ++p_;  // opening quote
    out.clear();
    while (true) {
      if (p_ == e_) return bad("EOF while parsing a string");
      const unsigned char c = (unsigned char)*p_++;
      if (c == '"') return true;
      if (c < 0x20) return bad("control character found while parsing a string");
      if (c != '\\') {
        out += (char)c;
        continue;
      }
      if (p_ == e_) return bad("EOF while parsing a string");
      const char esc = *p_++;
      switch (esc) {
        case '"': out += '"'; break;
        case '\\': out += '\\'; break;
        case '/': out += '/'; break;
        case 'b': out += '\b'; break;
        case 'f': out += '\f'; break;
        case 'n': out += '\n'; break;
        case 'r': out += '\r'; break;
        case 't': out += '\t'; break;
        case 'u': {
          uint32_t cp;
          if (!hex4(cp)) return false;
          if (cp >= 0xD800 && cp < 0xDC00) {
            uint32_t lo;
            if (e_ - p_ < 2 || p_[0] != '\\' || p_[1] != 'u') return bad("lone leading surrogate");
            p_ += 2;
            if (!hex4(lo)) return false;
            if (lo < 0xDC00 || lo > 0xDFFF) return bad("lone leading surrogate");
            cp = 0x10000 + ((cp - 0xD800) << 10) + (lo - 0xDC00);
          } else if (cp >= 0xDC00 && cp <= 0xDFFF) {
            return bad("lone trailing surrogate");
          }
          utf8(out, cp);
          break;
        }
        default: return bad("invalid escape");
      }
    }
  }
  bool number(Json& out) {
    const char* s = p_;
    bool neg = false, frac = false;
    if (p_ < e_ && *p_ == '-') {
      neg = true;
      ++p_;
    }
    if (p_ == e_ || *p_ < '0' || *p_ > '9') return bad("invalid number");
    if (*p_ == '0') {
      ++p_;
    } else {
      while (p_ < e_ && *p_ >= '0' && *p_ <= '9') ++p_;
    }
    if (p_ < e_ && *p_ == '.') {
      frac = true;
      ++p_;
      if (p_ == e_ || *p_ < '0' || *p_ > '9') return bad("invalid number");
      while (p_ < e_ && *p_ >= '0' && *p_ <= '9') ++p_;
    }
    if (p_ < e_ && (*p_ == 'e' || *p_ == 'E')) {
      frac = true;
      ++p_;
      if (p_ < e_ && (*p_ == '+' || *p_ == '-')) ++p_;
      if (p_ == e_ || *p_ < '0' || *p_ > '9') return bad("invalid number");
      while (p_ < e_ && *p_ >= '0' && *p_ <= '9') ++p_;
    }
    const std::string text(s, p_);
    out.kind = Json::Num;
    out.num = std::strtod(text.c_str(), nullptr);
    out.integral = false;
    if (!neg && !frac && text.size() <= 19) {  // 19 digits always fit 64 bits
      out.integral = true;
      out.u = std::strtoull(text.c_str(), nullptr, 10);
    }
    return true;
  }
  bool value(Json& out, int depth) {
    if (depth > 128) return bad("recursion limit exceeded");
    ws();
    if (p_ == e_) return bad("EOF while parsing a value");
    switch (*p_) {
      case '{': {
        ++p_;
        out.kind = Json::Obj;
        ws();
        if (p_ < e_ && *p_ == '}') {
          ++p_;
          return true;
        }
        while (true) {
          ws();
          if (p_ == e_ || *p_ != '"') return bad("key must be a string");
          std::string key;
          if (!string(key)) return false;
          ws();
          if (p_ == e_ || *p_ != ':') return bad("expected `:`");
          ++p_;
          Json v;
          if (!value(v, depth + 1)) return false;
          out.obj.emplace_back(std::move(key), std::move(v));
          ws();
          if (p_ < e_ && *p_ == ',') {
            ++p_;
            continue;
          }
          if (p_ < e_ && *p_ == '}') {
            ++p_;
            return true;
          }
          return bad("expected `,` or `}`");
        }
      }
      case '[': {
        ++p_;
        out.kind = Json::Arr;
        ws();
        if (p_ < e_ && *p_ == ']') {
          ++p_;
          return true;
        }
        while (true) {
          Json v;
          if (!value(v, depth + 1)) return false;
          out.arr.push_back(std::move(v));
          ws();
          if (p_ < e_ && *p_ == ',') {
            ++p_;
            continue;
          }
          if (p_ < e_ && *p_ == ']') {
            ++p_;
            return true;
          }
          return bad("expected `,` or `]`");
        }
      }
      case '"':
        out.kind = Json::Str;
        return string(out.str);
      case 't':
        out.kind = Json::Bool;
        out.b = true;
        return literal("true");
      case 'f':
        out.kind = Json::Bool;
        out.b = false;
        return literal("false");
      case 'n':
        out.kind = Json::Null;
        return literal("null");
      default:
        if (*p_ == '-' || (*p_ >= '0' && *p_ <= '9')) return number(out);
        return bad("expected value");
    }
  }
};

// Reads and parses `path` (a JSON object).  Failures are PG_ASSET, worded as the reference's
// ConfigLoadError (src/models/config.rs:19-29): "failed to read {what} {path}: ...".
__attribute__((visibility("hidden"))) pg_status read_json_file(const std::string& path, const char* what, Json* out);

}  // namespace pgh
