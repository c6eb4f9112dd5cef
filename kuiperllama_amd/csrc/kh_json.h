// kh_json.h — JSON reading (host only): a streaming reader for large documents whose members are picked out one by
// one (tokenizer.json, the header of a safetensors file), and a small value tree on top of it for configurations.
#pragma once
#include <stdint.h>
#include <stdlib.h>

#include <string>
#include <utility>
#include <vector>

namespace khm {

// ---- UTF-8 ---------------------------------------------------------------------------------------
// decodes one code point at s[i]; malformed bytes come back as themselves (length 1), which keeps
// the scanner total: such a byte is "other" for the pattern and goes through the byte-level BPE.
inline uint32_t utf8_next(const std::string& s, size_t i, size_t* len) {
  const unsigned char c = (unsigned char)s[i];
  auto cont = [&](size_t k) { return i + k < s.size() && ((unsigned char)s[i + k] & 0xC0) == 0x80; };
  if (c < 0x80) {
    *len = 1;
    return c;
  }
  if ((c & 0xE0) == 0xC0 && cont(1)) {
    *len = 2;
    return ((c & 0x1Fu) << 6) | ((unsigned char)s[i + 1] & 0x3Fu);
  }
  if ((c & 0xF0) == 0xE0 && cont(1) && cont(2)) {
    *len = 3;
    return ((c & 0x0Fu) << 12) | (((unsigned char)s[i + 1] & 0x3Fu) << 6) | ((unsigned char)s[i + 2] & 0x3Fu);
  }
  if ((c & 0xF8) == 0xF0 && cont(1) && cont(2) && cont(3)) {
    *len = 4;
    return ((c & 0x07u) << 18) | (((unsigned char)s[i + 1] & 0x3Fu) << 12) |
           (((unsigned char)s[i + 2] & 0x3Fu) << 6) | ((unsigned char)s[i + 3] & 0x3Fu);
  }
  *len = 1;
  return 0xFFFD0000u | c;  // not a code point: classified as "other"
}
inline void utf8_put(std::string& out, uint32_t cp) {
  if (cp < 0x80) {
    out += (char)cp;
  } else if (cp < 0x800) {
    out += (char)(0xC0 | (cp >> 6));
    out += (char)(0x80 | (cp & 0x3F));
  } else if (cp < 0x10000) {
    out += (char)(0xE0 | (cp >> 12));
    out += (char)(0x80 | ((cp >> 6) & 0x3F));
    out += (char)(0x80 | (cp & 0x3F));
  } else {
    out += (char)(0xF0 | (cp >> 18));
    out += (char)(0x80 | ((cp >> 12) & 0x3F));
    out += (char)(0x80 | ((cp >> 6) & 0x3F));
    out += (char)(0x80 | (cp & 0x3F));
  }
}

// ---- reader: walks a document without building it (tokenizer.json, safetensors headers) ----------
struct Json {
  const char* p;
  const char* end;
  bool ok = true;
  void ws() {
    while (p < end && (*p == ' ' || *p == '\n' || *p == '\r' || *p == '\t')) ++p;
  }
  bool eat(char c) {
    ws();
    if (p < end && *p == c) {
      ++p;
      return true;
    }
    return false;
  }
  bool peek(char c) {
    ws();
    return p < end && *p == c;
  }
  static int hex4(const char* q) {
    int v = 0;
    for (int i = 0; i < 4; ++i) {
      const char c = q[i];
      v <<= 4;
      if (c >= '0' && c <= '9') v |= c - '0';
      else if (c >= 'a' && c <= 'f') v |= c - 'a' + 10;
      else if (c >= 'A' && c <= 'F') v |= c - 'A' + 10;
      else return -1;
    }
    return v;
  }
  bool str(std::string* out) {  // out may be null (skip)
    ws();
    if (p >= end || *p != '"') return ok = false;
    ++p;
    while (p < end && *p != '"') {
      if (*p == '\\') {
        if (p + 1 >= end) return ok = false;
        const char e = p[1];
        p += 2;
        uint32_t cp;
        switch (e) {
          case 'n': cp = '\n'; break;
          case 't': cp = '\t'; break;
          case 'r': cp = '\r'; break;
          case 'b': cp = '\b'; break;
          case 'f': cp = '\f'; break;
          case 'u': {
            if (p + 4 > end) return ok = false;
            int v = hex4(p);
            if (v < 0) return ok = false;
            p += 4;
            cp = (uint32_t)v;
            if (cp >= 0xD800 && cp < 0xDC00 && p + 6 <= end && p[0] == '\\' && p[1] == 'u') {
              const int lo = hex4(p + 2);
              if (lo >= 0xDC00 && lo < 0xE000) {
                cp = 0x10000 + ((cp - 0xD800) << 10) + ((uint32_t)lo - 0xDC00);
                p += 6;
              }
            }
            break;
          }
          default: cp = (unsigned char)e; break;  // \" \\ \/
        }
        if (out) utf8_put(*out, cp);
      } else {
        if (out) *out += *p;
        ++p;
      }
    }
    if (p >= end) return ok = false;
    ++p;
    return true;
  }
  bool integer(long* v) {
    // digits parsed by hand, bounded by `end`: the buffer (kh_bpe_create_from_memory's ptr/nbytes)
    // is not NUL-terminated, so strtol could read past a file that is truncated inside a number
    ws();
    const char* q = p;
    bool neg = false;
    if (q < end && (*q == '-' || *q == '+')) neg = *q++ == '-';
    if (q >= end || *q < '0' || *q > '9') return ok = false;
    long x = 0;
    while (q < end && *q >= '0' && *q <= '9') {
      if (x > (0x7fffffffL - 9) / 10) return ok = false;  // ids are int32
      x = x * 10 + (*q++ - '0');
    }
    // a fraction / exponent would not be an id
    p = q;
    if (v) *v = neg ? -x : x;
    return true;
  }
  bool skip() {  // any value
    ws();
    if (p >= end) return ok = false;
    if (*p == '"') return str(nullptr);
    if (*p == '{') {
      ++p;
      if (eat('}')) return true;
      do {
        if (!str(nullptr) || !eat(':') || !skip()) return ok = false;
      } while (eat(','));
      return eat('}') ? true : (ok = false);
    }
    if (*p == '[') {
      ++p;
      if (eat(']')) return true;
      do {
        if (!skip()) return ok = false;
      } while (eat(','));
      return eat(']') ? true : (ok = false);
    }
    while (p < end && *p != ',' && *p != '}' && *p != ']' && *p != ' ' && *p != '\n' && *p != '\r' && *p != '\t') ++p;
    return true;  // number / true / false / null
  }
  // iterate the members of an object: fn(key) must consume the value
  template <class F>
  bool object(F&& fn) {
    if (!eat('{')) return ok = false;
    if (eat('}')) return true;
    do {
      std::string key;
      if (!str(&key) || !eat(':')) return ok = false;
      if (!fn(key)) return ok = false;
    } while (eat(','));
    return eat('}') ? true : (ok = false);
  }
};


// ---- value tree (config.json) --------------------------------------------------------------------
struct JsonValue {
  enum Kind { NUL, BOOL, NUM, STR, ARR, OBJ } kind = NUL;
  bool b = false;
  double num = 0;
  std::string s;
  std::vector<JsonValue> arr;
  std::vector<std::pair<std::string, JsonValue>> obj;

  const JsonValue* get(const char* key) const {  // nullptr: no such member (or null)
    for (const auto& kv : obj)
      if (kv.first == key) return kv.second.kind == NUL ? nullptr : &kv.second;
    return nullptr;
  }
  double number(const char* key, double dflt) const {
    const JsonValue* v = get(key);
    return v && v->kind == NUM ? v->num : dflt;
  }
  int integer(const char* key, int dflt) const { return (int)number(key, (double)dflt); }
  std::string text(const char* key) const {
    const JsonValue* v = get(key);
    return v && v->kind == STR ? v->s : std::string();
  }
};

inline bool json_parse(Json& j, JsonValue* v, int depth = 0) {
  if (depth > 64) return j.ok = false;
  j.ws();
  if (j.p >= j.end) return j.ok = false;
  if (*j.p == '"') {
    v->kind = JsonValue::STR;
    return j.str(&v->s);
  }
  if (*j.p == '{') {
    v->kind = JsonValue::OBJ;
    return j.object([&](const std::string& key) {
      v->obj.emplace_back(key, JsonValue());
      return json_parse(j, &v->obj.back().second, depth + 1);
    });
  }
  if (*j.p == '[') {
    v->kind = JsonValue::ARR;
    ++j.p;
    if (j.eat(']')) return true;
    do {
      v->arr.emplace_back();
      if (!json_parse(j, &v->arr.back(), depth + 1)) return j.ok = false;
    } while (j.eat(','));
    return j.eat(']') ? true : (j.ok = false);
  }
  const char* q = j.p;  // number / true / false / null
  if (!j.skip()) return false;
  const std::string t(q, (size_t)(j.p - q));
  if (t == "null") return true;
  if (t == "true" || t == "false") {
    v->kind = JsonValue::BOOL;
    v->b = t == "true";
    return true;
  }
  char* e = nullptr;
  v->kind = JsonValue::NUM;
  v->num = strtod(t.c_str(), &e);
  return e && *e == 0 && e != t.c_str() ? true : (j.ok = false);
}

}  // namespace khm
