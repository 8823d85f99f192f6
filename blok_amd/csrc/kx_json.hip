// kx_json.hip -- see kx_json.h.
#include <errno.h>
#include <math.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>
#include "kx_common.h"
#include "kx_json.h"

namespace {

struct Reader {
  const char *p, *begin, *end;
  std::string &err;
  int depth = 0;

  bool fail(const char *what) {
    if (err.empty()) err = std::string(what) + " at byte " + std::to_string(p - begin);
    return false;
  }
  void space() {
    while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) ++p;
  }
  bool word(const char *w) {
    const size_t n = strlen(w);
    if ((size_t)(end - p) < n || memcmp(p, w, n)) return fail("unknown word");
    p += n;
    return true;
  }
  bool hex4(uint32_t &v) {
    if (end - p < 4) return fail("short \\u escape");
    v = 0;
    for (int i = 0; i < 4; ++i, ++p) {
      const char c = *p;
      const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
      if (d < 0) return fail("bad \\u escape");
      v = v * 16 + (uint32_t)d;
    }
    return true;
  }
  void utf8(uint32_t c, std::string &s) {
    if (c < 0x80) { s += (char)c; return; }
    if (c < 0x800) { s += (char)(0xc0 | (c >> 6)); s += (char)(0x80 | (c & 63)); return; }
    if (c < 0x10000) { s += (char)(0xe0 | (c >> 12)); s += (char)(0x80 | ((c >> 6) & 63)); s += (char)(0x80 | (c & 63)); return; }
    s += (char)(0xf0 | (c >> 18)); s += (char)(0x80 | ((c >> 12) & 63)); s += (char)(0x80 | ((c >> 6) & 63)); s += (char)(0x80 | (c & 63));
  }
  bool string(std::string &s) {
    ++p;  // the opening quote
    while (p < end && *p != '"') {
      if ((unsigned char)*p < 0x20) return fail("control character in a string");
      if (*p != '\\') { s += *p++; continue; }
      if (++p == end) return fail("unfinished escape");
      const char c = *p++;
      switch (c) {
        case '"': case '\\': case '/': s += c; break;
        case 'b': s += '\b'; break;
        case 'f': s += '\f'; break;
        case 'n': s += '\n'; break;
        case 'r': s += '\r'; break;
        case 't': s += '\t'; break;
        case 'u': {
          uint32_t v, lo;
          if (!hex4(v)) return false;
          if (v >= 0xd800 && v < 0xdc00) {
            if (end - p < 2 || p[0] != '\\' || p[1] != 'u') return fail("lone surrogate");
            p += 2;
            if (!hex4(lo)) return false;
            if (lo < 0xdc00 || lo > 0xdfff) return fail("lone surrogate");
            v = 0x10000 + ((v - 0xd800) << 10) + (lo - 0xdc00);
          }
          utf8(v, s);
          break;
        }
        default: return fail("unknown escape");
      }
    }
    if (p == end) return fail("unfinished string");
    ++p;
    return true;
  }
  bool number(double &v) {
    const char *q = p;
    while (q < end && (*q == '-' || *q == '+' || *q == '.' || *q == 'e' || *q == 'E' || (*q >= '0' && *q <= '9'))) ++q;
    const std::string t(p, q);  // strtod needs a terminator
    char *stop = nullptr;
    v = strtod(t.c_str(), &stop);
    if (t.empty() || *stop || !isfinite(v)) return fail("bad number");
    p = q;
    return true;
  }
  bool value(KxJson &out) {
    if (++depth > 64) return fail("nested too deep");
    space();
    if (p == end) return fail("unexpected end");
    bool ok = true;
    if (*p == '{') {
      out.kind = KxJson::OBJECT;
      ++p;
      space();
      if (p < end && *p == '}') ++p;
      else for (;;) {
        space();
        if (p == end || *p != '"') return fail("expected a member name");
        out.members.emplace_back();
        if (!string(out.members.back().first)) return false;
        space();
        if (p == end || *p != ':') return fail("expected ':'");
        ++p;
        KxJson v;
        if (!value(v)) return false;
        out.members.back().second = std::move(v);
        space();
        if (p < end && *p == ',') { ++p; continue; }
        if (p < end && *p == '}') { ++p; break; }
        return fail("expected ',' or '}'");
      }
    } else if (*p == '[') {
      out.kind = KxJson::ARRAY;
      ++p;
      space();
      if (p < end && *p == ']') ++p;
      else for (;;) {
        KxJson v;
        if (!value(v)) return false;
        out.items.push_back(std::move(v));
        space();
        if (p < end && *p == ',') { ++p; continue; }
        if (p < end && *p == ']') { ++p; break; }
        return fail("expected ',' or ']'");
      }
    } else if (*p == '"') {
      out.kind = KxJson::STRING;
      ok = string(out.str);
    } else if (*p == 't') {
      out.kind = KxJson::BOOL; out.b = true;
      ok = word("true");
    } else if (*p == 'f') {
      out.kind = KxJson::BOOL;
      ok = word("false");
    } else if (*p == 'n') {
      ok = word("null");
    } else {
      out.kind = KxJson::NUMBER;
      ok = number(out.num);
    }
    --depth;
    return ok;
  }
};

}  // namespace

const KxJson *KxJson::get(const char *key) const {
  for (const auto &m : members)
    if (m.first == key) return &m.second;
  return nullptr;
}

bool kx_json_parse(const char *text, size_t len, KxJson &out, std::string &err) {
  err.clear();
  out = KxJson();
  Reader r{text, text, text + len, err};
  if (!r.value(out)) return false;
  r.space();
  return r.p == r.end ? true : r.fail("text after the document");
}

int kx_json_file(const std::string &path, KxJson &out) {
  FILE *f = fopen(path.c_str(), "rb");
  KX_REQUIRE(f, "cannot open %s: %s", path.c_str(), strerror(errno));
  std::string text;
  char buf[65536];
  size_t n;
  while ((n = fread(buf, 1, sizeof buf, f)) > 0) text.append(buf, n);
  fclose(f);
  std::string err;
  KX_REQUIRE(kx_json_parse(text.data(), text.size(), out, err), "%s: %s", path.c_str(), err.c_str());
  return KX_OK;
}
