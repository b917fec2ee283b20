#include "checkpoint.hpp"

#include <errno.h>
#include <fcntl.h>
#include <limits.h>
#include <stdlib.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include "engine.hpp"

const Json* Json::find(const std::string& key) const {
  if (type != Object) return nullptr;
  for (const auto& m : members)
    if (m.first == key) return &m.second;
  return nullptr;
}

namespace {

struct Parser {
  const char* p;
  const char* end;
  std::string* err;
  int depth = 0;

  bool fail(const char* what) {
    if (err->empty()) *err = what;
    return false;
  }
  void space() {
    while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) ++p;
  }
  bool word(const char* w) {
    const size_t n = strlen(w);
    if ((size_t)(end - p) < n || memcmp(p, w, n) != 0) return fail("unexpected word");
    p += n;
    return true;
  }
  static void utf8(uint32_t c, std::string* s) {
    if (c < 0x80) {
      *s += (char)c;
    } else if (c < 0x800) {
      *s += (char)(0xc0 | (c >> 6));
      *s += (char)(0x80 | (c & 63));
    } else if (c < 0x10000) {
      *s += (char)(0xe0 | (c >> 12));
      *s += (char)(0x80 | ((c >> 6) & 63));
      *s += (char)(0x80 | (c & 63));
    } else {
      *s += (char)(0xf0 | (c >> 18));
      *s += (char)(0x80 | ((c >> 12) & 63));
      *s += (char)(0x80 | ((c >> 6) & 63));
      *s += (char)(0x80 | (c & 63));
    }
  }
  bool hex4(uint32_t* out) {
    if (end - p < 4) return fail("short \\u escape");
    uint32_t v = 0;
    for (int i = 0; i < 4; ++i) {
      const char c = *p++;
      v = v * 16 + (c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : 99);
      if (v > 0xffff) return fail("bad \\u escape");
    }
    *out = v;
    return true;
  }
  bool string(std::string* s) {
    if (p >= end || *p != '"') return fail("expected a string");
    ++p;
    for (;;) {
      if (p >= end) return fail("unterminated string");
      const unsigned char c = (unsigned char)*p++;
      if (c == '"') return true;
      if (c < 0x20) return fail("control character in a string");
      if (c != '\\') {
        *s += (char)c;
        continue;
      }
      if (p >= end) return fail("unterminated string");
      switch (*p++) {
        case '"': *s += '"'; break;
        case '\\': *s += '\\'; break;
        case '/': *s += '/'; break;
        case 'b': *s += '\b'; break;
        case 'f': *s += '\f'; break;
        case 'n': *s += '\n'; break;
        case 'r': *s += '\r'; break;
        case 't': *s += '\t'; break;
        case 'u': {
          uint32_t v, w;
          if (!hex4(&v)) return false;
          if (v >= 0xd800 && v < 0xdc00) {
            if (end - p < 2 || p[0] != '\\' || p[1] != 'u') return fail("lone surrogate");
            p += 2;
            if (!hex4(&w)) return false;
            if (w < 0xdc00 || w > 0xdfff) return fail("lone surrogate");
            v = 0x10000 + ((v - 0xd800) << 10) + (w - 0xdc00);
          }
          utf8(v, s);
          break;
        }
        default: return fail("unknown escape");
      }
    }
  }
  bool number(double* out) {
    const char* b = p;
    while (p < end && (strchr("+-.eE", *p) || (*p >= '0' && *p <= '9'))) ++p;
    const std::string t(b, p);
    char* stop = nullptr;
    *out = strtod(t.c_str(), &stop);
    if (t.empty() || *stop != 0) return fail("bad number");
    return true;
  }
  bool value(Json* v) {
    if (++depth > 64) return fail("nested too deeply");
    space();
    if (p >= end) return fail("unexpected end");
    bool ok = true;
    if (*p == '{') {
      v->type = Json::Object;
      ++p;
      space();
      if (p < end && *p == '}') {
        ++p;
      } else {
        for (;;) {
          v->members.emplace_back();
          space();
          if (!string(&v->members.back().first)) return false;
          space();
          if (p >= end || *p++ != ':') return fail("expected ':'");
          if (!value(&v->members.back().second)) return false;
          space();
          if (p >= end) return fail("unexpected end");
          const char c = *p++;
          if (c == '}') break;
          if (c != ',') return fail("expected ',' or '}'");
        }
      }
    } else if (*p == '[') {
      v->type = Json::Array;
      ++p;
      space();
      if (p < end && *p == ']') {
        ++p;
      } else {
        for (;;) {
          v->items.emplace_back();
          if (!value(&v->items.back())) return false;
          space();
          if (p >= end) return fail("unexpected end");
          const char c = *p++;
          if (c == ']') break;
          if (c != ',') return fail("expected ',' or ']'");
        }
      }
    } else if (*p == '"') {
      v->type = Json::String;
      ok = string(&v->str);
    } else if (*p == 't' || *p == 'f') {
      v->type = Json::Bool;
      v->boolean = *p == 't';
      ok = word(v->boolean ? "true" : "false");
    } else if (*p == 'n') {
      ok = word("null");
    } else {
      v->type = Json::Number;
      ok = number(&v->number);
    }
    --depth;
    return ok;
  }
};

}  // namespace

bool json_parse(const char* text, size_t n, Json* out, std::string* err) {
  *out = Json();
  err->clear();
  Parser ps{text, text + n, err};
  if (!ps.value(out)) return false;
  ps.space();
  return ps.p == ps.end || ps.fail("text behind the value");
}

int awq_read_json(const std::string& path, Json* out) {
  struct stat st;
  if (stat(path.c_str(), &st) != 0 || !S_ISREG(st.st_mode)) {
    awq_set_error("could not open " + path);
    return AWQ_ERR_IO;
  }
  std::string text((size_t)st.st_size, '\0'), err;
  if (int rc = awq_read_file(path, 0, (int64_t)text.size(), &text[0], &err)) {
    awq_set_error(err);
    return rc;
  }
  if (!json_parse(text.data(), text.size(), out, &err)) {
    awq_set_error(path + ": " + err);
    return AWQ_ERR_ARG;
  }
  return AWQ_OK;
}

int awq_config_architecture(const std::string& dir, std::string* out) {
  Json j;
  if (int rc = awq_read_json(dir + "/config.json", &j)) return rc;
  const Json* a = j.find("architecture");
  if (!a || !a->is(Json::String)) {
    awq_set_error(dir + "/config.json names no architecture");
    return AWQ_ERR_ARG;
  }
  *out = a->str;
  return AWQ_OK;
}

Safetensors::~Safetensors() {
  if (map_) munmap(map_, size_);
}

int Safetensors::open(const std::string& path) {
  const auto bad = [&](const std::string& why) {
    awq_set_error(path + ": " + why);
    return AWQ_ERR_IO;
  };
  const int fd = ::open(path.c_str(), O_RDONLY);
  if (fd < 0) return bad(std::string("could not open: ") + strerror(errno));
  struct stat st;
  if (fstat(fd, &st) != 0 || st.st_size < 8) {
    close(fd);
    return bad("too short");
  }
  size_ = (size_t)st.st_size;
  void* m = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
  close(fd);
  if (m == MAP_FAILED) return bad("could not be mapped");
  map_ = m;
  const uint8_t* base = (const uint8_t*)m;
  uint64_t header = 0;
  for (int i = 7; i >= 0; --i) header = header << 8 | base[i];
  if (header > size_ - 8) return bad("the header does not fit the file");
  Json j;
  std::string err;
  if (!json_parse((const char*)base + 8, (size_t)header, &j, &err) || !j.is(Json::Object)) return bad("header: " + err);
  const uint64_t room = size_ - 8 - header;
  for (const auto& m2 : j.members) {
    if (m2.first == "__metadata__") continue;
    const Json *dt = m2.second.find("dtype"), *sh = m2.second.find("shape"), *off = m2.second.find("data_offsets");
    if (!dt || !sh || !off || off->items.size() != 2) return bad("entry of " + m2.first + " is incomplete");
    Tensor t;
    t.dtype = dt->str;
    double n = 1.0;
    for (const Json& d : sh->items) {
      if (!(d.number >= 0.0 && d.number < 1e15)) return bad("shape of " + m2.first);
      t.shape.push_back((int64_t)d.number);
      n *= d.number;
    }
    const double b = off->items[0].number, e = off->items[1].number;
    if (!(b >= 0.0 && e >= b && e <= (double)room)) return bad("offsets of " + m2.first + " lie outside the file");
    const int unit = t.dtype == "BF16" || t.dtype == "F16" ? 2 : t.dtype == "F32" || t.dtype == "I32" ? 4 : 0;
    if (unit && n * unit != e - b) return bad("size of " + m2.first + " does not fit its shape");
    t.data = base + 8 + header + (uint64_t)b;
    t.bytes = (int64_t)(e - b);
    tensors_.emplace(m2.first, std::move(t));
  }
  return AWQ_OK;
}

const Tensor* Safetensors::find(const std::string& name) const {
  const auto it = tensors_.find(name);
  return it == tensors_.end() ? nullptr : &it->second;
}
