#include "json.hpp"

#include <cmath>
#include <cstdlib>

namespace llama_cu {

namespace {

const json NOTHING;

struct reader {
  std::string_view s;
  size_t at{0};
  std::string error;

  bool fail(const char* what) {
    if (error.empty()) error = std::string(what) + " at byte " + std::to_string(at);
    return false;
  }
  void space() {
    while (at < s.size() && (s[at] == ' ' || s[at] == '\t' || s[at] == '\n' || s[at] == '\r')) ++at;
  }
  bool word(std::string_view w) {
    if (s.substr(at, w.size()) != w) return fail("unknown word");
    at += w.size();
    return true;
  }
  bool hex4(uint32_t& v) {
    if (at + 4 > s.size()) return fail("short escape");
    v = 0;
    for (int i = 0; i < 4; ++i) {
      const char c = s[at++];
      const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
      if (d < 0) return fail("bad escape");
      v = v * 16 + (uint32_t)d;
    }
    return true;
  }
  static void put_utf8(std::string& out, uint32_t c) {
    if (c < 0x80) {
      out += (char)c;
    } else if (c < 0x800) {
      out += (char)(0xC0 | c >> 6);
      out += (char)(0x80 | (c & 63));
    } else if (c < 0x10000) {
      out += (char)(0xE0 | c >> 12);
      out += (char)(0x80 | (c >> 6 & 63));
      out += (char)(0x80 | (c & 63));
    } else {
      out += (char)(0xF0 | c >> 18);
      out += (char)(0x80 | (c >> 12 & 63));
      out += (char)(0x80 | (c >> 6 & 63));
      out += (char)(0x80 | (c & 63));
    }
  }
  bool quoted(std::string& out) {
    ++at;  // the opening quote
    while (at < s.size() && s[at] != '"') {
      if (s[at] != '\\') {
        out += s[at++];
        continue;
      }
      if (++at >= s.size()) break;
      const char c = s[at++];
      uint32_t v, low;
      switch (c) {
        case 'b': out += '\b'; break;
        case 'f': out += '\f'; break;
        case 'n': out += '\n'; break;
        case 'r': out += '\r'; break;
        case 't': out += '\t'; break;
        case '"': case '\\': case '/': out += c; break;
        case 'u':
          if (!hex4(v)) return false;
          if (v >= 0xD800 && v < 0xDC00 && s.substr(at, 2) == "\\u") {  // a surrogate pair
            at += 2;
            if (!hex4(low)) return false;
            v = 0x10000 + ((v - 0xD800) << 10) + (low - 0xDC00);
          }
          put_utf8(out, v);
          break;
        default: return fail("bad escape");
      }
    }
    if (at >= s.size()) return fail("unended string");
    ++at;
    return true;
  }
  bool value(json& v, int depth) {
    if (depth > 64) return fail("nested too deep");
    space();
    if (at >= s.size()) return fail("unexpected end");
    const char c = s[at];
    if (c == '{' || c == '[') {
      const bool obj = c == '{';
      const char close = obj ? '}' : ']';
      v.kind = obj ? json::object : json::array;
      ++at;
      space();
      if (at < s.size() && s[at] == close) {
        ++at;
        return true;
      }
      while (true) {
        space();
        std::string key;
        if (obj) {
          if (at >= s.size() || s[at] != '"') return fail("expected a name");
          if (!quoted(key)) return false;
          space();
          if (at >= s.size() || s[at] != ':') return fail("expected a colon");
          ++at;
        }
        json item;
        if (!value(item, depth + 1)) return false;
        if (obj) {
          v.members.emplace_back(std::move(key), std::move(item));
        } else {
          v.items.push_back(std::move(item));
        }
        space();
        if (at < s.size() && s[at] == ',') {
          ++at;
          continue;
        }
        if (at < s.size() && s[at] == close) {
          ++at;
          return true;
        }
        return fail("expected a comma or the end of the list");
      }
    }
    if (c == '"') {
      v.kind = json::string;
      return quoted(v.text);
    }
    if (c == 't' || c == 'f') {
      v.kind = json::boolean;
      v.flag = c == 't';
      return word(v.flag ? "true" : "false");
    }
    if (c == 'n') return word("null");
    size_t end = at;
    while (end < s.size() && (s[end] == '-' || s[end] == '+' || s[end] == '.' || s[end] == 'e' || s[end] == 'E' ||
                              (s[end] >= '0' && s[end] <= '9'))) {
      ++end;
    }
    if (end == at) return fail("unexpected character");
    const std::string digits(s.substr(at, end - at));
    char* stop = nullptr;
    v.kind = json::number;
    v.num = strtod(digits.c_str(), &stop);
    if (stop != digits.c_str() + digits.size()) return fail("bad number");
    at = end;
    return true;
  }
};

}  // namespace

bool json::parse(std::string_view text, json& out, std::string& error) {
  reader r{text, 0, {}};
  out = json();
  bool ok = r.value(out, 0);
  if (ok) {
    r.space();
    ok = r.at == text.size() || r.fail("text after the value");
  }
  error = r.error;
  return ok;
}

json const& json::operator[](std::string_view key) const {
  for (auto const& m : members) {
    if (m.first == key) return m.second;
  }
  return NOTHING;
}

json const& json::operator[](size_t i) const { return kind == array && i < items.size() ? items[i] : NOTHING; }

bool json::get_int(int64_t lo, int64_t hi, int64_t& out) const {
  if (kind != number || num != std::floor(num) || num < (double)lo || num > (double)hi) return false;
  out = (int64_t)num;
  return true;
}

}  // namespace llama_cu
