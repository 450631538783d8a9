// Typed access to a parsed config.json; the first missing or unfit value is reported.
#pragma once
#include <cmath>
#include <cstdio>
#include <string>

#include "json.hpp"

namespace llama_cu {

struct config_reader {
  bool ok{true};
  void complain(std::string const& where, const char* key) {
    if (ok) fprintf(stderr, "Invalid config.json: %s\"%s\" is missing or out of range\n", where.c_str(), key);
    ok = false;
  }
  int integer(json const& v, const char* key, std::string const& where, int64_t lo = 1, int64_t hi = 1 << 28) {
    int64_t n = lo;
    if (!v[key].get_int(lo, hi, n)) complain(where, key);
    return (int)n;
  }
  double number(json const& v, const char* key, std::string const& where) {
    if (!v[key].is(json::number) || !std::isfinite(v[key].num)) complain(where, key);
    return v[key].num;
  }
  float real(json const& v, const char* key, std::string const& where) { return (float)number(v, key, where); }
};

}  // namespace llama_cu
