// A JSON reader for configuration files, weight-file headers and replayed steps.
#pragma once
#include <cstdint>
#include <string>
#include <string_view>
#include <utility>
#include <vector>

namespace llama_cu {

// One parsed value.  Lookups on a value of another kind, or of a missing member, give the null value.
struct json {
  enum kind_t { null, boolean, number, string, array, object };
  kind_t kind{null};
  bool flag{false};
  double num{0.0};
  std::string text;
  std::vector<json> items;                           // array
  std::vector<std::pair<std::string, json>> members;  // object, in file order

  // Parses the whole text; on failure returns false and says where in `error`.
  static bool parse(std::string_view text, json& out, std::string& error);

  json const& operator[](std::string_view key) const;
  json const& operator[](size_t i) const;
  bool is(kind_t k) const { return kind == k; }
  explicit operator bool() const { return kind != null; }
  size_t size() const { return kind == array ? items.size() : members.size(); }
  // a number that is an integer in [lo, hi]
  bool get_int(int64_t lo, int64_t hi, int64_t& out) const;
};

}  // namespace llama_cu
