#include "safetensors.hpp"

#include <string.h>

#include "json.hpp"

namespace llama_cu {

float stored_tensor::at(size_t i) const {
  if (type == f32) {
    float v;
    memcpy(&v, static_cast<const char*>(data) + i * 4, 4);
    return v;
  }
  uint16_t h;
  memcpy(&h, static_cast<const char*>(data) + i * 2, 2);
  if (type == bf16) {
    const uint32_t u = (uint32_t)h << 16;
    float v;
    memcpy(&v, &u, 4);
    return v;
  }
  _Float16 v;
  memcpy(&v, &h, 2);
  return (float)v;
}

bool safetensors_file::open(std::string const& path) {
  file_ = mapped_buffer(path);
  tensors_.clear();
  const auto bad = [&](std::string const& why) {
    fprintf(stderr, "%s: %s\n", path.c_str(), why.c_str());
    return false;
  };
  if (!file_.is_ok() || file_.size() < 8) return bad("cannot be read");
  uint64_t len;
  memcpy(&len, file_.data(), 8);
  if (len > file_.size() - 8) return bad("header longer than the file");
  const char* base = static_cast<const char*>(file_.data());
  json head;
  std::string error;
  if (!json::parse(std::string_view(base + 8, len), head, error) || !head.is(json::object)) return bad("header: " + error);
  const size_t bytes = file_.size() - 8 - len;
  for (auto const& [name, t] : head.members) {
    if (name == "__metadata__") continue;
    stored_tensor s;
    std::string const& dtype = t["dtype"].text;
    s.type = dtype == "BF16" ? stored_tensor::bf16 : dtype == "F16" ? stored_tensor::f16 : dtype == "F32" ? stored_tensor::f32
                                                                                                           : stored_tensor::other;
    s.count = 1;
    for (json const& d : t["shape"].items) {
      int64_t v;
      if (!d.get_int(0, INT32_MAX, v)) return bad(name + ": bad shape");
      s.shape.push_back((size_t)v);
      s.count *= (size_t)v;
    }
    int64_t lo, hi;
    if (!t["data_offsets"][(size_t)0].get_int(0, (int64_t)bytes, lo) || !t["data_offsets"][1].get_int(lo, (int64_t)bytes, hi)) {
      return bad(name + ": data outside the file");
    }
    if (s.type != stored_tensor::other && (size_t)(hi - lo) != s.count * (s.type == stored_tensor::f32 ? 4 : 2)) {
      return bad(name + ": size does not fit the shape");
    }
    s.data = base + 8 + len + lo;
    tensors_.emplace(name, std::move(s));
  }
  return true;
}

stored_tensor const* safetensors_file::find(std::string const& name, std::vector<size_t> const& shape) const {
  const auto it = tensors_.find(name);
  const auto describe = [](std::vector<size_t> const& v) {
    std::string d = "[";
    for (size_t i = 0; i < v.size(); ++i) d += (i ? ", " : "") + std::to_string(v[i]);
    return d + "]";
  };
  if (it == tensors_.end()) {
    fprintf(stderr, "failed to load tensor %s: not in the file\n", name.c_str());
    return nullptr;
  }
  if (it->second.shape != shape || it->second.type == stored_tensor::other) {
    fprintf(stderr, "failed to load tensor %s: %s%s, expected %s\n", name.c_str(), describe(it->second.shape).c_str(),
            it->second.type == stored_tensor::other ? " of an unsupported type" : "", describe(shape).c_str());
    return nullptr;
  }
  return &it->second;
}

}  // namespace llama_cu
