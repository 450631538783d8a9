// Weights in a safetensors file: an 8-byte little-endian header length, a JSON header (name -> dtype,
// shape, data_offsets) and the data, mapped read-only.
#pragma once
#include <string>
#include <unordered_map>
#include <vector>

#include "host_common.hpp"

namespace llama_cu {

struct stored_tensor {
  enum type_t { bf16, f16, f32, other };
  type_t type{other};
  std::vector<size_t> shape;
  const void* data{nullptr};
  size_t count{0};
  float at(size_t i) const;  // element i as fp32 (bf16, f16, f32)
};

struct safetensors_file {
  bool open(std::string const& path);  // false (and a message) when the file is missing or malformed
  // the tensor of that name and shape; nullptr (and a message) when it is missing, shaped otherwise or of
  // a type at() does not read
  stored_tensor const* find(std::string const& name, std::vector<size_t> const& shape) const;
  bool has(std::string const& name) const { return tensors_.count(name) != 0; }

 private:
  mapped_buffer file_;
  std::unordered_map<std::string, stored_tensor> tensors_;
};

}  // namespace llama_cu
