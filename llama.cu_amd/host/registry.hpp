// Model families by the name a model directory gives itself.
#pragma once
#include <memory>
#include <string>

#include "host_common.hpp"
#include "json.hpp"

namespace llama_cu {

// A family that is configured by config.json: "architecture" names it.
struct model_family {
  const char* architecture;
  // the model in `dir` (its config already parsed), or nullptr with a message
  std::unique_ptr<llama_model> (*load)(json const& config, std::string const& dir, element_type type);
  // the same with seeded pseudo-random weights
  std::unique_ptr<llama_model> (*synthesize)(json const& config, uint64_t seed, element_type type);
};

model_family const* find_family(std::string const& architecture);

}  // namespace llama_cu
