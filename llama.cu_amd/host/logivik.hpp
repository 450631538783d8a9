// The Logivik family: config.json of its models, in terms of layered_params.
#pragma once
#include "layered.hpp"

namespace llama_cu {

std::unique_ptr<llama_model> logivik_load(json const& config, std::string const& dir, element_type type);
std::unique_ptr<llama_model> logivik_synthesize(json const& config, uint64_t seed, element_type type);
// false with a message when a size or constant is missing or not supported
bool logivik_params(json const& config, layered_params& out);

}  // namespace llama_cu
