// llama_model::open: any model directory.  A config.json names its family; a `params` file is a LLaMA in the
// reference's format (main.cpp:24-57).
#include "registry.hpp"

#include "logivik.hpp"
#include "rirulix.hpp"

namespace llama_cu {

namespace {
const model_family FAMILIES[] = {
    {"Rirulix", rirulix_load, rirulix_synthesize},
    {"Logivik", logivik_load, logivik_synthesize},
};

bool parse_config(std::string_view text, json& config, model_family const*& family) {
  std::string error;
  if (!json::parse(text, config, error)) {
    fprintf(stderr, "Invalid config.json: %s\n", error.c_str());
    return false;
  }
  family = find_family(config["architecture"].text);
  if (family == nullptr) {
    fprintf(stderr, "Unknown architecture \"%s\"\n", config["architecture"].text.c_str());
    return false;
  }
  return true;
}
}  // namespace

model_family const* find_family(std::string const& architecture) {
  for (model_family const& f : FAMILIES) {
    if (architecture == f.architecture) return &f;
  }
  return nullptr;
}

/* static */ std::unique_ptr<llama_model> llama_model::open(std::string const& dir, int context_len, element_type type) {
  mapped_buffer config_buf(dir + "/config.json");
  if (config_buf.is_ok()) {
    json config;
    model_family const* family = nullptr;
    if (!parse_config(std::string_view(static_cast<const char*>(config_buf.data()), config_buf.size()), config, family)) {
      return nullptr;
    }
    return family->load(config, dir, type);
  }
  mapped_buffer params_buf(dir + "/params");
  llama_params p;
  if (!params_buf.is_ok() || !p.load(params_buf)) {
    fprintf(stderr, "Could not load params file\n");
    return nullptr;
  }
  if (type != element_type::native) {
    fprintf(stderr, "A LLaMA model runs in the type of its weights only\n");
    return nullptr;
  }
  llama_partition partition;
  partition.autopipe(p, (size_t)context_len);
  if (!partition.is_valid()) {
    fprintf(stderr, "Could not partition model\n");
    return nullptr;
  }
  return llama_model::load(p, partition, dir);
}

/* static */ std::unique_ptr<llama_model> llama_model::create_synthetic(std::string const& config_text, uint64_t seed,
                                                                        element_type type) {
  json config;
  model_family const* family = nullptr;
  if (!parse_config(config_text, config, family)) {
    return nullptr;
  }
  return family->synthesize(config, seed, type);
}

}  // namespace llama_cu
