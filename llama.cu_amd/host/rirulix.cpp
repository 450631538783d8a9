#include "rirulix.hpp"

#include "config_reader.hpp"

namespace llama_cu {

namespace {

// constants of the design
constexpr float DECAY = -8.0f;         // log a = DECAY r softplus(lam)
constexpr float GATE_ALPHA = 1.702f;   // g sigmoid(GATE_ALPHA g) (u + GATE_SHIFT)
constexpr float GATE_SHIFT = 1.0f;

}  // namespace

bool rirulix_params(json const& config, layered_params& p) {
  config_reader r;
  p.family = "Rirulix";
  p.vocab = r.integer(config, "vocab", "");
  p.width = r.integer(config, "width", "");
  p.max_positions = r.integer(config, "max_positions", "");
  p.norm_groups = r.integer(config["norm"], "groups", "norm ");
  p.norm_eps = r.real(config["norm"], "eps", "norm ");
  if (r.ok && p.width % p.norm_groups != 0) r.complain("norm ", "groups");
  if (!config["layers"].is(json::array)) r.complain("", "layers");
  for (size_t l = 0; r.ok && l < config["layers"].size(); ++l) {
    json const& entry = config["layers"][l];
    json const& m = entry["mixer"];
    const std::string where = "layer " + std::to_string(l) + " ";
    layer_params L;
    if (entry["type"].text == "rglru") {
      L.mixer = mixer_type::rglru;
      L.recurrence.width = r.integer(m, "width", where);
      L.recurrence.blocks = r.integer(m, "blocks", where);
      L.recurrence.taps = r.integer(m, "conv", where, 1, 64);
      L.recurrence.decay = DECAY;
      if (r.ok && L.recurrence.width % L.recurrence.blocks != 0) r.complain(where, "blocks");
    } else if (entry["type"].text == "attention") {
      L.mixer = mixer_type::attention;
      L.attention.heads = r.integer(m, "heads", where);
      L.attention.kv_heads = r.integer(m, "kv_heads", where);
      L.attention.dim = r.integer(m, "dim", where);
      L.attention.vdim = r.integer(m, "vdim", where);
      L.attention.scale = r.real(m, "scale", where);
      L.attention.window = r.integer(m["mask"], "size", where + "mask ");
      L.attention.keep_first = r.integer(m["mask"], "keep_first", where + "mask ", 0);
      L.attention.v_mix = m["v_mix"].flag;
      if (r.ok && L.attention.heads % L.attention.kv_heads != 0) r.complain(where, "kv_heads");
    } else {
      r.complain(where, "type");
    }
    json const& f = entry["mlp"];
    if (f) {
      L.has_mlp = true;
      if (f["kind"].text != "moe") r.complain(where + "mlp ", "kind");
      L.mlp.experts = r.integer(f["router"], "experts", where + "router ");
      L.mlp.top = r.integer(f["router"], "top", where + "router ");
      if (r.ok && L.mlp.top > L.mlp.experts) r.complain(where + "router ", "top");
      L.mlp.ff = r.integer(f["expert"], "ff", where + "expert ");
      L.mlp.gate = lcu_gate_params{r.real(f["expert"], "limit", where + "expert "), GATE_ALPHA, GATE_SHIFT};
      if (f["shared"]) {
        L.mlp.shared_ff = r.integer(f["shared"], "ff", where + "shared ");
        L.mlp.shared_gate = lcu_gate_params{r.real(f["shared"], "limit", where + "shared "), GATE_ALPHA, GATE_SHIFT};
      }
    }
    p.layers.push_back(L);
  }
  if (r.ok && p.layers.empty()) r.complain("", "layers");
  return r.ok;
}

std::unique_ptr<llama_model> rirulix_load(json const& config, std::string const& dir, element_type type) {
  layered_params p;
  if (!rirulix_params(config, p)) return nullptr;
  return layered_model_impl::load(p, type, dir + "/model.safetensors");
}

std::unique_ptr<llama_model> rirulix_synthesize(json const& config, uint64_t seed, element_type type) {
  layered_params p;
  if (!rirulix_params(config, p)) return nullptr;
  return layered_model_impl::synthesize(p, type, seed);
}

}  // namespace llama_cu
