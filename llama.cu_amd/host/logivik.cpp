#include "logivik.hpp"

#include <limits>

#include "config_reader.hpp"

namespace llama_cu {

namespace {

// Nothing in the weights bounds a sequence; angles stay exact far beyond this many positions.
constexpr int MAX_POSITIONS = 1 << 20;

rotation_params read_rotation(config_reader& r, json const& rot, int rot_dim, std::string const& where) {
  rotation_params out;
  out.dims = r.integer(rot, "dims", where, 2, rot_dim);
  out.base = r.number(rot, "base", where);
  if (r.ok && (out.dims % 2 != 0)) r.complain(where, "dims");
  if (r.ok && out.base <= 1.0) r.complain(where, "base");
  json const& s = rot["scaling"];
  if (s) {
    out.scaled = true;
    out.factor = r.number(s, "factor", where + "scaling ");
    out.original = r.number(s, "original", where + "scaling ");
    out.fast = r.number(s, "fast", where + "scaling ");
    out.slow = r.number(s, "slow", where + "scaling ");
    for (double v : {out.factor, out.original, out.fast, out.slow}) {
      if (r.ok && v <= 0.0) r.complain(where, "scaling");
    }
  }
  return out;
}

void read_latent(config_reader& r, json const& m, latent_params& p, std::string const& where) {
  p.heads = r.integer(m, "heads", where, 1, 4096);
  p.dim = r.integer(m, "dim", where);
  p.vdim = r.integer(m, "vdim", where);
  p.kv_rank = r.integer(m, "kv_rank", where);
  p.scale = r.real(m, "scale", where);
}

}  // namespace

bool logivik_params(json const& config, layered_params& p) {
  config_reader r;
  p.family = "Logivik";
  p.vocab = r.integer(config, "vocab", "");
  p.width = r.integer(config, "width", "");
  p.max_positions = MAX_POSITIONS;
  p.learned_positions = false;
  p.embed_norm = false;
  p.embed_scale = r.real(config["embedding"], "scale", "embedding ");
  p.norm_ahead = false;
  p.norm_shift = 1.0f;  // weights are stored around zero
  p.norm_eps = r.real(config["norm"], "eps", "norm ");
  if (!config["layers"].is(json::array)) r.complain("", "layers");
  for (size_t l = 0; r.ok && l < config["layers"].size(); ++l) {
    json const& entry = config["layers"][l];
    json const& m = entry["mixer"];
    const std::string where = "layer " + std::to_string(l) + " ";
    layer_params L;
    if (entry["type"].text == "delta") {
      L.mixer = mixer_type::delta;
      L.delta.heads = r.integer(m, "heads", where);
      L.delta.kv_heads = r.integer(m, "kv_heads", where);
      L.delta.dim = r.integer(m, "dim", where);
      L.delta.vdim = r.integer(m, "vdim", where);
      L.delta.taps = r.integer(m, "conv", where, 1, 64);
      if (r.ok && L.delta.heads % L.delta.kv_heads != 0) r.complain(where, "kv_heads");
    } else if (entry["type"].text == "latent_attention") {
      L.mixer = mixer_type::latent;
      read_latent(r, m, L.latent, where);
      L.latent.sink = L.latent.gate = true;
      L.latent.rot_dim = r.integer(m, "rot_dim", where, 2);
      if (r.ok) L.latent.rot = read_rotation(r, m["rot"], L.latent.rot_dim, where + "rot ");
    } else if (entry["type"].text == "latent_attention_2") {
      L.mixer = mixer_type::latent;
      read_latent(r, m, L.latent, where);
      L.latent.q_rank = r.integer(m, "q_rank", where);
      L.latent.window = r.integer(m["mask"], "size", where + "mask ", 1, std::numeric_limits<int>::max());
    } else {
      r.complain(where, "type");
    }
    json const& f = entry["mlp"];
    if (f) {
      L.has_mlp = true;
      if (f["kind"].text != "dense") r.complain(where + "mlp ", "kind");
      L.dense.ff = r.integer(f, "ff", where + "mlp ");
      L.dense.gate = lcu_gate_params{std::numeric_limits<float>::infinity(), 1.0f, 0.0f};  // silu(g) u
    }
    p.layers.push_back(L);
  }
  if (r.ok && p.layers.empty()) r.complain("", "layers");
  return r.ok;
}

std::unique_ptr<llama_model> logivik_load(json const& config, std::string const& dir, element_type type) {
  layered_params p;
  if (!logivik_params(config, p)) return nullptr;
  return layered_model_impl::load(p, type, dir + "/model.safetensors");
}

std::unique_ptr<llama_model> logivik_synthesize(json const& config, uint64_t seed, element_type type) {
  layered_params p;
  if (!logivik_params(config, p)) return nullptr;
  return layered_model_impl::synthesize(p, type, seed);
}

}  // namespace llama_cu
