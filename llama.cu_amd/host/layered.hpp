// Layered decoders: models whose layers are a list of mixers (recurrences, attention) and feed-forwards
// chosen per layer.  A family (rirulix.cpp, logivik.cpp) fills layered_params from its configuration;
// everything here is driven by these.  The numbers of a layer are in its own entry, so any order and mixture
// runs.
#pragma once
#include <string>
#include <vector>

#include "host_common.hpp"
#include "json.hpp"

namespace llama_cu {

enum class mixer_type { rglru, attention, latent, delta };

struct recurrence_params {
  int width{0}, blocks{1}, taps{1};
  float decay{0.0f};  // log a = decay r softplus(lam)
};

struct attention_params {
  int heads{0}, kv_heads{0}, dim{0}, vdim{0};
  int window{0}, keep_first{0};
  float scale{1.0f};
  bool v_mix{false};
};

// Rotation of neighbouring pairs; scaled: frequencies of slow pairs divided by factor (YaRN)
struct rotation_params {
  int dims{0};
  double base{1.0};
  bool scaled{false};
  double factor{1.0}, original{1.0}, fast{1.0}, slow{1.0};
  // frequency of each pair, and the factor on cosine and sine
  std::vector<float> frequencies(float& gain) const;
};

// Keys and values out of a latent per token.  rot_dim: size of the rotated part of a head (0: none); q_rank: size of the
// queries' latent (0: queries are projected directly); window 0: every key before.
struct latent_params {
  int heads{0}, dim{0}, rot_dim{0}, vdim{0}, kv_rank{0}, q_rank{0}, window{0};
  float scale{1.0f};
  bool sink{false}, gate{false};
  rotation_params rot;
};

// gated delta rule behind causal convolutions
struct delta_params {
  int heads{0}, kv_heads{0}, dim{0}, vdim{0}, taps{1};
};

struct dense_params {
  int ff{0};  // 0: the layer's feed-forward is of another kind
  lcu_gate_params gate{};
};

struct experts_params {
  int experts{0}, top{0}, ff{0};
  lcu_gate_params gate{};
  int shared_ff{0};  // 0: no shared expert
  lcu_gate_params shared_gate{};
};

struct layer_params {
  mixer_type mixer{mixer_type::rglru};
  recurrence_params recurrence;
  attention_params attention;
  latent_params latent;
  delta_params delta;
  bool has_mlp{false};
  dense_params dense;
  experts_params mlp;
};

struct layered_params {
  std::string family;
  int vocab{0}, width{0}, max_positions{0};
  bool learned_positions{true}, embed_norm{true};  // x = norm(embed[token] embed_scale + pos[position])
  float embed_scale{1.0f};
  bool norm_ahead{true};  // sublayers read the norm of x, and not x itself
  int norm_groups{1};
  float norm_eps{0.0f};
  float norm_shift{0.0f};  // added to the stored weights of the norms on x and on sublayers' results
  std::vector<layer_params> layers;
};

// ---- weights on the device ----------------------------------------------------------------------------
// Matrices are [rows][ld] of the element type with zeros in the padding; vectors are fp32.
struct recurrence_weights {
  int block{0}, channels{0}, ld{0};     // padded block width, all blocks, row stride
  gpu_buffer yx, yx_bias;               // rows: y channels [ld], then x channels [ld]
  gpu_buffer conv, conv_bias;           // [taps][ld]
  gpu_buffer gate_r, gate_i, bias_r, bias_i, decay;
  gpu_buffer out;                       // [width][ld]
};

struct attention_weights {
  int dk{0}, dv{0}, q_cols{0}, k_cols{0}, v_cols{0}, ldq{0}, ldo{0};
  int v_mode{0};                        // lcu_kv_store
  gpu_buffer qkv, qkv_bias, out, out_bias, r1, r2, v_mix;
};

struct latent_weights {
  int dn{0}, dr{0}, dv{0}, ldc{0}, low_ld{0}, q_cols{0};  // padded parts of a head, latent, queries' latent, all queries
  int latent_at{0}, key_at{0}, gate_at{0}, ldw{0}, ldo{0};
  bool few{false};       // the kernels for few tokens take these sizes
  gpu_buffer in;         // rows: queries or their latent | latent | rotated key part | gate
  gpu_buffer low_norm, latent_norm, uq;
  gpu_buffer ukv;        // rows: keys of all heads, values of all heads; [ldc]
  gpu_buffer uk_t;       // [heads][ldc][dn]
  gpu_buffer sink, freq, out;
  float gain{1.0f};
};

struct delta_weights {
  int dk{0}, dv{0}, channels{0}, plain{0}, rows{0}, ldo{0};
  gpu_buffer in;         // rows: q | k | v (`channels`) | gate (`plain`) | b | a
  gpu_buffer conv, a_log, dt_bias, norm, out;
};

struct dense_weights {
  int ld{0};
  gpu_buffer up, down;   // up in 32-row gate / up blocks
};

struct experts_weights {
  int ld{0}, shared_ld{0};              // padded ff: row stride of the hidden activations
  gpu_buffer router;                    // experts rows, then the shared expert's gate row
  gpu_buffer up, down;                  // all experts; up in 32-row gate / up blocks
  size_t up_stride{0}, down_stride{0};  // bytes of one expert
  gpu_buffer shared_up, shared_down;
};

struct layer_weights {
  gpu_buffer norm1, norm2;    // ahead of a sublayer
  gpu_buffer norm1b, norm2b;  // on its result
  recurrence_weights recurrence;
  attention_weights attention;
  latent_weights latent;
  delta_weights delta;
  dense_weights dense;
  experts_weights mlp;
};

struct layered_model_impl : public llama_model {
  static std::unique_ptr<llama_model> load(layered_params const& p, element_type type, std::string const& weight_file);
  static std::unique_ptr<llama_model> synthesize(layered_params const& p, element_type type, uint64_t seed);
  layered_model_impl(layered_params const& p, element_type type);
  std::unique_ptr<llama_context> make_context(int context_len, float temperature) override;
  int max_context() const override;

  layered_params shape;
  int dtype;        // LCU_BF16 or LCU_F32
  size_t elem;      // bytes of an element
  int ld;           // row stride of the residual stream
  gpu_buffer embed, pos, embed_norm, final_norm, head;
  std::vector<layer_weights> layers;

 private:
  bool shapes_supported() const;
  void make_tables();
  void lay_out();  // the sizes of every layer's padded operands
};

}  // namespace llama_cu
