// One sequence of a layered decoder: its cache and state, and the step over its layers.
#pragma once
#include "layered.hpp"

namespace llama_cu {

struct layered_context_impl final : public llama_context {
  layered_context_impl(layered_model_impl* model, int context_len, float temperature);
  ~layered_context_impl() override;
  void clear_tokens() override;
  size_t context_memory_usage() override;
  short next_token(std::vector<short> const& new_tokens) override;
  int forward(const int32_t* tokens, int n, const int32_t* want, int n_want, float* logits) override;
  void sample_with_seed(uint64_t seed) override;
  void greedy() override;

  void* stream() const { return stream_; }
  // fp16 softmax(logits / temperature) of the last call's last token
  int read_probs(uint16_t* out);
  void record_residual(bool on) { recording_ = on; }
  int read_residual(int layer, float* out, int rows) const;

 private:
  // what a layer carries from token to token
  struct layer_state {
    gpu_buffer k, v;         // attention: [context][kv_heads * dk], [context][kv_heads * dv]; latent: [context][ldc], [context][dr]
    gpu_buffer conv, s;      // recurrences: the convolution's last inputs [taps - 1][ld], the fp32 state
  };
  gpu_buffer zeroed(size_t bytes);
  void enqueue_rows(int n);                        // n tokens, launch by launch
  void enqueue_one();                              // one token in bfloat16: fused launches, position from t_step_
  void step_one();                                 // enqueue_one, captured and replayed
  void drop_graph();
  void recurrence(recurrence_weights const& w, recurrence_params const& p, layer_state& s, int n);
  void attention(attention_weights const& w, attention_params const& p, layer_state& s, int n);
  void latent(latent_weights const& w, latent_params const& p, layer_state& s, int n, bool fused);
  void delta(delta_weights const& w, delta_params const& p, layer_state& s, int n);
  void decode_delta(delta_weights const& w, delta_params const& p, layer_state& s);
  void dense(dense_weights const& w, dense_params const& p, int n);
  void experts(experts_weights const& w, experts_params const& p, int n);
  void embed(int n, void* w_next);
  lcu_delta_params delta_shape(delta_weights const& w, delta_params const& p) const;
  void enqueue_head(int n_rows);
  void* next_norm(size_t layer) const;             // weights of the norm in front of layer `layer`, or NULL

  layered_model_impl* model_;
  int rows_;                                       // tokens of one pass; longer calls run in several
  std::vector<layer_state> state_;
  gpu_buffer t_x_, t_h_, t_m_, t_wide_, t_u_, t_rec_, t_scratch_, t_hidden_, t_shared_hidden_, t_expert_out_, t_shared_out_;
  gpu_buffer t_low_, t_queries_, t_latent_queries_, t_keys_values_, t_tail_;  // latent attention, delta rule
  gpu_buffer t_v_first_, t_choice_, t_weight_, t_shared_gate_, t_row_token_, t_row_weight_, t_inverse_, t_tile_expert_,
      t_tile_row_, t_expert_end_, t_n_tiles_;
  gpu_buffer t_step_, t_want_, t_head_in_, t_logits_, t_probs_, t_index_;
  // t_step_: position of the pass's first token, then its ids (int32); the launches read both from here
  void* start() const { return t_step_.data(); }
  void* ids() const { return (char*)t_step_.data() + 4; }
  std::vector<int32_t> host_step_, host_want_;
  size_t last_logits_row_{0};
  float* last_logits() const { return (float*)t_logits_.data() + last_logits_row_ * model_->shape.vocab; }
  int want_cap_{0};
  lcu_expert_plan plan_{};
  bool fused_step_{true};                          // one-token steps in bfloat16 take enqueue_one
  bool recording_{false};
  std::vector<std::vector<float>> residual_;
  bool sampling_{false};
  uint64_t sample_seed_{0}, samples_drawn_{0};
  void* decode_graph_{nullptr};
  int decode_calls_{0};
  gpu_buffer t_arrived_;                           // counters of the attention step, zero between launches
  void* stream_{nullptr};
};

}  // namespace llama_cu
