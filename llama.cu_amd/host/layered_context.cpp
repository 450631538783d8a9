// The step of a layered decoder.  A layer is x += norm1b(mixer(norm1(x))), x += norm2b(ff(norm2(x))); the
// launch that adds a sublayer's result also normalises the next sublayer's input.
#include "layered_context.hpp"

#include <assert.h>
#include <string.h>

#include <algorithm>

namespace llama_cu {

namespace {
constexpr int MAX_ROWS = 2048;  // tokens of one pass: bounds the activations, not the prompt
}

layered_context_impl::layered_context_impl(layered_model_impl* model, int context_len, float temperature)
    : llama_context(context_len, temperature), model_(model), rows_(std::min(context_len, MAX_ROWS)) {
  device_structure_lock lock(device_structure_mutex());
  LCU_CHECK(lcu_init(0));
  LCU_CHECK(lcu_stream_create(&stream_));
  layered_model_impl const& m = *model_;
  const size_t R = rows_, e = m.elem, ctx = context_len_;
  size_t wide = 0, u = 0, rec = 0, scratch = 0, hidden = 0, shared = 0, expert_rows = 0, v_first = 0, experts = 0, tiles = 0;
  state_.resize(m.layers.size());
  for (size_t l = 0; l < m.layers.size(); ++l) {
    layer_params const& p = m.shape.layers[l];
    layer_weights const& w = m.layers[l];
    if (p.mixer == mixer_type::rglru) {
      const size_t ld = w.recurrence.ld;
      wide = std::max(wide, 2 * ld);
      u = std::max(u, ld);
      rec = std::max(rec, ld);
      scratch = std::max(scratch, lcu_gated_recurrence_scratch((int)R, (int)ld));
      if (p.recurrence.taps > 1) state_[l].conv = zeroed((p.recurrence.taps - 1) * ld * e);
      state_[l].s = zeroed(ld * 4);
    } else {
      wide = std::max(wide, (size_t)w.attention.ldq);
      rec = std::max(rec, (size_t)w.attention.ldo);
      if (w.attention.v_mode != 0) v_first = std::max(v_first, (size_t)w.attention.v_cols);
      state_[l].k = zeroed(ctx * w.attention.k_cols * e);
      state_[l].v = zeroed(ctx * w.attention.v_cols * e);
    }
    if (p.has_mlp) {
      const size_t top = p.mlp.top, E = p.mlp.experts;
      expert_rows = std::max(expert_rows, R * top);
      hidden = std::max(hidden, R * top * (size_t)w.mlp.ld);
      shared = std::max(shared, R * (size_t)w.mlp.shared_ld);
      experts = std::max(experts, E);
      tiles = std::max(tiles, R * top / 32 + std::min(E, R * top));
    }
  }
  const size_t ld = m.ld;
  t_x_ = zeroed(R * ld * 4);
  t_h_ = zeroed(R * ld * e);
  t_m_ = zeroed(R * ld * 4);
  t_wide_ = zeroed(R * wide * e);
  t_u_ = zeroed(R * u * e);
  t_rec_ = zeroed(R * rec * e);
  t_scratch_ = zeroed(scratch);
  t_hidden_ = zeroed(hidden * e);
  t_shared_hidden_ = zeroed(shared * e);
  t_expert_out_ = zeroed(expert_rows * ld * 4);
  t_shared_out_ = zeroed(R * ld * 4);
  t_v_first_ = zeroed(R * v_first * e);
  for (gpu_buffer* b : {&t_choice_, &t_weight_, &t_row_token_, &t_row_weight_, &t_inverse_}) *b = zeroed(expert_rows * 4);
  t_shared_gate_ = zeroed(R * 4);
  t_tile_expert_ = zeroed(tiles * 4);
  t_tile_row_ = zeroed(tiles * 4);
  t_expert_end_ = zeroed(experts * 4);
  t_n_tiles_ = zeroed(4);
  t_ids_ = zeroed(R * 4);
  t_start_ = zeroed(4);
  t_probs_ = zeroed((size_t)m.shape.vocab * 2);
  t_index_ = zeroed(4);
  plan_ = lcu_expert_plan{t_row_token_.data(),   t_row_weight_.data(), t_inverse_.data(), t_tile_expert_.data(),
                          t_tile_row_.data(),    t_expert_end_.data(), t_n_tiles_.data(), 0, 0};
  LCU_CHECK(lcu_sync(stream_));
}

layered_context_impl::~layered_context_impl() {
  lcu_sync(stream_);
  device_structure_lock lock(device_structure_mutex());
  lcu_stream_destroy(stream_);
}

// Activations and caches start as zeros: the padding of their rows meets zero weights and must be finite.
gpu_buffer layered_context_impl::zeroed(size_t bytes) {
  gpu_buffer b(std::max<size_t>(bytes, 4));
  LCU_CHECK(lcu_memset(b.data(), 0, b.size(), stream_));
  return b;
}

void layered_context_impl::clear_tokens() {
  // Rows of the caches at or beyond the position are never read before they are written; the state is.
  for (layer_state& s : state_) {
    for (gpu_buffer* b : {&s.conv, &s.s}) {
      if (b->is_ok()) LCU_CHECK(lcu_memset(b->data(), 0, b->size(), stream_));
    }
  }
  LCU_CHECK(lcu_sync(stream_));
  start_pos_ = 0;
}

size_t layered_context_impl::context_memory_usage() {
  size_t count = 0;
  for (layer_state const& s : state_) count += s.k.size() + s.v.size() + s.conv.size() + s.s.size();
  for (gpu_buffer const* b :
       {&t_x_, &t_h_, &t_m_, &t_wide_, &t_u_, &t_rec_, &t_scratch_, &t_hidden_, &t_shared_hidden_, &t_expert_out_, &t_shared_out_,
        &t_v_first_, &t_choice_, &t_weight_, &t_shared_gate_, &t_row_token_, &t_row_weight_, &t_inverse_, &t_tile_expert_,
        &t_tile_row_, &t_expert_end_, &t_n_tiles_, &t_ids_, &t_start_, &t_want_, &t_head_in_, &t_logits_, &t_probs_, &t_index_}) {
    count += b->size();
  }
  return count;
}

void* layered_context_impl::next_norm(size_t layer) const {
  return layer < model_->layers.size() ? model_->layers[layer].norm1.data() : nullptr;
}

void layered_context_impl::recurrence(recurrence_weights const& w, recurrence_params const& p, layer_state& s, int n) {
  layered_model_impl const& m = *model_;
  const size_t e = m.elem;
  char* y = (char*)t_wide_.data();
  LCU_CHECK(lcu_linear(y, 0, 2 * w.ld, t_h_.data(), w.yx.data(), w.yx_bias.data(), w.ld, m.dtype, n, m.ld, 2 * w.ld, stream_));
  LCU_CHECK(lcu_conv_causal(t_u_.data(), y + (size_t)w.ld * e, 2 * w.ld, w.conv.data(), w.conv_bias.data(), s.conv.data(), p.taps,
                            m.dtype, n, w.channels, w.ld, stream_));
  LCU_CHECK(lcu_gated_recurrence(t_rec_.data(), t_u_.data(), y, 2 * w.ld, w.gate_r.data(), w.gate_i.data(), w.bias_r.data(),
                                 w.bias_i.data(), w.decay.data(), s.s.data(), t_scratch_.data(), m.dtype, n, w.channels, w.block,
                                 w.ld, stream_));
  LCU_CHECK(lcu_linear(t_m_.data(), 1, m.ld, t_rec_.data(), w.out.data(), nullptr, 0, m.dtype, n, w.ld, m.shape.width, stream_));
}

void layered_context_impl::attention(attention_weights const& w, attention_params const& p, layer_state& s, int n) {
  layered_model_impl const& m = *model_;
  const lcu_window_params window{p.heads, p.kv_heads, w.dk, w.dv, p.window, p.keep_first, p.scale, w.r1.data(), w.r2.data()};
  LCU_CHECK(lcu_linear(t_wide_.data(), 0, w.ldq, t_h_.data(), w.qkv.data(), w.qkv_bias.data(), 0, m.dtype, n, m.ld, w.ldq, stream_));
  LCU_CHECK(lcu_kv_store(s.k.data(), s.v.data(), t_wide_.data(), w.ldq, w.q_cols, w.k_cols, w.v_cols, t_v_first_.data(), w.v_mode,
                         w.v_mix.data(), t_start_.data(), context_len_, m.dtype, n, stream_));
  LCU_CHECK(lcu_attention_windowed(t_rec_.data(), w.ldo, t_wide_.data(), w.ldq, s.k.data(), s.v.data(), start_pos_, &window,
                                   m.dtype, n, stream_));
  LCU_CHECK(lcu_linear(t_m_.data(), 1, m.ld, t_rec_.data(), w.out.data(), w.out_bias.data(), 0, m.dtype, n, w.ldo, m.shape.width,
                       stream_));
}

void layered_context_impl::experts(experts_weights const& w, experts_params const& p, int n) {
  layered_model_impl const& m = *model_;
  const int rows = n * p.top, W = m.shape.width;
  plan_.tile_rows = m.dtype == LCU_F32 ? 32 : (rows >= 96 * p.experts ? 128 : 64);
  plan_.max_tiles = rows / plan_.tile_rows + std::min(p.experts, rows);
  LCU_CHECK(lcu_router(t_choice_.data(), t_weight_.data(), p.shared_ff > 0 ? t_shared_gate_.data() : nullptr, t_h_.data(),
                       w.router.data(), p.experts, p.top, m.dtype, n, m.ld, stream_));
  LCU_CHECK(lcu_experts_plan(&plan_, t_choice_.data(), t_weight_.data(), n, p.top, p.experts, stream_));
  LCU_CHECK(lcu_experts_up(t_hidden_.data(), w.ld, t_h_.data(), w.up.data(), w.up_stride, &p.gate, &plan_, m.dtype, n, m.ld,
                           2 * w.ld, stream_));
  LCU_CHECK(lcu_experts_down(t_expert_out_.data(), m.ld, t_hidden_.data(), w.down.data(), w.down_stride, &plan_, m.dtype, rows, w.ld,
                             W, stream_));
  if (p.shared_ff > 0) {
    LCU_CHECK(lcu_linear_gated(t_shared_hidden_.data(), w.shared_ld, t_h_.data(), w.shared_up.data(), &p.shared_gate, m.dtype, n,
                               m.ld, 2 * w.shared_ld, stream_));
    LCU_CHECK(lcu_linear(t_shared_out_.data(), 1, m.ld, t_shared_hidden_.data(), w.shared_down.data(), nullptr, 0, m.dtype, n,
                         w.shared_ld, W, stream_));
  }
}

void layered_context_impl::enqueue_rows(int n) {
  layered_model_impl const& m = *model_;
  layered_params const& p = m.shape;
  LCU_CHECK(lcu_embed_pos_norm(t_x_.data(), t_h_.data(), t_ids_.data(), n, m.embed.data(), p.vocab, m.pos.data(), p.max_positions,
                               t_start_.data(), m.embed_norm.data(), next_norm(0), m.dtype, p.width, m.ld, p.norm_groups, p.norm_eps,
                               stream_));
  for (size_t l = 0; l < m.layers.size(); ++l) {
    layer_params const& q = p.layers[l];
    layer_weights const& w = m.layers[l];
    if (q.mixer == mixer_type::rglru) {
      recurrence(w.recurrence, q.recurrence, state_[l], n);
    } else {
      attention(w.attention, q.attention, state_[l], n);
    }
    LCU_CHECK(lcu_residual_norm(t_x_.data(), t_h_.data(), t_m_.data(), nullptr, 0, nullptr, nullptr, w.norm1b.data(),
                                q.has_mlp ? w.norm2.data() : next_norm(l + 1), m.dtype, n, p.width, m.ld, p.norm_groups, p.norm_eps,
                                stream_));
    if (q.has_mlp) {
      experts(w.mlp, q.mlp, n);
      const bool shared = q.mlp.shared_ff > 0;
      LCU_CHECK(lcu_residual_norm(t_x_.data(), t_h_.data(), t_expert_out_.data(), t_inverse_.data(), q.mlp.top,
                                  shared ? t_shared_out_.data() : nullptr, shared ? t_shared_gate_.data() : nullptr, w.norm2b.data(),
                                  next_norm(l + 1), m.dtype, n, p.width, m.ld, p.norm_groups, p.norm_eps, stream_));
    }
    if (recording_) {
      std::vector<float> rows((size_t)n * m.ld);
      LCU_CHECK(lcu_d2h(rows.data(), t_x_.data(), rows.size() * 4, stream_));
      for (int r = 0; r < n; ++r) {
        residual_[l].insert(residual_[l].end(), rows.begin() + (size_t)r * m.ld, rows.begin() + (size_t)r * m.ld + p.width);
      }
    }
  }
}

int layered_context_impl::read_residual(int layer, float* out, int rows) const {
  if (layer < 0 || (size_t)layer >= residual_.size()) return -1;
  const size_t count = (size_t)rows * model_->shape.width;
  if (rows <= 0 || count > residual_[layer].size()) return -1;
  memcpy(out, residual_[layer].data(), count * 4);
  return 0;
}

// final norm and logits of the rows named in t_want_
void layered_context_impl::enqueue_head(int n_rows) {
  layered_model_impl const& m = *model_;
  layered_params const& p = m.shape;
  LCU_CHECK(lcu_group_norm(t_head_in_.data(), t_x_.data(), t_want_.data(), m.final_norm.data(), m.dtype, n_rows, p.width, m.ld,
                           p.norm_groups, p.norm_eps, stream_));
  LCU_CHECK(lcu_linear(t_logits_.data(), 1, p.vocab, t_head_in_.data(), m.head.data(), nullptr, 0, m.dtype, n_rows, m.ld, p.vocab,
                       stream_));
}

int layered_context_impl::forward(const int32_t* tokens, int n, const int32_t* want, int n_want, float* logits) {
  layered_model_impl const& m = *model_;
  const int vocab = m.shape.vocab;
  if (!call_fits(tokens, n, want, n_want, vocab)) {
    return -1;
  }
  if (recording_) residual_.assign(m.layers.size(), {});
  int token = -1;
  for (int at = 0; at < n; at += rows_) {
    const int count = std::min(rows_, n - at);
    const bool ends = at + count == n;
    // rows of this pass that go through the head: the wanted ones, then the last of the call
    std::vector<int32_t> rows, slots;
    for (int i = 0; i < n_want; ++i) {
      if (want[i] >= at && want[i] < at + count) {
        rows.push_back(want[i] - at);
        slots.push_back(i);
      }
    }
    if (ends) rows.push_back(count - 1);
    if ((int)rows.size() > want_cap_) {
      want_cap_ = (int)round_up(rows.size(), 64);
      t_want_ = zeroed((size_t)want_cap_ * 4);
      t_head_in_ = zeroed((size_t)want_cap_ * m.ld * m.elem);
      t_logits_ = zeroed((size_t)want_cap_ * vocab * 4);
    }
    LCU_CHECK(lcu_h2d(t_ids_.data(), tokens + at, (size_t)count * 4, stream_));
    LCU_CHECK(lcu_h2d(t_start_.data(), &start_pos_, 4, stream_));
    LCU_CHECK(lcu_h2d(t_want_.data(), rows.data(), rows.size() * 4, stream_));
    LCU_CHECK(lcu_sync(stream_));  // the host copies above may go away or change
    enqueue_rows(count);
    if (!rows.empty()) enqueue_head((int)rows.size());
    if (ends) {
      const size_t last = (rows.size() - 1) * (size_t)vocab * 4;
      LCU_CHECK(lcu_softmax_argmax_f32(t_probs_.data(), t_index_.data(), (char*)t_logits_.data() + last, vocab, temperature_, stream_));
      if (sampling_) {
        uint64_t z = sample_seed_ + ++samples_drawn_ * 0x9E3779B97F4A7C15ull;
        z = (z ^ (z >> 30)) * 0xBF58476D1CE4E5B9ull;
        z = (z ^ (z >> 27)) * 0x94D049BB133111EBull;
        LCU_CHECK(lcu_sample_row(t_index_.data(), t_probs_.data(), vocab, z ^ (z >> 31), nullptr, stream_));
      }
      LCU_CHECK(lcu_d2h(&token, t_index_.data(), 4, stream_));
    }
    for (size_t i = 0; i < slots.size(); ++i) {  // consecutive rows of logits
      LCU_CHECK(lcu_d2h(logits + (size_t)slots[i] * vocab, (char*)t_logits_.data() + i * (size_t)vocab * 4, (size_t)vocab * 4, stream_));
    }
    start_pos_ += count;
  }
  return token;
}

short layered_context_impl::next_token(std::vector<short> const& new_tokens) {
  const std::vector<int32_t> ids(new_tokens.begin(), new_tokens.end());
  return (short)forward(ids.data(), (int)ids.size(), nullptr, 0, nullptr);
}

void layered_context_impl::sample_with_seed(uint64_t seed) {
  sampling_ = true;
  sample_seed_ = seed;
  samples_drawn_ = 0;
}

void layered_context_impl::greedy() { sampling_ = false; }

std::unique_ptr<llama_context> layered_model_impl::make_context(int context_len, float temperature) {
  return std::make_unique<layered_context_impl>(this, context_len, temperature);
}

}  // namespace llama_cu
