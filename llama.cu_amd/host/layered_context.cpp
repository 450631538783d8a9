// The step of a layered decoder.  A layer is x += norm1b(mixer(norm1(x))), x += norm2b(ff(norm2(x))), without norm1
// and norm2 where sublayers read x itself; the launch that adds a sublayer's result also leaves the next
// sublayer's input.
#include "layered_context.hpp"

#include <stdlib.h>
#include <string.h>

#include <algorithm>
#include <limits>

namespace llama_cu {

namespace {
constexpr int MAX_ROWS = 2048;  // tokens of one pass: bounds the activations, not the prompt
// Calls of at most this many tokens attend over the latents; longer ones multiply keys and values out, which
// costs the visible keys once but makes every row's sums several times shorter.
constexpr int FEW_ROWS = 32;

lcu_latent_params latent_shape(latent_weights const& w, latent_params const& p) {
  return lcu_latent_params{p.heads, w.dn, w.dr, p.rot.dims, w.dv, p.kv_rank, w.ldc, p.window > 0 ? p.window : std::numeric_limits<int>::max(),
                           p.scale};
}
}  // namespace

layered_context_impl::layered_context_impl(layered_model_impl* model, int context_len, float temperature)
    : llama_context(context_len, temperature), model_(model), rows_(std::min(context_len, MAX_ROWS)) {
  device_structure_lock lock(device_structure_mutex());
  LCU_CHECK(lcu_init(0));
  LCU_CHECK(lcu_stream_create(&stream_));
  layered_model_impl const& m = *model_;
  const size_t R = rows_, e = m.elem, ctx = context_len_;
  size_t low = 0, queries = 0, latent_queries = 0, keys_values = 0, tail = 0;
  size_t counters = 1, wide = 0, u = 0, rec = 0, scratch = 0, hidden = 0, shared = 0, expert_rows = 0, v_first = 0, experts = 0, tiles = 0;
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
    } else if (p.mixer == mixer_type::latent) {
      latent_weights const& a = w.latent;
      const lcu_latent_params lp = latent_shape(a, p.latent);
      wide = std::max(wide, (size_t)a.ldw);
      rec = std::max(rec, (size_t)a.ldo);
      if (p.latent.q_rank > 0) {
        low = std::max(low, (size_t)a.low_ld);
        queries = std::max(queries, (size_t)a.q_cols);
      }
      if (a.few) {
        latent_queries = std::max(latent_queries, (size_t)p.latent.heads * a.ldc);
        for (size_t n = 1; n <= std::min<size_t>(FEW_ROWS, R); ++n) {
          scratch = std::max(scratch, lcu_latent_attention_scratch(&lp, (int)n, (int)ctx));
        }
      }
      const size_t seen = p.latent.window > 0 ? std::min(ctx, (size_t)p.latent.window + R) : ctx;
      keys_values = std::max(keys_values, seen * p.latent.heads * (a.dn + a.dv));
      state_[l].k = zeroed(ctx * a.ldc * e);
      if (a.dr > 0) state_[l].v = zeroed(ctx * a.dr * e);
    } else if (p.mixer == mixer_type::delta) {
      delta_weights const& d = w.delta;
      const lcu_delta_params dp = delta_shape(d, p.delta);
      wide = std::max(wide, (size_t)d.channels + d.plain);
      u = std::max(u, (size_t)d.channels);
      tail = std::max(tail, (size_t)2 * p.delta.heads);
      rec = std::max(rec, (size_t)d.ldo);
      scratch = std::max(scratch, lcu_delta_rule_scratch(&dp, (int)R));
      if (p.delta.taps > 1) state_[l].conv = zeroed((size_t)(p.delta.taps - 1) * d.channels * e);
      state_[l].s = zeroed((size_t)p.delta.heads * d.dk * d.dv * 4);
    } else {
      wide = std::max(wide, (size_t)w.attention.ldq);
      rec = std::max(rec, (size_t)w.attention.ldo);
      counters = std::max(counters, (size_t)p.attention.kv_heads);
      if (w.attention.v_mode != 0) v_first = std::max(v_first, (size_t)w.attention.v_cols);
      state_[l].k = zeroed(ctx * w.attention.k_cols * e);
      state_[l].v = zeroed(ctx * w.attention.v_cols * e);
    }
    if (p.dense.ff > 0) shared = std::max(shared, R * (size_t)w.dense.ld);
    if (p.has_mlp && p.dense.ff == 0) {
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
  t_low_ = zeroed(R * low * e);
  t_queries_ = zeroed(R * queries * e);
  t_latent_queries_ = zeroed(std::min<size_t>(FEW_ROWS, R) * latent_queries * e);
  t_keys_values_ = zeroed(keys_values * e);
  t_tail_ = zeroed(R * tail * 4);
  t_hidden_ = zeroed(hidden * e);
  t_shared_hidden_ = zeroed(shared * e);
  t_expert_out_ = zeroed((expert_rows + 1) * ld * 4);  // a one-token step keeps the shared expert's row behind the others
  t_shared_out_ = zeroed(R * ld * 4);
  t_v_first_ = zeroed(R * v_first * e);
  for (gpu_buffer* b : {&t_choice_, &t_weight_, &t_row_token_, &t_row_weight_, &t_inverse_}) *b = zeroed(expert_rows * 4);
  t_shared_gate_ = zeroed(R * 4);
  t_tile_expert_ = zeroed(tiles * 4);
  t_tile_row_ = zeroed(tiles * 4);
  t_expert_end_ = zeroed(experts * 4);
  t_n_tiles_ = zeroed(4);
  // the one-token attention kernel holds the heads of a group in registers and LDS
  for (size_t l = 0; l < m.layers.size(); ++l) {
    attention_params const& a = m.shape.layers[l].attention;
    if (m.shape.layers[l].mixer != mixer_type::attention) continue;
    const int group = a.heads / a.kv_heads;
    if (group > 16 || group * (m.layers[l].attention.dv + 2) > 2400) fused_step_ = false;
  }
  for (size_t l = 0; l < m.layers.size(); ++l) {
    if (m.shape.layers[l].mixer == mixer_type::latent && !m.layers[l].latent.few) fused_step_ = false;
  }
  t_arrived_ = zeroed(counters * 4);
  t_step_ = zeroed((1 + R) * 4);
  t_probs_ = zeroed((size_t)m.shape.vocab * 2);
  t_index_ = zeroed(4);
  plan_ = lcu_expert_plan{t_row_token_.data(),   t_row_weight_.data(), t_inverse_.data(), t_tile_expert_.data(),
                          t_tile_row_.data(),    t_expert_end_.data(), t_n_tiles_.data(), 0, 0};
  LCU_CHECK(lcu_sync(stream_));
}

layered_context_impl::~layered_context_impl() {
  lcu_sync(stream_);
  device_structure_lock lock(device_structure_mutex());
  lcu_graph_destroy(decode_graph_);
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
       {&t_low_, &t_queries_, &t_latent_queries_, &t_keys_values_, &t_tail_, &t_x_, &t_h_, &t_m_, &t_wide_, &t_u_, &t_rec_, &t_scratch_, &t_hidden_, &t_shared_hidden_, &t_expert_out_, &t_shared_out_,
        &t_v_first_, &t_choice_, &t_weight_, &t_shared_gate_, &t_row_token_, &t_row_weight_, &t_inverse_, &t_tile_expert_,
        &t_tile_row_, &t_expert_end_, &t_n_tiles_, &t_arrived_, &t_step_, &t_want_, &t_head_in_, &t_logits_, &t_probs_, &t_index_}) {
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
  LCU_CHECK(lcu_conv_causal(t_u_.data(), y + (size_t)w.ld * e, 2 * w.ld, w.conv.data(), w.conv_bias.data(), s.conv.data(), p.taps, 0,
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
                         w.v_mix.data(), start(), context_len_, m.dtype, n, stream_));
  LCU_CHECK(lcu_attention_windowed(t_rec_.data(), w.ldo, t_wide_.data(), w.ldq, s.k.data(), s.v.data(), start_pos_, &window,
                                   m.dtype, n, stream_));
  LCU_CHECK(lcu_linear(t_m_.data(), 1, m.ld, t_rec_.data(), w.out.data(), w.out_bias.data(), 0, m.dtype, n, w.ldo, m.shape.width,
                       stream_));
}

// `fused`: one token in bfloat16, products as weight streams.
void layered_context_impl::latent(latent_weights const& w, latent_params const& p, layer_state& s, int n, bool fused) {
  layered_model_impl const& m = *model_;
  const lcu_latent_params lp = latent_shape(w, p);
  const auto product = [&](gpu_buffer& out, gpu_buffer const& x, gpu_buffer const& weight, int K, int N) {
    if (fused) {
      LCU_CHECK(lcu_decode_linear_bf16(out.data(), x.data(), weight.data(), K, N, stream_));
    } else {
      LCU_CHECK(lcu_linear(out.data(), 0, N, x.data(), weight.data(), nullptr, 0, m.dtype, n, K, N, stream_));
    }
  };
  lcu_latent_rows_args rows{};
  rows.rows_dev = t_wide_.data();
  rows.ld = w.ldw;
  rows.n = n;
  rows.latent_at = w.latent_at;
  rows.key_at = w.key_at;
  rows.query_at = w.dn;
  rows.rotate_queries = w.dr > 0 && p.q_rank == 0;
  rows.low_rank = p.q_rank;
  rows.low_ld = w.low_ld;
  rows.max_positions = context_len_;
  rows.latent_norm_dev = w.latent_norm.data();
  rows.low_norm_dev = w.low_norm.data();
  rows.low_dev = t_low_.data();
  rows.latents_dev = s.k.data();
  rows.keys_dev = s.v.data();
  rows.freq_dev = w.freq.data();
  rows.gain = w.gain;
  rows.eps = m.shape.norm_eps;
  rows.start_dev = start();
  const bool few = w.few && n <= FEW_ROWS, low = p.q_rank > 0;
  product(t_wide_, t_h_, w.in, m.ld, w.ldw);
  if (low || !few) LCU_CHECK(lcu_latent_rows(&rows, &lp, m.dtype, stream_));
  if (low) product(t_queries_, t_low_, w.uq, w.low_ld, w.q_cols);
  const char* q = (char*)(low ? t_queries_ : t_wide_).data();
  const int ldq = low ? w.q_cols : w.ldw;
  const void* gate = p.gate ? (char*)t_wide_.data() + (size_t)w.gate_at * m.elem : nullptr;
  char* values = (char*)w.ukv.data() + (size_t)p.heads * w.dn * w.ldc * m.elem;
  if (few) {
    LCU_CHECK(lcu_latent_queries(t_latent_queries_.data(), q, ldq, w.uk_t.data(), &lp, low ? nullptr : &rows, n, stream_));
    LCU_CHECK(lcu_latent_attention(t_rec_.data(), w.ldo, t_latent_queries_.data(), q + (size_t)w.dn * m.elem, ldq, s.k.data(), s.v.data(),
                                   start(), context_len_, values, p.sink ? w.sink.data() : nullptr, gate, w.ldw, &lp, t_scratch_.data(), n,
                                   stream_));
  } else {
    // keys and values of every position the call sees
    const int first = p.window > 0 ? std::max(0, start_pos_ - p.window + 1) : 0, seen = start_pos_ + n - first;
    const int keys = p.heads * w.dn, cols = keys + p.heads * w.dv;
    LCU_CHECK(lcu_linear(t_keys_values_.data(), 0, cols, (char*)s.k.data() + (size_t)first * w.ldc * m.elem, w.ukv.data(), nullptr, 0,
                         m.dtype, seen, w.ldc, cols, stream_));
    lcu_window_params window{};
    window.heads = window.kv_heads = p.heads;
    window.dk = w.dn + w.dr;
    window.dv = w.dv;
    window.window = lp.window;
    window.scale = p.scale;
    window.dk_shared = w.dr;
    window.k_ld = window.v_ld = cols;
    window.first_position = first;
    window.k_shared_dev = w.dr > 0 ? (char*)s.v.data() + (size_t)first * w.dr * m.elem : nullptr;
    window.sink_dev = p.sink ? w.sink.data() : nullptr;
    window.gate_dev = gate;
    window.ldg = w.ldw;
    LCU_CHECK(lcu_attention_windowed(t_rec_.data(), w.ldo, q, ldq, t_keys_values_.data(),
                                     (char*)t_keys_values_.data() + (size_t)keys * m.elem, start_pos_, &window, m.dtype, n, stream_));
  }
  if (fused) {
    LCU_CHECK(lcu_decode_linear(t_m_.data(), t_rec_.data(), w.out.data(), nullptr, w.ldo, m.shape.width, stream_));
  } else {
    LCU_CHECK(lcu_linear(t_m_.data(), 1, m.ld, t_rec_.data(), w.out.data(), nullptr, 0, m.dtype, n, w.ldo, m.shape.width, stream_));
  }
}

lcu_delta_params layered_context_impl::delta_shape(delta_weights const& w, delta_params const& p) const {
  return lcu_delta_params{p.heads, p.kv_heads, w.dk, w.dv, p.dim, p.vdim, model_->shape.norm_eps, w.a_log.data(), w.dt_bias.data(),
                          w.norm.data()};
}

void layered_context_impl::delta(delta_weights const& w, delta_params const& p, layer_state& s, int n) {
  layered_model_impl const& m = *model_;
  const lcu_delta_params d = delta_shape(w, p);
  const int ld = w.channels + w.plain, tail = 2 * p.heads;
  LCU_CHECK(lcu_linear_tail(t_wide_.data(), ld, t_tail_.data(), tail, ld, t_h_.data(), w.in.data(), m.dtype, n, m.ld, w.rows, stream_));
  LCU_CHECK(lcu_conv_causal(t_u_.data(), t_wide_.data(), ld, w.conv.data(), nullptr, s.conv.data(), p.taps, 1, m.dtype, n, w.channels,
                            w.channels, stream_));
  LCU_CHECK(lcu_delta_rule(t_rec_.data(), w.ldo, t_u_.data(), w.channels, (char*)t_wide_.data() + (size_t)w.channels * m.elem, ld,
                           t_tail_.data(), tail, &d, s.s.data(), t_scratch_.data(), m.dtype, n, stream_));
  LCU_CHECK(lcu_linear(t_m_.data(), 1, m.ld, t_rec_.data(), w.out.data(), nullptr, 0, m.dtype, n, w.ldo, m.shape.width, stream_));
}

void layered_context_impl::decode_delta(delta_weights const& w, delta_params const& p, layer_state& s) {
  layered_model_impl const& m = *model_;
  const lcu_delta_params d = delta_shape(w, p);
  LCU_CHECK(lcu_decode_delta_in(t_u_.data(), t_wide_.data(), t_tail_.data(), s.conv.data(), t_h_.data(), w.in.data(), w.conv.data(), p.taps,
                                m.ld, w.channels, w.plain, w.rows, stream_));
  LCU_CHECK(lcu_decode_delta_step(t_rec_.data(), t_u_.data(), t_wide_.data(), t_tail_.data(), &d, s.s.data(), stream_));
  LCU_CHECK(lcu_decode_linear(t_m_.data(), t_rec_.data(), w.out.data(), nullptr, w.ldo, m.shape.width, stream_));
}

void layered_context_impl::dense(dense_weights const& w, dense_params const& p, int n) {
  layered_model_impl const& m = *model_;
  LCU_CHECK(lcu_linear_gated(t_shared_hidden_.data(), w.ld, t_h_.data(), w.up.data(), &p.gate, m.dtype, n, m.ld, 2 * w.ld, stream_));
  LCU_CHECK(lcu_linear(t_m_.data(), 1, m.ld, t_shared_hidden_.data(), w.down.data(), nullptr, 0, m.dtype, n, w.ld, m.shape.width, stream_));
}

void layered_context_impl::embed(int n, void* w_next) {
  layered_model_impl const& m = *model_;
  layered_params const& p = m.shape;
  if (p.learned_positions && p.embed_norm) {
    LCU_CHECK(lcu_embed_pos_norm(t_x_.data(), t_h_.data(), ids(), n, m.embed.data(), p.vocab, m.pos.data(), p.max_positions, start(),
                                 m.embed_norm.data(), w_next, m.dtype, p.width, m.ld, p.norm_groups, p.norm_eps, stream_));
  } else {
    LCU_CHECK(lcu_embed_scaled(t_x_.data(), t_h_.data(), ids(), n, m.embed.data(), p.vocab, p.embed_scale, w_next, m.dtype, p.width, m.ld,
                               p.norm_groups, p.norm_eps, stream_));
  }
}

void layered_context_impl::experts(experts_weights const& w, experts_params const& p, int n) {
  layered_model_impl const& m = *model_;
  const int rows = n * p.top, W = m.shape.width;
  // tiles of about half an expert's rows: larger ones multiply faster, but every expert ends in a part of one
  plan_.tile_rows = m.dtype == LCU_F32 ? 32 : (rows >= 384 * p.experts ? 256 : rows >= 96 * p.experts ? 128 : 64);
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
  embed(n, next_norm(0));
  for (size_t l = 0; l < m.layers.size(); ++l) {
    layer_params const& q = p.layers[l];
    layer_weights const& w = m.layers[l];
    const bool last = l + 1 == m.layers.size();  // nobody reads t_h_ after it
    switch (q.mixer) {
      case mixer_type::rglru: recurrence(w.recurrence, q.recurrence, state_[l], n); break;
      case mixer_type::attention: attention(w.attention, q.attention, state_[l], n); break;
      case mixer_type::latent: latent(w.latent, q.latent, state_[l], n, false); break;
      case mixer_type::delta: delta(w.delta, q.delta, state_[l], n); break;
    }
    LCU_CHECK(lcu_residual_norm(t_x_.data(), last && !q.has_mlp ? nullptr : t_h_.data(), t_m_.data(), nullptr, 1, nullptr, nullptr,
                                w.norm1b.data(), q.has_mlp ? w.norm2.data() : next_norm(l + 1), m.dtype, n, p.width, m.ld, p.norm_groups,
                                p.norm_eps, stream_));
    if (q.dense.ff > 0) {
      dense(w.dense, q.dense, n);
      LCU_CHECK(lcu_residual_norm(t_x_.data(), last ? nullptr : t_h_.data(), t_m_.data(), nullptr, 1, nullptr, nullptr, w.norm2b.data(),
                                  next_norm(l + 1), m.dtype, n, p.width, m.ld, p.norm_groups, p.norm_eps, stream_));
    } else if (q.has_mlp) {
      experts(w.mlp, q.mlp, n);
      const bool shared = q.mlp.shared_ff > 0;
      LCU_CHECK(lcu_residual_norm(t_x_.data(), last ? nullptr : t_h_.data(), t_expert_out_.data(), t_inverse_.data(), q.mlp.top,
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

// One token: launches fused around the weight streams.  A recurrent layer's mixer takes three (projections
// with the convolution, gates with the state, output product), an attention layer's too (projections with the
// cache rows, attention, output product), a latent layer's five (projections; keys applied to the queries, with norm,
// rotations and cache rows; scores; values; output product; two more with a queries' latent), a feed-forward two
// (first products, second products); between sublayers one launch adds the result, takes both norms and, in front of a feed-forward, routes.  The last
// layer's norms end in the final one.
void layered_context_impl::enqueue_one() {
  layered_model_impl const& m = *model_;
  layered_params const& p = m.shape;
  const size_t n_layers = m.layers.size();
  const auto norm_ahead = [&](size_t l) { return l < n_layers ? m.layers[l].norm1.data() : m.final_norm.data(); };
  embed(1, norm_ahead(0));
  for (size_t l = 0; l < n_layers; ++l) {
    layer_params const& q = p.layers[l];
    layer_weights const& L = m.layers[l];
    layer_state& s = state_[l];
    if (q.mixer == mixer_type::rglru) {
      recurrence_weights const& w = L.recurrence;
      LCU_CHECK(lcu_decode_recurrent_in(t_wide_.data(), t_u_.data(), s.conv.data(), t_h_.data(), w.yx.data(), w.yx_bias.data(),
                                        w.conv.data(), w.conv_bias.data(), q.recurrence.taps, m.ld, w.ld, stream_));
      LCU_CHECK(lcu_decode_recurrent_step(t_rec_.data(), t_u_.data(), t_wide_.data(), w.gate_r.data(), w.gate_i.data(), w.bias_r.data(),
                                          w.bias_i.data(), w.decay.data(), s.s.data(), w.channels, w.block, stream_));
      LCU_CHECK(lcu_decode_linear(t_m_.data(), t_rec_.data(), w.out.data(), nullptr, w.ld, p.width, stream_));
    } else if (q.mixer == mixer_type::latent) {
      latent(L.latent, q.latent, s, 1, true);
    } else if (q.mixer == mixer_type::delta) {
      decode_delta(L.delta, q.delta, s);
    } else {
      attention_weights const& w = L.attention;
      attention_params const& a = q.attention;
      const lcu_window_params window{a.heads, a.kv_heads, w.dk, w.dv, a.window, a.keep_first, a.scale, w.r1.data(), w.r2.data()};
      LCU_CHECK(lcu_decode_kv(t_wide_.data(), s.k.data(), s.v.data(), t_h_.data(), w.qkv.data(), w.qkv_bias.data(), w.q_cols, w.k_cols,
                              w.v_cols, t_v_first_.data(), w.v_mode, w.v_mix.data(), start(), context_len_, m.ld, stream_));
      LCU_CHECK(lcu_attention_windowed_decode(t_rec_.data(), t_wide_.data(), s.k.data(), s.v.data(), start(), context_len_, &window,
                                              t_arrived_.data(), stream_));
      LCU_CHECK(lcu_decode_linear(t_m_.data(), t_rec_.data(), w.out.data(), w.out_bias.data(), w.ldo, p.width, stream_));
    }
    experts_weights const& w = L.mlp;
    const bool shared = q.has_mlp && q.mlp.shared_ff > 0;
    LCU_CHECK(lcu_decode_residual_router(t_x_.data(), t_h_.data(), t_m_.data(), 1, nullptr, nullptr, L.norm1b.data(),
                                         q.has_mlp ? L.norm2.data() : norm_ahead(l + 1), p.width, m.ld, p.norm_groups, p.norm_eps,
                                         w.router.data(), q.mlp.experts, q.mlp.top, t_choice_.data(), t_weight_.data(),
                                         shared ? t_shared_gate_.data() : nullptr, stream_));
    if (q.dense.ff > 0) {
      LCU_CHECK(lcu_decode_gated(t_shared_hidden_.data(), t_h_.data(), L.dense.up.data(), &q.dense.gate, L.dense.ld, m.ld, stream_));
      LCU_CHECK(lcu_decode_linear(t_m_.data(), t_shared_hidden_.data(), L.dense.down.data(), nullptr, L.dense.ld, p.width, stream_));
      LCU_CHECK(lcu_decode_residual_router(t_x_.data(), t_h_.data(), t_m_.data(), 1, nullptr, nullptr, L.norm2b.data(), norm_ahead(l + 1),
                                           p.width, m.ld, p.norm_groups, p.norm_eps, nullptr, 0, 0, nullptr, nullptr, nullptr, stream_));
    } else if (q.has_mlp) {
      LCU_CHECK(lcu_decode_experts_up(t_hidden_.data(), t_shared_hidden_.data(), t_h_.data(), t_choice_.data(), t_weight_.data(),
                                      w.up.data(), w.up_stride, &q.mlp.gate, w.shared_up.data(), &q.mlp.shared_gate, q.mlp.top, w.ld,
                                      w.shared_ld, m.ld, stream_));
      LCU_CHECK(lcu_decode_experts_down(t_expert_out_.data(), m.ld, t_hidden_.data(), t_choice_.data(), w.down.data(), w.down_stride,
                                        q.mlp.top, w.ld, t_shared_hidden_.data(), w.shared_down.data(), w.shared_ld, p.width, stream_));
      const float* shared_row = (float*)t_expert_out_.data() + (size_t)q.mlp.top * m.ld;
      LCU_CHECK(lcu_decode_residual_router(t_x_.data(), t_h_.data(), t_expert_out_.data(), q.mlp.top, shared ? shared_row : nullptr,
                                           shared ? t_shared_gate_.data() : nullptr, L.norm2b.data(), norm_ahead(l + 1), p.width, m.ld,
                                           p.norm_groups, p.norm_eps, nullptr, 0, 0, nullptr, nullptr, nullptr, stream_));
    }
  }
  LCU_CHECK(lcu_decode_linear(t_logits_.data(), t_h_.data(), m.head.data(), nullptr, m.ld, p.vocab, stream_));
  LCU_CHECK(lcu_argmax_f32(t_index_.data(), t_logits_.data(), p.vocab, stream_));
}

// The first step runs eagerly (and loads the kernels), the second is captured, every later one replays it.
void layered_context_impl::step_one() {
  device_structure_lock lock(device_structure_mutex());  // capture, instantiation, launch: see host_common.hpp
  static const bool no_graph = getenv("LLAMA_CU_NO_GRAPH") != nullptr && atoi(getenv("LLAMA_CU_NO_GRAPH")) != 0;
  if (!decode_graph_ && ++decode_calls_ >= 2 && !no_graph) {
    LCU_CHECK(lcu_graph_begin_capture(stream_));
    enqueue_one();
    LCU_CHECK(lcu_graph_end_capture(stream_, &decode_graph_));
  }
  if (decode_graph_) {
    LCU_CHECK(lcu_graph_launch(decode_graph_, stream_));
  } else {
    enqueue_one();
  }
}

void layered_context_impl::drop_graph() {
  if (decode_graph_) {
    device_structure_lock lock(device_structure_mutex());
    LCU_CHECK(lcu_graph_destroy(decode_graph_));
    decode_graph_ = nullptr;
  }
  decode_calls_ = 0;
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
  if (n_rows == 1 && m.dtype == LCU_BF16) {
    LCU_CHECK(lcu_decode_linear(t_logits_.data(), t_head_in_.data(), m.head.data(), nullptr, m.ld, p.vocab, stream_));
    return;
  }
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
  const bool fused = n == 1 && m.dtype == LCU_BF16 && fused_step_ && !recording_;
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
      drop_graph();  // it holds the address of the logits
      want_cap_ = (int)round_up(rows.size(), 64);
      t_want_ = zeroed((size_t)want_cap_ * 4);
      t_head_in_ = zeroed((size_t)want_cap_ * m.ld * m.elem);
      t_logits_ = zeroed((size_t)want_cap_ * vocab * 4);
    }
    if (at > 0) LCU_CHECK(lcu_sync(stream_));  // the host's copies of the previous pass are about to change
    host_step_.assign(1, start_pos_);
    host_step_.insert(host_step_.end(), tokens + at, tokens + at + count);
    LCU_CHECK(lcu_h2d(t_step_.data(), host_step_.data(), host_step_.size() * 4, stream_));
    if (!fused && !rows.empty()) {
      host_want_ = rows;
      LCU_CHECK(lcu_h2d(t_want_.data(), host_want_.data(), host_want_.size() * 4, stream_));
    }
    if (fused) {
      step_one();
    } else {
      enqueue_rows(count);
      if (!rows.empty()) enqueue_head((int)rows.size());
      if (ends) {
        LCU_CHECK(lcu_argmax_f32(t_index_.data(), (float*)t_logits_.data() + (rows.size() - 1) * (size_t)vocab, vocab, stream_));
      }
    }
    if (ends) {
      last_logits_row_ = fused ? 0 : rows.size() - 1;
      if (sampling_) {
        LCU_CHECK(lcu_softmax_f32(t_probs_.data(), last_logits(), vocab, temperature_, stream_));
        uint64_t z = sample_seed_ + ++samples_drawn_ * 0x9E3779B97F4A7C15ull;
        z = (z ^ (z >> 30)) * 0xBF58476D1CE4E5B9ull;
        z = (z ^ (z >> 27)) * 0x94D049BB133111EBull;
        LCU_CHECK(lcu_sample_row(t_index_.data(), t_probs_.data(), vocab, z ^ (z >> 31), nullptr, stream_));
      }
      LCU_CHECK(lcu_d2h(&token, t_index_.data(), 4, stream_));
    }
    for (size_t i = 0; i < slots.size(); ++i) {  // consecutive rows of logits
      const size_t row = fused ? 0 : i;
      LCU_CHECK(lcu_d2h(logits + (size_t)slots[i] * vocab, (char*)t_logits_.data() + row * vocab * 4, (size_t)vocab * 4, stream_));
    }
    start_pos_ += count;
  }
  return token;
}

int layered_context_impl::read_probs(uint16_t* out) {
  if (t_logits_.size() == 0) return -1;  // no call yet
  const int vocab = model_->shape.vocab;
  LCU_CHECK(lcu_softmax_f32(t_probs_.data(), last_logits(), vocab, temperature_, stream_));
  return lcu_d2h(out, t_probs_.data(), (size_t)vocab * 2, stream_);
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
