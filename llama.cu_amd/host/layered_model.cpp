// Weights of a layered decoder: packing from a weight file into the padded device layouts, or seeded
// pseudo-random values of the same shapes.
#include <math.h>
#include <string.h>

#include <algorithm>

#include "layered.hpp"
#include "safetensors.hpp"

namespace llama_cu {

namespace {

uint16_t bf16_of(float f) {  // nearest even
  uint32_t u;
  memcpy(&u, &f, 4);
  return (uint16_t)((u + 0x7FFF + ((u >> 16) & 1)) >> 16);
}

// A packed matrix being filled on the host.  Rows and columns not written stay zero.
struct packed_matrix {
  std::vector<uint16_t> h;
  std::vector<float> f;
  int dtype;
  size_t ld;
  packed_matrix(int dtype, size_t rows, size_t ld) : dtype(dtype), ld(ld) {
    if (dtype == LCU_F32) {
      f.assign(rows * ld, 0.0f);
    } else {
      h.assign(rows * ld, 0);
    }
  }
  void set(size_t row, size_t col, float v) {
    if (dtype == LCU_F32) {
      f[row * ld + col] = v;
    } else {
      h[row * ld + col] = bf16_of(v);
    }
  }
  // rows of t [rows][cols] to the rows and columns the two maps give
  template <class R, class C>
  void put(stored_tensor const& t, size_t rows, size_t cols, R&& to_row, C&& to_col) {
    for (size_t r = 0; r < rows; ++r) {
      const size_t at = to_row(r);
      for (size_t c = 0; c < cols; ++c) set(at, to_col(c), t.at(r * cols + c));
    }
  }
  void put(stored_tensor const& t, size_t rows, size_t cols, size_t first_row = 0) {
    put(t, rows, cols, [=](size_t r) { return first_row + r; }, [](size_t c) { return c; });
  }
  gpu_buffer upload() const {
    const size_t bytes = dtype == LCU_F32 ? f.size() * 4 : h.size() * 2;
    gpu_buffer b(bytes);
    b.copy_from(dtype == LCU_F32 ? (const void*)f.data() : (const void*)h.data(), bytes);
    LCU_CHECK(lcu_sync(nullptr));
    return b;
  }
};

gpu_buffer upload_vector(std::vector<float> const& v) {
  gpu_buffer b(v.size() * 4);
  b.copy_from(v.data(), v.size() * 4);
  LCU_CHECK(lcu_sync(nullptr));
  return b;
}

// vector t into an fp32 vector of n entries at the places the map gives
template <class M>
void put_vector(std::vector<float>& v, stored_tensor const& t, M&& to) {
  for (size_t i = 0; i < t.count; ++i) v[to(i)] = t.at(i);
}

// gate row j of a hidden layer in 64-row blocks of 32 gate and 32 up rows; the up row lies 32 further
size_t gate_row(size_t j) { return j / 32 * 64 + j % 32; }

int padded_value_size(int vdim) { return vdim <= 32 ? 32 : vdim <= 64 ? 64 : vdim <= 128 ? 128 : 256; }

// [heads][ldc][dn] from the keys' rows of a latent layer's ukv
std::vector<char> transposed_keys(latent_weights const& w, int heads, const char* ukv, size_t elem) {
  std::vector<char> t((size_t)heads * w.ldc * w.dn * elem);
  for (size_t h = 0; h < (size_t)heads; ++h) {
    for (size_t d = 0; d < (size_t)w.dn; ++d) {
      for (size_t r = 0; r < (size_t)w.ldc; ++r) {
        memcpy(&t[((h * w.ldc + r) * w.dn + d) * elem], ukv + ((h * w.dn + d) * w.ldc + r) * elem, elem);
      }
    }
  }
  return t;
}

gpu_buffer upload_bytes(std::vector<char> const& v) {
  gpu_buffer b(v.size());
  b.copy_from(v.data(), v.size());
  LCU_CHECK(lcu_sync(nullptr));
  return b;
}

struct loader {
  layered_model_impl& m;
  safetensors_file const& file;
  bool ok{true};

  stored_tensor const* get(std::string const& name, std::vector<size_t> const& shape) {
    static const stored_tensor none;
    stored_tensor const* t = ok ? file.find(name, shape) : nullptr;
    if (!t) {
      ok = false;
      return &none;
    }
    return t;
  }
  gpu_buffer vector(std::string const& name, size_t n, float shift = 0.0f) {
    std::vector<float> v(round_up(n, 64), 0.0f);  // padded like the rows they scale
    put_vector(v, *get(name, {n}), [](size_t i) { return i; });
    for (size_t i = 0; i < n; ++i) v[i] += shift;
    return upload_vector(v);
  }
  gpu_buffer norm(std::string const& name) { return vector(name, m.shape.width, m.shape.norm_shift); }
  gpu_buffer matrix(std::string const& name, size_t rows, size_t cols, size_t ld) {
    packed_matrix p(m.dtype, rows, ld);
    stored_tensor const& t = *get(name, {rows, cols});
    if (ok) p.put(t, rows, cols);
    return p.upload();
  }

  void recurrence(recurrence_weights& w, recurrence_params const& p, std::string const& at) {
    const size_t C = p.width, W = m.shape.width, B = p.blocks, cb = C / B, ld = w.ld;
    const auto lane = [&](size_t c) { return c / cb * w.block + c % cb; };  // channel -> padded channel
    packed_matrix yx(m.dtype, 2 * ld, m.ld);
    std::vector<float> bias(2 * ld, 0.0f), conv_bias(ld, 0.0f), br(ld, 0.0f), bi(ld, 0.0f), decay(ld, 0.0f), conv(p.taps * ld, 0.0f);
    stored_tensor const *y = get(at + "y", {C, W}), *yb = get(at + "y.b", {C}), *x = get(at + "x", {C, W}), *xb = get(at + "x.b", {C});
    stored_tensor const *cw = get(at + "conv", {C, (size_t)p.taps}), *cbias = get(at + "conv.b", {C}), *lam = get(at + "lam", {C});
    stored_tensor const *ra = get(at + "ra", {B, cb, cb}), *rab = get(at + "ra.b", {B, cb});
    stored_tensor const *ri = get(at + "ri", {B, cb, cb}), *rib = get(at + "ri.b", {B, cb});
    stored_tensor const* o = get(at + "o", {W, C});
    if (!ok) return;
    yx.put(*y, C, W, lane, [](size_t c) { return c; });
    yx.put(*x, C, W, [&](size_t c) { return ld + lane(c); }, [](size_t c) { return c; });
    put_vector(bias, *yb, lane);
    put_vector(bias, *xb, [&](size_t c) { return ld + lane(c); });
    put_vector(conv_bias, *cbias, lane);
    put_vector(br, *rab, lane);
    put_vector(bi, *rib, lane);
    for (size_t c = 0; c < C; ++c) {
      const double l = lam->at(c);
      decay[lane(c)] = (float)((double)p.decay * (l > 0 ? l + log1p(exp(-l)) : log1p(exp(l))));
      for (int k = 0; k < p.taps; ++k) conv[k * ld + lane(c)] = cw->at(c * p.taps + k);
    }
    packed_matrix gr(m.dtype, B * w.block, w.block), gi(m.dtype, B * w.block, w.block), out(m.dtype, W, ld);
    gr.put(*ra, C, cb, lane, [](size_t c) { return c; });
    gi.put(*ri, C, cb, lane, [](size_t c) { return c; });
    out.put(*o, W, C, [](size_t r) { return r; }, lane);
    w.yx = yx.upload();
    w.yx_bias = upload_vector(bias);
    w.conv = upload_vector(conv);
    w.conv_bias = upload_vector(conv_bias);
    w.gate_r = gr.upload();
    w.gate_i = gi.upload();
    w.bias_r = upload_vector(br);
    w.bias_i = upload_vector(bi);
    w.decay = upload_vector(decay);
    w.out = out.upload();
  }

  void attention(attention_weights& w, attention_params const& p, std::string const& at) {
    const size_t W = m.shape.width, H = p.heads, G = p.kv_heads, D = p.dim, E = p.vdim;
    packed_matrix qkv(m.dtype, w.ldq, m.ld), out(m.dtype, W, w.ldo);
    std::vector<float> bias(w.ldq, 0.0f);
    const auto part = [&](const char* name, size_t heads, size_t dim, size_t padded, size_t first) {
      stored_tensor const *t = get(at + name, {heads * dim, W}), *b = get(at + name + ".b", {heads * dim});
      if (!ok) return;
      const auto row = [=](size_t r) { return first + r / dim * padded + r % dim; };
      qkv.put(*t, heads * dim, W, row, [](size_t c) { return c; });
      put_vector(bias, *b, row);
    };
    part("q", H, D, w.dk, 0);
    part("k", G, D, w.dk, w.q_cols);
    part("v", G, E, w.dv, w.q_cols + w.k_cols);
    stored_tensor const* o = get(at + "o", {W, H * E});
    if (!ok) return;
    out.put(*o, W, H * E, [](size_t r) { return r; }, [&](size_t c) { return c / E * w.dv + c % E; });
    w.qkv = qkv.upload();
    w.qkv_bias = upload_vector(bias);
    w.out = out.upload();
    w.out_bias = vector(at + "o.b", W);
    w.r1 = vector(at + "r1", H);
    w.r2 = vector(at + "r2", H);
    if (w.v_mode == 2) {
      w.v_mix = upload_vector({get(at + "vmix", {})->count ? get(at + "vmix", {})->at(0) : 0.0f});
    }
  }

  void latent(latent_weights& w, latent_params const& p, std::string const& at) {
    const size_t W = m.shape.width, H = p.heads, D = p.dim, X = p.rot_dim, E = p.vdim, R = p.kv_rank, Q = p.q_rank;
    const auto same = [](size_t c) { return c; };
    packed_matrix in(m.dtype, w.ldw, m.ld), ukv(m.dtype, H * (w.dn + w.dv), w.ldc), out(m.dtype, W, w.ldo);
    // a query head is [unrotated | rotated], each part padded
    const auto query_row = [&](size_t r) {
      const size_t d = r % (D + X);
      return r / (D + X) * (w.dn + w.dr) + (d < D ? d : w.dn + d - D);
    };
    if (Q > 0) {
      stored_tensor const *dq = get(at + "dq", {Q, W}), *uq = get(at + "uq", {H * (D + X), Q});
      packed_matrix up(m.dtype, w.q_cols, w.low_ld);
      if (ok) in.put(*dq, Q, W);
      if (ok) up.put(*uq, H * (D + X), Q, query_row, same);
      w.uq = up.upload();
      w.low_norm = vector(at + "dq.norm", Q);
    } else {
      stored_tensor const* q = get(at + "q", {H * (D + X), W});
      if (ok) in.put(*q, H * (D + X), W, query_row, same);
    }
    stored_tensor const *dkv = get(at + "dkv", {R + X, W}), *uk = get(at + "uk", {H * D, R}), *uv = get(at + "uv", {H * E, R});
    stored_tensor const* o = get(at + "o", {W, H * E});
    if (!ok) return;
    in.put(*dkv, R + X, W, [&](size_t r) { return r < R ? w.latent_at + r : w.key_at + r - R; }, same);
    ukv.put(*uk, H * D, R, [&](size_t r) { return r / D * w.dn + r % D; }, same);
    const auto value = [&](size_t c) { return c / E * w.dv + c % E; };
    ukv.put(*uv, H * E, R, [&](size_t r) { return H * w.dn + value(r); }, same);
    out.put(*o, W, H * E, same, value);
    if (p.gate) {
      stored_tensor const* g = get(at + "g", {H * E, W});
      if (ok) in.put(*g, H * E, W, [&](size_t r) { return w.gate_at + value(r); }, same);
    }
    w.in = in.upload();
    w.ukv = ukv.upload();
    if (w.few) w.uk_t = upload_bytes(transposed_keys(w, p.heads, (const char*)ukv.h.data(), m.elem));
    w.out = out.upload();
    w.latent_norm = vector(at + "dkv.norm", R);
    if (p.sink) w.sink = vector(at + "sink", H);
  }

  void delta(delta_weights& w, delta_params const& p, std::string const& at) {
    const size_t W = m.shape.width, H = p.heads, G = p.kv_heads, D = p.dim, E = p.vdim, T = p.taps;
    const auto same = [](size_t c) { return c; };
    packed_matrix in(m.dtype, w.rows, m.ld), out(m.dtype, W, w.ldo);
    std::vector<float> conv(T * w.channels, 0.0f);
    const auto part = [&](const char* name, size_t heads, size_t dim, size_t padded, size_t first) {
      stored_tensor const *t = get(at + name, {heads * dim, W}), *c = get(at + name + ".conv", {heads * dim, T});
      if (!ok) return;
      const auto row = [&](size_t r) { return first + r / dim * padded + r % dim; };
      in.put(*t, heads * dim, W, row, same);
      for (size_t r = 0; r < heads * dim; ++r) {
        for (size_t k = 0; k < T; ++k) conv[k * w.channels + row(r)] = c->at(r * T + k);
      }
    };
    part("q", G, D, w.dk, 0);
    part("k", G, D, w.dk, G * w.dk);
    part("v", H, E, w.dv, 2 * G * w.dk);
    stored_tensor const *g = get(at + "g", {H * E, W}), *b = get(at + "b", {H, W}), *a = get(at + "a", {H, W}), *o = get(at + "o", {W, H * E});
    if (!ok) return;
    const auto value = [&](size_t c) { return c / E * w.dv + c % E; };
    in.put(*g, H * E, W, [&](size_t r) { return w.channels + value(r); }, same);
    in.put(*b, H, W, w.channels + w.plain);
    in.put(*a, H, W, w.channels + w.plain + H);
    out.put(*o, W, H * E, same, value);
    w.in = in.upload();
    w.conv = upload_vector(conv);
    w.out = out.upload();
    w.a_log = vector(at + "A_log", H);
    w.dt_bias = vector(at + "dt_bias", H);
    w.norm = vector(at + "norm", E);
  }

  void dense(dense_weights& w, dense_params const& p, std::string const& at) {
    packed_matrix up(m.dtype, 2 * w.ld, m.ld), down(m.dtype, m.shape.width, w.ld);
    expert(up, 0, down, 0, at, p.ff);
    w.up = up.upload();
    w.down = down.upload();
  }

  // one expert's matrices into rows of a packed pair
  void expert(packed_matrix& up, size_t up_row, packed_matrix& down, size_t down_row, std::string const& at, size_t ff) {
    const size_t W = m.shape.width;
    stored_tensor const *g = get(at + "gate", {ff, W}), *u = get(at + "up", {ff, W}), *d = get(at + "down", {W, ff});
    if (!ok) return;
    up.put(*g, ff, W, [=](size_t r) { return up_row + gate_row(r); }, [](size_t c) { return c; });
    up.put(*u, ff, W, [=](size_t r) { return up_row + gate_row(r) + 32; }, [](size_t c) { return c; });
    down.put(*d, W, ff, down_row);
  }

  void experts(experts_weights& w, experts_params const& p, std::string const& at) {
    const size_t W = m.shape.width, E = p.experts;
    packed_matrix router(m.dtype, E + 1, m.ld), up(m.dtype, E * 2 * w.ld, m.ld), down(m.dtype, E * W, w.ld);
    stored_tensor const* r = get(at + "router", {E, W});
    if (ok) router.put(*r, E, W);
    for (size_t e = 0; ok && e < E; ++e) {
      expert(up, e * 2 * w.ld, down, e * W, at + "e" + std::to_string(e) + ".", p.ff);
    }
    w.up = up.upload();
    w.down = down.upload();
    if (p.shared_ff > 0) {
      packed_matrix sup(m.dtype, 2 * w.shared_ld, m.ld), sdown(m.dtype, W, w.shared_ld);
      expert(sup, 0, sdown, 0, at + "shared.", p.shared_ff);
      stored_tensor const* sg = get(at + "shared.sg", {1, W});
      if (ok) router.put(*sg, 1, W, E);
      w.shared_up = sup.upload();
      w.shared_down = sdown.upload();
    }
    w.router = router.upload();
  }

  bool run() {
    layered_params const& s = m.shape;
    m.embed = matrix("embed", s.vocab, s.width, m.ld);
    if (s.learned_positions) m.pos = matrix("pos", s.max_positions, s.width, m.ld);
    if (s.embed_norm) m.embed_norm = norm("embed.norm");
    m.final_norm = norm("final.norm");
    m.head = matrix("head", s.vocab, s.width, m.ld);
    for (size_t l = 0; ok && l < s.layers.size(); ++l) {
      layer_params const& p = s.layers[l];
      layer_weights& w = m.layers[l];
      const std::string at = "l" + std::to_string(l) + ".";
      // the norm on a sublayer's result has the plain name where there is none ahead of it
      const std::string after = s.norm_ahead ? "b" : "";
      if (s.norm_ahead) w.norm1 = norm(at + "norm1");
      w.norm1b = norm(at + "norm1" + after);
      switch (p.mixer) {
        case mixer_type::rglru: recurrence(w.recurrence, p.recurrence, at + "mix."); break;
        case mixer_type::attention: attention(w.attention, p.attention, at + "mix."); break;
        case mixer_type::latent: latent(w.latent, p.latent, at + "mix."); break;
        case mixer_type::delta: delta(w.delta, p.delta, at + "mix."); break;
      }
      if (p.has_mlp) {
        if (s.norm_ahead) w.norm2 = norm(at + "norm2");
        w.norm2b = norm(at + "norm2" + after);
        if (p.dense.ff > 0) {
          dense(w.dense, p.dense, at + "mlp.");
        } else {
          experts(w.mlp, p.mlp, at + "mlp.");
        }
      }
    }
    return ok;
  }
};

}  // namespace

static llama_params outline(layered_params const& s) {
  // the fields of the reference's record that have a meaning for every decoder
  llama_params p{};
  p.magic = LLAMA_CU_MAGIC;
  p.dim = (uint32_t)s.width;
  p.multiple_of = 1;
  p.n_layers = (uint32_t)s.layers.size();
  p.n_vocab = (uint32_t)s.vocab;
  p.norm_eps = s.norm_eps;
  for (layer_params const& l : s.layers) {
    for (int heads : {l.attention.heads, l.latent.heads, l.delta.heads}) {
      if ((uint32_t)heads > p.n_heads) p.n_heads = (uint32_t)heads;
    }
  }
  return p;
}

layered_model_impl::layered_model_impl(layered_params const& p, element_type type)
    : llama_model(outline(p), llama_partition()), shape(p), dtype(type == element_type::f32 ? LCU_F32 : LCU_BF16),
      elem(type == element_type::f32 ? 4 : 2), ld((int)round_up(p.width, 64)), layers(p.layers.size()) {
  partition.use_default(params);
  lay_out();
}

void layered_model_impl::lay_out() {
  bool first_mix = true;
  for (size_t l = 0; l < layers.size(); ++l) {
    layer_params const& p = shape.layers[l];
    if (p.mixer == mixer_type::rglru) {
      recurrence_weights& w = layers[l].recurrence;
      w.block = (int)round_up(p.recurrence.width / p.recurrence.blocks, 32);
      w.channels = w.block * p.recurrence.blocks;
      w.ld = (int)round_up(w.channels, 64);
    } else if (p.mixer == mixer_type::latent) {
      latent_weights& w = layers[l].latent;
      latent_params const& a = p.latent;
      w.dn = (int)round_up(a.dim, 32);
      w.dr = (int)round_up(a.rot_dim, 32);
      w.dv = padded_value_size(a.vdim);
      w.ldc = (int)round_up(a.kv_rank, 64);
      w.low_ld = (int)round_up(a.q_rank, 64);
      w.q_cols = a.heads * (w.dn + w.dr);
      w.latent_at = a.q_rank > 0 ? w.low_ld : w.q_cols;
      w.key_at = w.latent_at + w.ldc;
      w.gate_at = w.key_at + w.dr;
      w.ldw = (int)round_up(w.gate_at + (a.gate ? a.heads * w.dv : 0), 64);
      w.ldo = (int)round_up(a.heads * w.dv, 64);
      const lcu_latent_params lp{a.heads, w.dn, w.dr, a.rot.dims, w.dv, a.kv_rank, w.ldc, 1, a.scale};
      w.few = dtype == LCU_BF16 && lcu_latent_attention_fits(&lp) != 0;
    } else if (p.mixer == mixer_type::delta) {
      delta_weights& w = layers[l].delta;
      w.dk = padded_value_size(p.delta.dim);
      w.dv = (int)round_up(p.delta.vdim, 32);
      w.channels = (int)round_up(2 * p.delta.kv_heads * w.dk + p.delta.heads * w.dv, 64);
      w.plain = p.delta.heads * w.dv;
      w.rows = w.channels + w.plain + 2 * p.delta.heads;
      w.ldo = (int)round_up(w.plain, 64);
    } else {
      attention_weights& w = layers[l].attention;
      w.dk = (int)round_up(p.attention.dim, 32);
      w.dv = padded_value_size(p.attention.vdim);
      w.q_cols = p.attention.heads * w.dk;
      w.k_cols = p.attention.kv_heads * w.dk;
      w.v_cols = p.attention.kv_heads * w.dv;
      w.ldq = (int)round_up(w.q_cols + w.k_cols + w.v_cols, 64);
      w.ldo = (int)round_up(p.attention.heads * w.dv, 64);
      if (p.attention.v_mix) {
        w.v_mode = first_mix ? 1 : 2;
        first_mix = false;
      }
    }
    if (p.dense.ff > 0) layers[l].dense.ld = (int)round_up(p.dense.ff, 64);
    if (p.has_mlp && p.dense.ff == 0) {
      experts_weights& w = layers[l].mlp;
      w.ld = (int)round_up(p.mlp.ff, 64);
      w.shared_ld = (int)round_up(p.mlp.shared_ff, 64);
      w.up_stride = (size_t)2 * w.ld * ld * elem;
      w.down_stride = (size_t)shape.width * w.ld * elem;
    }
  }
}

bool layered_model_impl::shapes_supported() const {
  const auto bad = [](std::string const& why) {
    fprintf(stderr, "unsupported model shape: %s\n", why.c_str());
    return false;
  };
  if (shape.width > 12288) return bad("width " + std::to_string(shape.width) + " (at most 12288)");
  if (shape.norm_groups > 2048) return bad("norm groups " + std::to_string(shape.norm_groups) + " (at most 2048)");
  attention_params const* first_v = nullptr;
  for (size_t l = 0; l < shape.layers.size(); ++l) {
    layer_params const& p = shape.layers[l];
    const std::string at = "layer " + std::to_string(l) + " ";
    if (p.mixer == mixer_type::attention) {
      attention_params const& a = p.attention;
      if (a.dim > 256 || a.vdim > 256) return bad(at + "head size " + std::to_string(a.dim) + " / " + std::to_string(a.vdim) + " (at most 256)");
      if (a.v_mix) {
        if (first_v != nullptr && (first_v->kv_heads != a.kv_heads || first_v->vdim != a.vdim)) {
          return bad(at + "mixes values of another size");
        }
        first_v = &a;
      }
    }
    if (p.mixer == mixer_type::latent && (layers[l].latent.dn + layers[l].latent.dr > 256 || p.latent.vdim > 256)) {
      return bad(at + "head size " + std::to_string(p.latent.dim) + " + " + std::to_string(p.latent.rot_dim) + " / " +
                 std::to_string(p.latent.vdim) + " (at most 256, parts in multiples of 32)");
    }
    if (p.mixer == mixer_type::delta && (p.delta.dim > 256 || p.delta.vdim > 256)) {
      return bad(at + "head size " + std::to_string(p.delta.dim) + " / " + std::to_string(p.delta.vdim) + " (at most 256)");
    }
    if (p.has_mlp && p.mlp.experts > 512) return bad(at + std::to_string(p.mlp.experts) + " experts (at most 512)");
  }
  return true;
}

int layered_model_impl::max_context() const {
  // the fp32 attention kernel keeps the scores of every visible key
  if (dtype == LCU_F32) {
    for (layer_params const& p : shape.layers) {
      if (p.mixer == mixer_type::latent && (p.latent.window == 0 || p.latent.window > 32768)) return std::min(shape.max_positions, 32768);
    }
  }
  return shape.max_positions;
}

std::vector<float> rotation_params::frequencies(float& gain) const {
  const double pi = 3.14159265358979323846;
  std::vector<float> f(dims / 2);
  // the pair that turns t times within `original` positions
  const auto pair_of = [&](double t) { return dims * log(original / (2.0 * pi * t)) / (2.0 * log(base)); };
  const double lo = std::max(floor(pair_of(fast)), 0.0), hi = std::min(ceil(pair_of(slow)), dims - 1.0);
  for (int i = 0; i < dims / 2; ++i) {
    const double plain = pow(base, -2.0 * i / dims);
    const double ramp = scaled ? std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0) : 0.0;
    f[i] = (float)(plain / factor * ramp + plain * (1.0 - ramp));
  }
  gain = scaled ? (float)(0.1 * log(factor) + 1.0) : 1.0f;
  return f;
}

// the rotation's table, which no weight file holds
void layered_model_impl::make_tables() {
  for (size_t l = 0; l < layers.size(); ++l) {
    if (shape.layers[l].latent.rot.dims == 0) continue;
    latent_weights& w = layers[l].latent;
    w.freq = upload_vector(shape.layers[l].latent.rot.frequencies(w.gain));
  }
}

/* static */ std::unique_ptr<llama_model> layered_model_impl::load(layered_params const& p, element_type type,
                                                                   std::string const& weight_file) {
  auto m = std::make_unique<layered_model_impl>(p, type);
  if (!m->shapes_supported()) return nullptr;
  safetensors_file file;
  if (!file.open(weight_file)) return nullptr;
  LCU_CHECK(lcu_init(0));
  loader l{*m, file};
  if (!l.run()) return nullptr;
  m->make_tables();
  return m;
}

/* static */ std::unique_ptr<llama_model> layered_model_impl::synthesize(layered_params const& p, element_type type, uint64_t seed) {
  auto m = std::make_unique<layered_model_impl>(p, type);
  if (!m->shapes_supported()) return nullptr;
  LCU_CHECK(lcu_init(0));
  uint64_t stream = 0;
  const int dtype = m->dtype;
  const auto matrix = [&](size_t rows, size_t cols, size_t ld, float std) {
    gpu_buffer b(rows * ld * m->elem);
    LCU_CHECK(lcu_memset(b.data(), 0, b.size(), nullptr));
    LCU_CHECK(lcu_fill_normal_matrix(b.data(), rows, (int)cols, (int)ld, dtype, seed, ++stream, 0.0f, std, nullptr));
    return b;
  };
  const auto linear = [&](size_t rows, size_t cols, size_t ld) { return matrix(rows, cols, ld, 1.0f / sqrtf((float)cols)); };
  const auto vector = [&](size_t n, float mean, float std) {
    gpu_buffer b(round_up(n, 64) * 4);
    LCU_CHECK(lcu_memset(b.data(), 0, b.size(), nullptr));
    LCU_CHECK(lcu_fill_normal_matrix(b.data(), 1, (int)n, (int)n, LCU_F32, seed, ++stream, mean, std, nullptr));
    return b;
  };
  // `count` blocks of `rows` rows, `apart` rows from one to the next, from row `first` of b on: padding rows stay zero
  const auto blocks = [&](gpu_buffer& b, size_t first, size_t count, size_t rows, size_t apart, size_t cols, size_t row_ld) {
    for (size_t k = 0; k < count; ++k) {
      LCU_CHECK(lcu_fill_normal_matrix((char*)b.data() + (first + k * apart) * row_ld * m->elem, rows, (int)cols, (int)row_ld, dtype, seed,
                                       ++stream, 0.0f, 1.0f / sqrtf((float)cols), nullptr));
    }
  };
  const auto zeros = [&](size_t rows, size_t row_ld) {
    gpu_buffer b(rows * row_ld * m->elem);
    LCU_CHECK(lcu_memset(b.data(), 0, b.size(), nullptr));
    return b;
  };
  const size_t W = p.width, V = p.vocab, ld = m->ld;
  m->embed = matrix(V, W, ld, 1.0f / p.embed_scale);
  if (p.learned_positions) m->pos = matrix(p.max_positions, W, ld, 0.5f);
  m->embed_norm = vector(W, 1.0f, 0.1f);
  m->final_norm = vector(W, 1.0f, 0.1f);
  m->head = linear(V, W, ld);
  for (size_t l = 0; l < p.layers.size(); ++l) {
    layer_params const& q = p.layers[l];
    layer_weights& L = m->layers[l];
    for (gpu_buffer* n : {&L.norm1, &L.norm1b, &L.norm2, &L.norm2b}) *n = vector(W, 1.0f, 0.1f);
    if (q.mixer == mixer_type::rglru) {
      recurrence_weights& w = L.recurrence;
      const size_t C = w.ld, B = (size_t)q.recurrence.blocks * w.block;
      w.yx = linear(2 * C, W, ld);
      w.yx_bias = vector(2 * C, 0.0f, 0.1f);
      w.conv = vector(q.recurrence.taps * C, 0.0f, 0.5f);
      w.conv_bias = vector(C, 0.0f, 0.1f);
      w.gate_r = linear(B, w.block, w.block);
      w.gate_i = linear(B, w.block, w.block);
      w.bias_r = vector(C, 0.0f, 0.1f);
      w.bias_i = vector(C, 0.0f, 0.1f);
      w.decay = vector(C, q.recurrence.decay * 0.1f, 0.05f);
      w.out = linear(W, C, C);
    } else if (q.mixer == mixer_type::latent) {
      latent_weights& w = L.latent;
      latent_params const& a = q.latent;
      const size_t H = a.heads, D = a.dim, X = a.rot_dim, E = a.vdim;
      const auto queries = [&](gpu_buffer& b, size_t cols, size_t row_ld) {
        blocks(b, 0, H, D, w.dn + w.dr, cols, row_ld);
        if (X > 0) blocks(b, w.dn, H, X, w.dn + w.dr, cols, row_ld);
      };
      w.in = zeros(w.ldw, ld);
      if (a.q_rank > 0) {
        blocks(w.in, 0, 1, a.q_rank, 0, W, ld);
        w.uq = zeros(w.q_cols, w.low_ld);
        queries(w.uq, a.q_rank, w.low_ld);
        w.low_norm = vector(a.q_rank, 1.0f, 0.1f);
      } else {
        queries(w.in, W, ld);
      }
      blocks(w.in, w.latent_at, 1, a.kv_rank, 0, W, ld);
      if (X > 0) blocks(w.in, w.key_at, 1, X, 0, W, ld);
      if (a.gate) blocks(w.in, w.gate_at, H, E, w.dv, W, ld);
      w.ukv = zeros(H * (w.dn + w.dv), w.ldc);
      blocks(w.ukv, 0, H, D, w.dn, a.kv_rank, w.ldc);
      blocks(w.ukv, H * w.dn, H, E, w.dv, a.kv_rank, w.ldc);
      if (w.few) {
        std::vector<char> keys(H * w.dn * w.ldc * m->elem);
        LCU_CHECK(lcu_d2h(keys.data(), w.ukv.data(), keys.size(), nullptr));
        LCU_CHECK(lcu_sync(nullptr));
        w.uk_t = upload_bytes(transposed_keys(w, a.heads, keys.data(), m->elem));
      }
      w.latent_norm = vector(a.kv_rank, 1.0f, 0.1f);
      if (a.sink) w.sink = vector(H, 0.5f, 1.0f);
      w.out = linear(W, w.ldo, w.ldo);
    } else if (q.mixer == mixer_type::delta) {
      delta_weights& w = L.delta;
      delta_params const& d = q.delta;
      const size_t H = d.heads, G = d.kv_heads;
      w.in = zeros(w.rows, ld);
      blocks(w.in, 0, 2 * G, d.dim, w.dk, W, ld);
      blocks(w.in, 2 * G * w.dk, H, d.vdim, w.dv, W, ld);
      blocks(w.in, w.channels, H, d.vdim, w.dv, W, ld);
      blocks(w.in, w.channels + w.plain, 1, 2 * H, 0, W, ld);
      w.conv = vector((size_t)d.taps * w.channels, 0.0f, 0.5f);
      w.a_log = vector(H, -1.0f, 1.0f);
      w.dt_bias = vector(H, -1.0f, 0.5f);
      w.norm = vector(d.vdim, 1.0f, 0.1f);
      w.out = linear(W, w.ldo, w.ldo);
    } else {
      attention_weights& w = L.attention;
      w.qkv = linear(w.ldq, W, ld);
      w.qkv_bias = vector(w.ldq, 0.0f, 0.1f);
      w.out = linear(W, w.ldo, w.ldo);
      w.out_bias = vector(W, 0.0f, 0.1f);
      w.r1 = vector(q.attention.heads, 0.5f, 0.05f);
      w.r2 = vector(q.attention.heads, 0.3f, 0.02f);
      w.v_mix = vector(1, 0.3f, 0.0f);
    }
    if (q.dense.ff > 0) {
      dense_weights& w = L.dense;
      w.up = linear(2 * w.ld, W, ld);
      w.down = linear(W, w.ld, w.ld);
    } else if (q.has_mlp) {
      experts_weights& w = L.mlp;
      const size_t E = q.mlp.experts;
      w.router = linear(E + 1, W, ld);
      w.up = linear(E * 2 * w.ld, W, ld);
      w.down = linear(E * W, w.ld, w.ld);
      if (q.mlp.shared_ff > 0) {
        w.shared_up = linear(2 * w.shared_ld, W, ld);
        w.shared_down = linear(W, w.shared_ld, w.shared_ld);
      }
    }
  }
  LCU_CHECK(lcu_sync(nullptr));
  m->make_tables();
  return m;
}

}  // namespace llama_cu
