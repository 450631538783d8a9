"""Every mechanism of the layered decoders on its own, against the plain restatement (plain_stack.py).

Both element types: fp32 has to agree to fp32 rounding, bfloat16 to the rounding of its inputs and outputs
(the oracle gets the same rounded inputs).  Sizes are chosen to be ragged: nothing here is a multiple of
what a kernel's tile happens to be.
"""
import ctypes as C

import numpy as np
import pytest

import plain_stack as S
from layered_helpers import BF16, BOTH, F32, call, close, get, get_ints, gpu, ints, pack_gated, pad, put, rounded, up64, zeros  # noqa: F401

pytestmark = pytest.mark.gpu


# ---- linear ---------------------------------------------------------------------------------------------
@BOTH
@pytest.mark.parametrize("M,K,N", [(1, 64, 5), (3, 192, 70), (37, 320, 100), (64, 128, 129), (130, 256, 200), (300, 448, 2048),
                                   (513, 128, 4100), (2, 1024, 300), (31, 2048, 1100), (48, 1536, 65), (64, 512, 3000)])
def test_linear_with_bias_and_gelu_columns(gpu, dt, M, K, N):
    rng = np.random.default_rng(M * 7 + N)
    x, w, b = rounded(rng.standard_normal((M, K))), rounded(rng.standard_normal((N, K)) / K ** 0.5), rng.standard_normal(N)
    cut, ldo = N // 3, up64(N)
    out = zeros(gpu, (M, ldo), dt)
    call(gpu, "lcu_linear", out, 0, ldo, put(gpu, x, dt), put(gpu, w, dt), put(gpu, b), cut, dt, M, K, N)
    want = x @ w.T + b
    want[:, :cut] = S.gelu_tanh(want[:, :cut])
    got = get(gpu, out, (M, ldo), dt)
    close(got[:, :N], want, dt)
    assert (got[:, N:] == 0).all()                                    # the padding of the rows is left alone
    out = zeros(gpu, (M, N))
    call(gpu, "lcu_linear", out, 1, N, put(gpu, x, dt), put(gpu, w, dt), None, 0, dt, M, K, N)
    close(get(gpu, out, (M, N)), x @ w.T, F32)                        # fp32 output of either type
    gpu.release()


@BOTH
@pytest.mark.parametrize("M,K,ff", [(1, 64, 32), (5, 128, 40), (66, 192, 100), (200, 128, 640), (700, 64, 1000), (2, 1024, 70), (40, 768, 500)])
def test_gated_linear_clamps(gpu, dt, M, K, ff):
    rng = np.random.default_rng(ff)
    x, gw, uw = rounded(2 * rng.standard_normal((M, K))), rounded(rng.standard_normal((ff, K)) / K ** 0.5), \
        rounded(rng.standard_normal((ff, K)) / K ** 0.5)
    limit, ld = 0.75, up64(ff)
    packed = pack_gated(gw, uw, ld)
    out = zeros(gpu, (M, ld), dt)
    gate = gpu.B.GateParams(limit, 1.702, 1.0)
    call(gpu, "lcu_linear_gated", out, ld, put(gpu, x, dt), put(gpu, packed, dt), C.byref(gate), dt, M, K, 2 * ld)
    want = S.expert(x, gw, uw, np.eye(ff), limit)
    assert (x @ gw.T > limit).any() and (np.abs(x @ uw.T) > limit).any()
    close(get(gpu, out, (M, ld), dt)[:, :ff], want, dt)
    gpu.release()


# ---- norms and the residual -----------------------------------------------------------------------------
@BOTH
@pytest.mark.parametrize("width,groups", [(96, 1), (100, 5), (192, 3), (512, 2), (768, 3), (1280, 5), (2048, 8), (3000, 4), (4352, 17), (12288, 2), (10000, 2000)])
@pytest.mark.parametrize("rows", [1, 3])
def test_grouped_norm_residual_and_embedding(gpu, dt, width, groups, rows):
    rng = np.random.default_rng(width + groups)
    ld, eps, vocab, n_pos, start = up64(width), 1e-3, 11, 9, 4
    ws = [1 + 0.3 * rng.standard_normal(width) for _ in range(3)]
    dw = [put(gpu, pad(w, ld)) for w in ws]
    # parts of very different size: a norm over the wrong part shows
    part = np.repeat(10.0 ** rng.integers(-2, 3, groups), width // groups)
    table, pos = rounded(part * rng.standard_normal((vocab, width))), rounded(part * rng.standard_normal((n_pos, width)))
    ids = rng.integers(0, vocab, rows)
    x, h = zeros(gpu, (rows, ld)), zeros(gpu, (rows, ld), dt)
    call(gpu, "lcu_embed_pos_norm", x, h, ints(gpu, ids), rows, put(gpu, pad(table, ld), dt), vocab, put(gpu, pad(pos, ld), dt), n_pos,
         ints(gpu, [start]), dw[0], dw[1], dt, width, ld, groups, eps)
    e = S.group_rms_norm(table[ids] + pos[start:start + rows], ws[0], groups, eps)
    close(get(gpu, x, (rows, ld))[:, :width], e, F32)
    close(get(gpu, h, (rows, ld), dt)[:, :width], S.group_rms_norm(e, ws[1], groups, eps), dt)
    # the sum of two expert rows and a gated shared one, from scattered places
    out, shared, gate = part * rng.standard_normal((2 * rows, width)), part * rng.standard_normal((rows, width)), rng.random(rows)
    inverse = rng.permutation(2 * rows)
    call(gpu, "lcu_residual_norm", x, h, put(gpu, pad(out, ld)), ints(gpu, inverse), 2, put(gpu, pad(shared, ld)), put(gpu, gate),
         dw[1], dw[2], dt, rows, width, ld, groups, eps)
    m = out[inverse].reshape(rows, 2, width).sum(1) + gate[:, None] * shared
    want = e + S.group_rms_norm(m, ws[1], groups, eps)
    got = get(gpu, x, (rows, ld))
    close(got[:, :width], want, F32)
    assert (got[:, width:] == 0).all()
    close(get(gpu, h, (rows, ld), dt)[:, :width], S.group_rms_norm(want, ws[2], groups, eps), dt)
    call(gpu, "lcu_group_norm", h, x, ints(gpu, [rows - 1]), dw[0], dt, 1, width, ld, groups, eps)
    close(get(gpu, h, (1, ld), dt)[:, :width], S.group_rms_norm(want[-1:], ws[0], groups, eps), dt)
    gpu.release()


@pytest.mark.parametrize("width,groups,experts,top", [(96, 1, 5, 1), (320, 5, 12, 3), (1024, 2, 40, 2), (4352, 17, 70, 4), (9216, 9, 17, 2), (12288, 3, 512, 5), (11000, 1000, 20, 1)])
def test_one_row_step_with_router(gpu, width, groups, experts, top):
    rng = np.random.default_rng(width)
    ld, eps = up64(width), 1e-5
    x, out, gate = rng.standard_normal(width), rng.standard_normal((2, width)), np.array([0.3])
    shared = rng.standard_normal(width)
    wa, wn = 1 + 0.2 * rng.standard_normal(width), 1 + 0.2 * rng.standard_normal(width)
    router = rounded(rng.standard_normal((experts + 1, width)) / width ** 0.5)
    dx, dh = put(gpu, pad(x, ld)), zeros(gpu, ld, BF16)
    e, w, sg = ints(gpu, np.zeros(top)), zeros(gpu, top), zeros(gpu, 1)
    call(gpu, "lcu_decode_residual_router", dx, dh, put(gpu, pad(out, ld)), 2, put(gpu, pad(shared, ld)), put(gpu, gate),
         put(gpu, pad(wa, ld)), put(gpu, pad(wn, ld)), width, ld, groups, eps, put(gpu, pad(router, ld), BF16), experts, top, e, w, sg)
    want = x + S.group_rms_norm(out.sum(0) + gate * shared, wa, groups, eps)
    close(get(gpu, dx, (ld,))[:width], want, F32)
    h = get(gpu, dh, (ld,), BF16)[:width]
    close(h, S.group_rms_norm(want, wn, groups, eps), BF16)
    order, scores = S.route(router[:experts] @ h, top)
    assert list(get_ints(gpu, e, (top,))) == order
    close(get(gpu, w, (top,)), scores, F32)
    close(get(gpu, sg, (1,)), S.sigmoid(router[experts] @ h), F32)
    gpu.release()


# ---- recurrence -----------------------------------------------------------------------------------------
def block_layout(width, blocks):
    """(channel -> padded channel, padded block, row stride)."""
    cb = width // blocks
    bw = (cb + 31) // 32 * 32
    c = np.arange(width)
    return c // cb * bw + c % cb, bw, up64(blocks * bw)


@BOTH
@pytest.mark.parametrize("width,blocks,taps", [(60, 3, 2), (96, 2, 4), (70, 1, 1), (128, 4, 3), (320, 2, 6), (512, 2, 4), (384, 3, 5)])
@pytest.mark.parametrize("cuts", [(150,), (1, 2, 2, 61, 3, 64, 17), (2,) * 5 + (140,)])
def test_recurrence_in_portions(gpu, dt, width, blocks, taps, cuts):
    """Convolution, gates and state over any cut of the tokens; in bfloat16 the one-token kernels take the
    portions of one token."""
    rng = np.random.default_rng(width + taps)
    to, bw, ld = block_layout(width, blocks)
    T, cb = sum(cuts), width // blocks
    z, y = rounded(rng.standard_normal((T, width))), rounded(rng.standard_normal((T, width)))
    cw, cbias = rng.standard_normal((width, taps)) / taps ** 0.5, 0.2 * rng.standard_normal(width)
    ra, ri = (rounded(rng.standard_normal((blocks, cb, cb)) / cb ** 0.5) for _ in range(2))
    ba, bi, lam = rng.standard_normal((blocks, cb)), rng.standard_normal((blocks, cb)), -4 + 3 * rng.standard_normal(width)

    def spread(v, shape):
        out = np.zeros(shape)
        out[..., to] = v
        return out

    def square(w):
        out = np.zeros((blocks, bw, bw))
        out[:, :cb, :cb] = w
        return out

    decay = -8.0 * S.softplus(lam)
    args = dict(conv=put(gpu, spread(cw.T, (taps, ld))), convb=put(gpu, spread(cbias, ld)), wr=put(gpu, square(ra), dt),
                wi=put(gpu, square(ri), dt), br=put(gpu, spread(ba.ravel(), ld)), bi=put(gpu, spread(bi.ravel(), ld)),
                decay=put(gpu, spread(decay, ld)))
    conv_state, state = zeros(gpu, (max(taps - 1, 1), ld), dt), zeros(gpu, ld)
    channels = blocks * bw
    got_u, got_s, at = [], [], 0
    for n in cuts:
        dz, dy = put(gpu, spread(z[at:at + n], (n, ld)), dt), put(gpu, spread(y[at:at + n], (n, ld)), dt)
        u, out = zeros(gpu, (n, ld), dt), zeros(gpu, (n, ld), dt)
        call(gpu, "lcu_conv_causal", u, dz, ld, args["conv"], args["convb"], conv_state, taps, 0, dt, n, channels, ld)
        if n == 1 and dt == BF16:
            call(gpu, "lcu_decode_recurrent_step", out, u, dy, args["wr"], args["wi"], args["br"], args["bi"], args["decay"], state,
                 channels, bw)
        else:
            scratch = zeros(gpu, gpu.L().lcu_gated_recurrence_scratch(n, ld) // 4)
            call(gpu, "lcu_gated_recurrence", out, u, dy, ld, args["wr"], args["wi"], args["br"], args["bi"], args["decay"], state, scratch,
                 dt, n, channels, bw, ld)
        got_u.append(get(gpu, u, (n, ld), dt)[:, to])
        got_s.append(get(gpu, out, (n, ld), dt)[:, to])
        at += n
    u = S.causal_conv(z, cw, cbias)
    close(np.concatenate(got_u), u, dt)
    if dt == BF16:
        u = np.concatenate(got_u)   # the rest is held to the rounded inputs the kernels saw
    s = S.gated_linear_recurrence(u, S.block_gate(u, ra, ba), S.block_gate(u, ri, bi), lam)
    close(np.concatenate(got_s), s * y, dt)
    close(get(gpu, state, (ld,))[to], s[-1], F32, f32=2e-5)
    assert (get(gpu, state, (ld,))[np.setdiff1d(np.arange(channels), to)] == 0).all()
    gpu.release()


def test_recurrence_remembers_for_thousands_of_tokens(gpu):
    """A decay of almost one: an impulse at the first token is still in the state 5000 tokens later, to fp32."""
    width, T, ld = 32, 5000, 64
    lam = np.full(width, -14.0)                    # softplus ~ 8.3e-7: log a ~ -3.3e-6 per token
    u = np.zeros((T, width))
    u[0] = 1.0
    y = np.ones((T, width))
    wz = np.zeros((1, width, width))
    state = zeros(gpu, ld)
    scratch = zeros(gpu, gpu.L().lcu_gated_recurrence_scratch(T, ld) // 4)
    for dt in (BF16, F32):
        state = zeros(gpu, ld)
        out = zeros(gpu, (T, ld), dt)
        call(gpu, "lcu_gated_recurrence", out, put(gpu, pad(u, ld), dt), put(gpu, pad(y, ld), dt), ld, put(gpu, wz, dt), put(gpu, wz, dt),
             zeros(gpu, ld), zeros(gpu, ld), put(gpu, pad(-8.0 * S.softplus(lam), ld)), state, scratch, dt, T, width, width, ld)
        half = np.full((T, width), 0.5)
        want = S.gated_linear_recurrence(u, half, half, lam)
        close(get(gpu, state, (ld,))[:width], want[-1], F32, f32=1e-4)
        assert want[-1, 0] > 0.9 * want[0, 0]
    gpu.release()


# ---- attention ------------------------------------------------------------------------------------------
PADDED_V = {20: 32, 32: 32, 33: 64, 64: 64, 80: 128, 128: 128, 200: 256}


def attention_case(gpu, dt, heads, kv_heads, dim, vdim, window, keep, T, seed, far=None):
    rng = np.random.default_rng(seed)
    dk, dv = (dim + 31) // 32 * 32, PADDED_V[vdim]
    q, k, v = rng.standard_normal((T, heads, dim)), rng.standard_normal((T, kv_heads, dim)), rng.standard_normal((T, kv_heads, vdim))
    if far is not None:
        # queries `far` tokens behind a key all but copy it: one score stands out
        for i in range(far, T):
            for h in range(heads):
                q[i, h] = 3.0 * k[i - far, h // (heads // kv_heads)]
    q, k, v = rounded(q), rounded(k), rounded(v)
    scale, r1, r2 = 1.3 / dim ** 0.5, rng.random(heads), 0.05 + rng.random(heads)
    dr1, dr2 = put(gpu, r1), put(gpu, r2)
    wp = gpu.B.WindowParams(heads, kv_heads, dk, dv, window, keep, scale, dr1.ptr, dr2.ptr)
    want = S.windowed_attention(q, k, v, scale, r1, r2, window, keep)
    return dict(q=pad(q, dk), k=pad(k, dk), v=pad(v, dv), want=want, wp=wp, dk=dk, dv=dv, heads=heads, kv=kv_heads, vdim=vdim, T=T)


def run_attention(gpu, c, dt, cuts):
    heads, kv, dk, dv, T = c["heads"], c["kv"], c["dk"], c["dv"], c["T"]
    kc, vc = put(gpu, c["k"], dt), put(gpu, c["v"], dt)
    got, at = [], 0
    arrived = ints(gpu, np.zeros(kv))
    for n in cuts:
        ldq, ldo = heads * dk, heads * dv
        q, out = put(gpu, c["q"][at:at + n], dt), zeros(gpu, (n, ldo), dt)
        if n == 1 and dt == BF16:
            call(gpu, "lcu_attention_windowed_decode", out, q, kc, vc, ints(gpu, [at]), T, C.byref(c["wp"]), arrived)
        else:
            call(gpu, "lcu_attention_windowed", out, ldo, q, ldq, kc, vc, at, C.byref(c["wp"]), dt, n)
        got.append(get(gpu, out, (n, heads, dv), dt)[..., :c["vdim"]])
        at += n
    assert not get_ints(gpu, arrived, (kv,)).any()
    return np.concatenate(got)


@BOTH
@pytest.mark.parametrize("heads,kv,dim,vdim,window,keep", [
    (4, 2, 24, 20, 16, 0), (6, 1, 40, 33, 1, 3), (3, 3, 96, 64, 65, 1), (8, 2, 64, 128, 100, 70), (16, 1, 128, 128, 40, 5),
    (2, 2, 160, 200, 64, 64), (5, 5, 56, 80, 500, 2), (12, 2, 32, 32, 33, 130)])
def test_windowed_attention_in_portions(gpu, dt, heads, kv, dim, vdim, window, keep):
    T = 200
    c = attention_case(gpu, dt, heads, kv, dim, vdim, window, keep, T, heads * 100 + dim)
    whole = run_attention(gpu, c, dt, (T,))
    close(whole, c["want"], dt, bf16=2.0 ** -7)
    cut = run_attention(gpu, c, dt, (1, 1, 2, 3, 59, 64, 1, 2, 1, 37) + (1,) * 29)
    close(cut, c["want"], dt, bf16=2.0 ** -7)
    gpu.release()


@BOTH
@pytest.mark.parametrize("window,keep,edge", [(48, 0, "window"), (64, 6, "window"), (65, 0, "window"), (32, 0, "window"), (20, 70, "keep")])
def test_attention_edges(gpu, dt, window, keep, edge):
    """One key stands out: just inside the window it decides the output, one token further it must not be seen;
    the same for the last kept token and the one behind it."""
    heads, kv, dim, vdim, T = 4, 2, 48, 20, 180
    for dist in (window - 1, window, window + 1):
        c = attention_case(gpu, dt, heads, kv, dim, vdim, window, keep, T, 7 + dist, far=dist)
        whole = run_attention(gpu, c, dt, (T,))
        close(whole, c["want"], dt, bf16=2.0 ** -7)
        close(run_attention(gpu, c, dt, (90,) + (1,) * 90), c["want"], dt, bf16=2.0 ** -7)
        seen = attention_case(gpu, dt, heads, kv, dim, vdim, window + 1, keep, T, 7 + dist, far=dist)["want"]
        if dist == window:   # a window one longer would have shown
            assert np.max(np.abs(seen - c["want"])) > 0.2
    if edge == "keep":
        rng = np.random.default_rng(3)
        for key in (keep - 1, keep):
            c = attention_case(gpu, dt, heads, kv, dim, vdim, window, keep, T, 5)
            c["q"][100:, :, :dim] = rounded(3.0 * np.repeat(c["k"][key, :, :dim], heads // kv, axis=0))
            r1, r2 = (gpu.B.from_device(b, (heads,), np.float32).astype(float) for b in last_two_vectors(gpu))
            c["want"] = S.windowed_attention(c["q"][..., :dim], c["k"][..., :dim], c["v"][..., :vdim], c["wp"].scale, r1, r2, window, keep)
            close(run_attention(gpu, c, dt, (60, 70) + (1,) * 50), c["want"], dt, bf16=2.0 ** -7)
            dominated = np.max(np.abs(c["want"][150, 0] - c["v"][key, 0, :vdim])) < 0.5
            assert dominated == (key < keep)
    gpu.release()


def last_two_vectors(gpu):
    """Device copies of r1 and r2 of the latest attention_case."""
    return gpu._keep[-2:]


def test_attention_far_key_over_a_long_window(gpu):
    """A key 900 tokens back among hundreds, in a prompt and token by token (several slices of keys)."""
    c = attention_case(gpu, BF16, 8, 2, 64, 64, 1000, 3, 1100, 1, far=900)
    close(run_attention(gpu, c, BF16, (1060,) + (1,) * 40), c["want"], BF16, bf16=2.0 ** -7)
    gpu.release()


@BOTH
def test_kv_rows_and_value_mixing(gpu, dt):
    rng = np.random.default_rng(0)
    n, ctx, qc, kc, vc, start = 5, 20, 32, 64, 32, 7
    ld = up64(qc + kc + vc)
    qkv = rounded(rng.standard_normal((n, ld)))
    first = rounded(rng.standard_normal((n, vc)))
    for mode, lam in ((0, 0.0), (1, 0.0), (2, 0.3)):
        kcache, vcache, vf = zeros(gpu, (ctx, kc), dt), zeros(gpu, (ctx, vc), dt), put(gpu, first, dt)
        call(gpu, "lcu_kv_store", kcache, vcache, put(gpu, qkv, dt), ld, qc, kc, vc, vf, mode, put(gpu, [lam]), ints(gpu, [start]), ctx, dt, n)
        k, v, f = get(gpu, kcache, (ctx, kc), dt), get(gpu, vcache, (ctx, vc), dt), get(gpu, vf, (n, vc), dt)
        own = qkv[:, qc + kc:qc + kc + vc]
        assert (k[start:start + n] == qkv[:, qc:qc + kc]).all() and not k[:start].any() and not k[start + n:].any()
        close(v[start:start + n], S.mix_values(own, first, lam) if mode == 2 else own, dt)
        assert (f == (own if mode == 1 else first)).all()
    gpu.release()


# ---- experts --------------------------------------------------------------------------------------------
@BOTH
@pytest.mark.parametrize("n,K,experts,top", [(1, 64, 3, 1), (5, 192, 12, 2), (70, 128, 17, 4), (33, 320, 70, 3), (40, 64, 1, 1), (18, 64, 200, 8), (20, 128, 512, 6)])
def test_router(gpu, dt, n, K, experts, top):
    rng = np.random.default_rng(K + experts)
    h, w = rounded(rng.standard_normal((n, K))), rounded(rng.standard_normal((experts + 1, K)) / K ** 0.5)
    e, wt, sg = ints(gpu, np.zeros((n, top))), zeros(gpu, (n, top)), zeros(gpu, n)
    call(gpu, "lcu_router", e, wt, sg, put(gpu, h, dt), put(gpu, w, dt), experts, top, dt, n, K)
    got, weights = get_ints(gpu, e, (n, top)), get(gpu, wt, (n, top))
    z = h @ w.T
    for t in range(n):
        order, s = S.route(z[t, :experts], top)
        assert list(got[t]) == order
        close(weights[t], s, F32)
    close(get(gpu, sg, (n,)), S.sigmoid(z[:, experts]), F32)
    gpu.release()


@BOTH
@pytest.mark.parametrize("n,K,ff,experts,top,tile", [(1, 64, 40, 3, 2, 64), (7, 128, 33, 5, 1, 64), (50, 64, 100, 4, 4, 128), (300, 128, 64, 3, 2, 256),
                                                     (150, 192, 70, 20, 2, 64)])
def test_experts(gpu, dt, n, K, ff, experts, top, tile):
    """Sorting by expert (one of them gets nothing, one gets every token), both products, and the inverse order."""
    rng = np.random.default_rng(n + ff)
    N, ld, tile = 96, up64(ff), 32 if dt == F32 else tile
    h = rounded(rng.standard_normal((n, K)))
    gate, up = (rounded(rng.standard_normal((experts, ff, K)) / K ** 0.5) for _ in range(2))
    down = rounded(rng.standard_normal((experts, N, ff)) / ff ** 0.5)
    choice = np.stack([rng.permutation(experts - 1)[:top] if experts > top else rng.permutation(experts)[:top] for _ in range(n)])
    weight = rng.random((n, top))
    rows, max_tiles = n * top, n * top // tile + experts
    plan = gpu.B.ExpertPlan()
    keep = {}
    for name, count in (("row_token", rows), ("row_weight", rows), ("inverse", rows), ("tile_expert", max_tiles), ("tile_row", max_tiles),
                        ("expert_end", experts), ("n_tiles", 1)):
        keep[name] = ints(gpu, np.zeros(count))
        setattr(plan, name, keep[name].ptr)
    plan.tile_rows, plan.max_tiles = tile, max_tiles
    call(gpu, "lcu_experts_plan", C.byref(plan), ints(gpu, choice), put(gpu, weight), n, top, experts)
    packed = np.stack([pack_gated(gate[e], up[e], ld) for e in range(experts)])
    es = 2 if dt == BF16 else 4
    hidden, out = zeros(gpu, (rows, ld), dt), zeros(gpu, (rows, N))
    g = gpu.B.GateParams(0.8, 1.702, 1.0)
    call(gpu, "lcu_experts_up", hidden, ld, put(gpu, h, dt), put(gpu, packed, dt), 2 * ld * K * es, C.byref(g), C.byref(plan), dt, n, K, 2 * ld)
    call(gpu, "lcu_experts_down", out, N, hidden, put(gpu, pad(down, ld), dt), N * ld * es, C.byref(plan), dt, rows, ld, N)
    got, inv = get(gpu, out, (rows, N)), get_ints(gpu, keep["inverse"], (n, top))
    assert sorted(inv.ravel()) == list(range(rows))
    want = np.stack([[S.expert(weight[t, k] * h[t], gate[e], up[e], down[e], 0.8) for k, e in enumerate(choice[t])] for t in range(n)])
    close(got[inv], want, dt)
    # the one-token kernels on the last token, with a shared expert of another size
    if dt == BF16:
        sff = ff + 50
        sld = up64(sff)
        sg, su, sd = (rounded(rng.standard_normal(s) / 8) for s in ((sff, K), (sff, K), (N, sff)))
        hid, shid, res = zeros(gpu, (top, ld), BF16), zeros(gpu, sld, BF16), zeros(gpu, (top + 1, N))
        ch, g2 = ints(gpu, choice[-1]), gpu.B.GateParams(0.5, 1.702, 1.0)
        call(gpu, "lcu_decode_experts_up", hid, shid, put(gpu, h[-1], BF16), ch, put(gpu, weight[-1]), put(gpu, packed, BF16),
             2 * ld * K * 2, C.byref(g), put(gpu, pack_gated(sg, su, sld), BF16), C.byref(g2), top, ld, sld, K)
        call(gpu, "lcu_decode_experts_down", res, N, hid, ch, put(gpu, pad(down, ld), BF16), N * ld * 2, top, ld, shid,
             put(gpu, pad(sd, sld), BF16), sld, N)
        got = get(gpu, res, (top + 1, N))
        close(got[:top], want[-1], BF16)
        close(got[top], S.expert(h[-1], sg, su, sd, 0.5), BF16)
    gpu.release()


@pytest.mark.parametrize("n", [1, 7, 640, 32000, 50257])
def test_argmax_and_softmax(gpu, n):
    rng = np.random.default_rng(n)
    x = np.round(rng.standard_normal(n) * 4).astype(np.float32)     # ties: the first maximum counts
    idx, probs = ints(gpu, [0]), gpu.dev_keep(np.zeros(n, np.float16))
    dx = put(gpu, x)
    call(gpu, "lcu_argmax_f32", idx, dx, n)
    call(gpu, "lcu_softmax_f32", probs, dx, n, 0.7)
    gpu.B.check(gpu.L().lcu_sync(gpu.stream))
    assert get_ints(gpu, idx, (1,))[0] == x.argmax()
    p = np.exp((x.astype(float) - x.max()) / 0.7)
    assert np.max(np.abs(gpu.host(probs, (n,), np.float16) - p / p.sum())) < 1e-3
    gpu.release()


def test_unsupported_shapes_are_refused_before_any_launch(gpu):
    L, B = gpu.L(), gpu.B
    a = zeros(gpu, 4096)
    assert L.lcu_linear(a.ptr, 0, 64, a.ptr, a.ptr, None, 0, 0, 4, 40, 64, gpu.stream) == -2      # K not a multiple of 64
    assert L.lcu_linear(a.ptr, 0, 8, a.ptr, a.ptr, None, 0, 0, 4, 64, 64, gpu.stream) == -2       # rows shorter than N
    assert L.lcu_linear(a.ptr, 0, 64, a.ptr, a.ptr, None, 0, 7, 4, 64, 64, gpu.stream) == -2      # no such element type
    wp = B.WindowParams(3, 2, 64, 64, 8, 0, 1.0, a.ptr, a.ptr)                                    # 3 heads on 2
    assert L.lcu_attention_windowed(a.ptr, 192, a.ptr, 192, a.ptr, a.ptr, 0, C.byref(wp), 0, 1, gpu.stream) == -2
    assert L.lcu_router(a.ptr, a.ptr, None, a.ptr, a.ptr, 4, 5, 0, 1, 64, gpu.stream) == -2       # more choices than experts
    assert L.lcu_group_norm(a.ptr, a.ptr, None, a.ptr, 0, 1, 100, 128, 3, 1e-5, gpu.stream) == -2  # 100 in 3 parts
    assert L.lcu_gated_recurrence(*([a.ptr] * 3), 64, *([a.ptr] * 7), 0, 1, 64, 20, 64, gpu.stream) == -2  # block width
    gpu.release()
