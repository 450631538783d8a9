"""Latent attention, the gated delta rule and what goes with them, each on its own against the plain restatement
(plain_latent_delta.py), in both element types; the sizes are ragged.  Keys that matter are made to stand out: one
score decides the output where the key is seen, and must leave no trace one token further."""
import ctypes as C

import numpy as np
import pytest

import plain_latent_delta as D
import plain_stack as S
from layered_helpers import BF16, BOTH, F32, call, close, get, gpu, ints, pack_gated, pad, put, rounded, up64, zeros  # noqa: F401

pytestmark = pytest.mark.gpu


def up32(n):
    return (n + 31) // 32 * 32


def value_size(n):
    return 32 if n <= 32 else 64 if n <= 64 else 128 if n <= 128 else 256


# ---- rows -------------------------------------------------------------------------------------------------
@BOTH
@pytest.mark.parametrize("width,rows", [(70, 1), (70, 5), (960, 3), (4200, 2)])
@pytest.mark.parametrize("ahead", [False, True])
def test_scaled_embedding_and_norm_behind(gpu, dt, width, rows, ahead):
    """x = scale table[id]; x += norm(m); the next sublayer's input is x itself, or its norm."""
    rng = np.random.default_rng(width + rows)
    ld, eps, vocab, scale = up64(width), 1e-3, 9, 5.3
    table, out = rounded(rng.standard_normal((vocab, width))), rng.standard_normal((rows, width))
    w1, w2 = (1 + 0.3 * rng.standard_normal(width) for _ in range(2))
    ids = rng.integers(0, vocab, rows)
    d1, d2 = put(gpu, pad(w1, ld)), put(gpu, pad(w2, ld)) if ahead else None
    x, h = zeros(gpu, (rows, ld)), zeros(gpu, (rows, ld), dt)
    seen = lambda v: D.rms_norm(v, w2, eps) if ahead else v
    call(gpu, "lcu_embed_scaled", x, h, ints(gpu, ids), rows, put(gpu, pad(table, ld), dt), vocab, scale, d2, dt, width, ld, 1, eps)
    e = table[ids] * np.float32(scale)
    close(get(gpu, x, (rows, ld))[:, :width], e, F32)
    close(get(gpu, h, (rows, ld), dt)[:, :width], seen(e), dt)
    call(gpu, "lcu_residual_norm", x, h, put(gpu, pad(out, ld)), None, 1, None, None, d1, d2, dt, rows, width, ld, 1, eps)
    want = e + D.rms_norm(out, w1, eps)
    close(get(gpu, x, (rows, ld))[:, :width], want, F32)
    got = get(gpu, h, (rows, ld), dt)
    close(got[:, :width], seen(want), dt)
    assert (got[:, width:] == 0).all()
    if rows == 1 and dt == BF16:   # the one-token step's launch
        call(gpu, "lcu_decode_residual_router", x, h, put(gpu, pad(out, ld)), 1, None, None, d1, d2, width, ld, 1, eps, None, 0, 0, None, None,
             None)
        want = want + D.rms_norm(out, w1, eps)
        close(get(gpu, x, (rows, ld))[:, :width], want, F32)
        close(get(gpu, h, (rows, ld), dt)[:, :width], seen(want), dt)
    gpu.release()


@BOTH
@pytest.mark.parametrize("M,K,N,tail", [(1, 64, 40, 6), (5, 128, 160, 2), (70, 192, 200, 17), (300, 320, 1088, 64), (40, 1024, 96, 4)])
def test_linear_with_a_tail_in_fp32(gpu, dt, M, K, N, tail):
    rng = np.random.default_rng(M + N)
    x, w = rounded(rng.standard_normal((M, K))), rounded(rng.standard_normal((N, K)) / K ** 0.5)
    cut, ldo = N - tail, up64(N)
    out, rest = zeros(gpu, (M, ldo), dt), zeros(gpu, (M, tail))
    call(gpu, "lcu_linear_tail", out, ldo, rest, tail, cut, put(gpu, x, dt), put(gpu, w, dt), dt, M, K, N)
    want = x @ w.T
    got = get(gpu, out, (M, ldo), dt)
    close(got[:, :cut], want[:, :cut], dt)
    assert (got[:, cut:] == 0).all()
    close(get(gpu, rest, (M, tail)), want[:, cut:], F32)
    gpu.release()


@pytest.mark.parametrize("K,N", [(64, 1), (192, 70), (2112, 33), (4224, 101)])
def test_one_row_products(gpu, K, N):
    rng = np.random.default_rng(K)
    x, w = rounded(rng.standard_normal(K)), rounded(rng.standard_normal((N, K)) / K ** 0.5)
    out = zeros(gpu, up64(N), BF16)
    call(gpu, "lcu_decode_linear_bf16", out, put(gpu, x, BF16), put(gpu, w, BF16), K, N)
    got = get(gpu, out, (up64(N),), BF16)
    close(got[:N], w @ x, BF16, scale=3.0)
    assert (got[N:] == 0).all()
    ff, ld = N, up64(N)
    g, u = w, rounded(rng.standard_normal((ff, K)) / K ** 0.5)
    for limit in (np.inf, 0.4):
        gate = gpu.B.GateParams(limit, 1.0, 0.0)
        call(gpu, "lcu_decode_gated", out, put(gpu, x, BF16), put(gpu, pack_gated(g, u, ld), BF16), C.byref(gate), ld, K)
        a, b = np.minimum(g @ x, limit), np.clip(u @ x, -limit, limit)
        close(get(gpu, out, (ld,), BF16)[:ff], D.silu(a) * b, BF16)
    gpu.release()


@BOTH
@pytest.mark.parametrize("channels,plain,taps", [(64, 32, 4), (192, 64, 2), (128, 96, 1), (320, 160, 7)])
@pytest.mark.parametrize("cuts", [(100,), (1, 1, 2, 3, 1, 60, 2, 30), (2,) * 4 + (1,) * 30])
def test_convolution_with_silu_in_portions(gpu, dt, channels, plain, taps, cuts):
    """Projections, convolution and silu over any cut; one token in bfloat16 takes the fused launch."""
    rng = np.random.default_rng(channels + taps)
    K, tail, T = 128, 6, sum(cuts)
    N, ld = channels + plain + tail, channels + plain
    x, w = rounded(rng.standard_normal((T, K))), rounded(rng.standard_normal((N, K)) / K ** 0.5)
    cw = rng.standard_normal((channels, taps)) / taps ** 0.5
    dw, dc, state = put(gpu, w, dt), put(gpu, cw.T), zeros(gpu, (max(taps - 1, 1), channels), dt)
    got, at = [], 0
    for n in cuts:
        u, rows, rest = zeros(gpu, (n, channels), dt), zeros(gpu, (n, ld), dt), zeros(gpu, (n, tail))
        xs = put(gpu, x[at:at + n], dt)
        if n == 1 and dt == BF16:
            own = zeros(gpu, plain, dt)
            call(gpu, "lcu_decode_delta_in", u, own, rest, state, xs, dw, dc, taps, K, channels, plain, N)
            p = get(gpu, own, (1, plain), dt)
        else:
            call(gpu, "lcu_linear_tail", rows, ld, rest, tail, ld, xs, dw, dt, n, K, N)
            call(gpu, "lcu_conv_causal", u, rows, ld, dc, None, state, taps, 1, dt, n, channels, channels)
            p = get(gpu, rows, (n, ld), dt)[:, channels:]
        got.append((get(gpu, u, (n, channels), dt), p, get(gpu, rest, (n, tail))))
        at += n
    z = x @ w.T
    u, p, rest = (np.concatenate(parts) for parts in zip(*got))
    seen = rounded(z[:, :channels]) if dt == BF16 else z[:, :channels]
    close(u, D.conv_silu(seen, cw), dt)
    close(p, z[:, channels:ld], dt)
    close(rest, z[:, ld:], F32)
    gpu.release()


# ---- latents and rotation -----------------------------------------------------------------------------------
ROTS = [dict(dims=16, base=1e4), dict(dims=48, base=250.0, scaling=dict(factor=8.0, original=300, fast=20.0, slow=0.5)),
        dict(dims=64, base=5e5, scaling=dict(factor=1.0, original=4096, fast=32.0, slow=1.0)),
        dict(dims=6, base=30.0, scaling=dict(factor=3.0, original=50, fast=4.0, slow=4.0))]


def frequencies(rot):
    return D.stretched_frequencies(rot["dims"], rot["base"], rot.get("scaling"))


@BOTH
@pytest.mark.parametrize("rot", ROTS, ids=lambda r: str(r["dims"]))
@pytest.mark.parametrize("heads,dim,rank,extra,start", [(3, 20, 45, 0, 0), (5, 64, 130, 8, 37), (1, 33, 300, 0, 4000)])
def test_latent_rows(gpu, dt, rot, heads, dim, rank, extra, start):
    """Normed latents and rotated key parts into the caches, queries rotated in place; `extra` dimensions of the rotated
    part stay as they are."""
    rng = np.random.default_rng(heads + rank)
    n, r = 7, rot["dims"]
    dr, dn, ldc, max_pos, eps = up32(r + extra), up32(dim), up64(rank), start + 9, 1e-2
    head = dn + dr
    latent_at, key_at = heads * head, heads * head + ldc
    ld = up64(key_at + dr)
    rows = np.zeros((n, ld))
    q, c, k = (rounded(rng.standard_normal(s)) for s in ((n, heads, dim + r + extra), (n, rank), (n, r + extra)))
    for h in range(heads):
        rows[:, h * head:h * head + dim] = q[:, h, :dim]
        rows[:, h * head + dn:h * head + dn + r + extra] = q[:, h, dim:]
    rows[:, latent_at:latent_at + rank] = c
    rows[:, key_at:key_at + r + extra] = k
    w = 1 + 0.3 * rng.standard_normal(rank)
    f, gain = frequencies(rot)
    drows, lat, keys = put(gpu, rows, dt), zeros(gpu, (max_pos, ldc), dt), zeros(gpu, (max_pos, dr), dt)
    args = gpu.B.LatentRows(drows.ptr, ld, n, latent_at, key_at, dn, 1, 0, 0, max_pos, put(gpu, pad(w, ldc)).ptr, None, None, lat.ptr, keys.ptr,
                            put(gpu, f).ptr, gain, eps, ints(gpu, [start]).ptr)
    p = gpu.B.LatentParams(heads, dn, dr, r, 32, rank, ldc, 10, 1.0)
    call(gpu, "lcu_latent_rows", C.byref(args), C.byref(p), dt)
    got = get(gpu, lat, (max_pos, ldc), dt)
    close(got[start:start + n, :rank], D.rms_norm(c, w, eps), dt)
    assert (got[:start] == 0).all() and (got[start + n:] == 0).all() and (got[:, rank:] == 0).all()
    turned = lambda x: np.concatenate([D.rotate_pairs(x[..., :r], rot, start), x[..., r:]], -1)
    got = get(gpu, keys, (max_pos, dr), dt)
    close(got[start:start + n, :r + extra], turned(k), dt, f32=1e-3 if start > 1000 else 2e-5)
    assert (got[:, r + extra:] == 0).all()
    got, want = get(gpu, drows, (n, ld), dt), rows.copy()
    for h in range(heads):
        want[:, h * head + dn:h * head + dn + r + extra] = turned(q[:, h, dim:])
    close(got, want, dt, f32=1e-3 if start > 1000 else 2e-5)
    assert (got[:, :dim] == rows[:, :dim]).all()
    gpu.release()


@BOTH
@pytest.mark.parametrize("rank,q_rank", [(40, 33), (70, 200)])
def test_latent_of_the_queries(gpu, dt, rank, q_rank):
    rng = np.random.default_rng(rank)
    n, start, ldc, low_ld, eps = 5, 3, up64(rank), up64(q_rank), 1e-3
    ld = low_ld + ldc
    rows = np.zeros((n, ld))
    a, c = rounded(rng.standard_normal((n, q_rank))), rounded(rng.standard_normal((n, rank)))
    rows[:, :q_rank], rows[:, low_ld:low_ld + rank] = a, c
    wa, wc = 1 + 0.3 * rng.standard_normal(q_rank), 1 + 0.3 * rng.standard_normal(rank)
    drows, low, lat = put(gpu, rows, dt), zeros(gpu, (n, low_ld), dt), zeros(gpu, (n + start, ldc), dt)
    args = gpu.B.LatentRows(drows.ptr, ld, n, low_ld, 0, 0, 0, q_rank, low_ld, n + start, put(gpu, pad(wc, ldc)).ptr, put(gpu, pad(wa, low_ld)).ptr,
                            low.ptr, lat.ptr, None, None, 1.0, eps, ints(gpu, [start]).ptr)
    p = gpu.B.LatentParams(2, 32, 0, 0, 32, rank, ldc, 10, 1.0)
    call(gpu, "lcu_latent_rows", C.byref(args), C.byref(p), dt)
    close(get(gpu, low, (n, low_ld), dt)[:, :q_rank], D.rms_norm(a, wa, eps), dt)
    close(get(gpu, lat, (n + start, ldc), dt)[start:, :rank], D.rms_norm(c, wc, eps), dt)
    gpu.release()


# ---- attention over latents, and over keys multiplied out of them -----------------------------------------------
def attention_case(seed, heads, dim, rot, vdim, rank, T, window, sink, gate, far=None, strength=14.0):
    """Latents, rotated key parts, head matrices and queries.  far: the query `far` tokens behind a key is made for it:
    its score is `strength`, the others are around one."""
    rng = np.random.default_rng(seed)
    r = lambda *s: rounded(rng.standard_normal(s))
    c, kr = r(T, rank), r(T, rot)
    uk, uv = rounded(rng.standard_normal((heads, dim, rank)) / rank ** 0.5), rounded(rng.standard_normal((heads, vdim, rank)) / rank ** 0.5)
    q = r(T, heads, dim + rot)
    k = np.concatenate([np.einsum("tr,hdr->thd", c, uk), np.repeat(kr[:, None], heads, 1)], -1)
    scale = 1.1 / (dim + rot) ** 0.5
    if far is not None:
        for i in range(far, T):
            q[i] = strength / scale * k[i - far] / (k[i - far] ** 2).sum(-1, keepdims=True)
        q = rounded(q)
    return dict(heads=heads, dim=dim, rot=rot, vdim=vdim, rank=rank, T=T, window=window, c=c, kr=kr, uk=uk, uv=uv, q=q, k=k, scale=scale,
                v=np.einsum("tr,her->the", c, uv), sink=rng.standard_normal(heads) + 1.0 if sink else None,
                gate=r(T, heads, vdim) if gate else None)


def expected(x, start, n, window="own"):
    o = D.masked_attention(x["q"][start:start + n], x["k"][:start + n], x["v"][:start + n], x["scale"], x["window"] if window == "own" else window,
                           x["sink"], start)
    return o * S.sigmoid(x["gate"][start:start + n]) if x["gate"] is not None else o


def over_latents(G, x, start, n, max_pos=None):
    """lcu_latent_queries and lcu_latent_attention for n tokens from `start` on."""
    H, dn, dr, dv, ldc = x["heads"], up32(x["dim"]), up32(x["rot"]), value_size(x["vdim"]), up64(x["rank"])
    max_pos = max_pos or x["T"]
    p = G.B.LatentParams(H, dn, dr, x["rot"], dv, x["rank"], ldc, x["window"] or 2 ** 31 - 1, x["scale"])
    assert G.L().lcu_latent_attention_fits(C.byref(p))
    q = np.zeros((n, H, dn + dr))
    q[..., :x["dim"]], q[..., dn:dn + x["rot"]] = x["q"][start:start + n, :, :x["dim"]], x["q"][start:start + n, :, x["dim"]:]
    uk_t = np.zeros((H, ldc, dn))
    uk_t[:, :x["rank"], :x["dim"]] = x["uk"].transpose(0, 2, 1)
    uv = np.zeros((H, dv, ldc))
    uv[:, :x["vdim"], :x["rank"]] = x["uv"]
    dq, ql, out = put(G, q, BF16), zeros(G, (n, H, ldc), BF16), zeros(G, (n, H, dv), BF16)
    call(G, "lcu_latent_queries", ql, dq, H * (dn + dr), put(G, uk_t, BF16), C.byref(p), None, n)
    # what lies behind the last token must not be looked at
    c, kr = np.full((max_pos, ldc), 77.0), np.full((max_pos, max(dr, 1)), 77.0)
    c[:start + n], kr[:start + n] = pad(x["c"], ldc)[:start + n], pad(x["kr"], max(dr, 1))[:start + n]
    scratch = G.dev_keep(np.full(G.L().lcu_latent_attention_scratch(C.byref(p), n, max_pos) // 4, np.nan, np.float32))
    gate = put(G, pad(x["gate"][start:start + n], dv), BF16) if x["gate"] is not None else None
    call(G, "lcu_latent_attention", out, H * dv, ql, dq.ptr + 2 * dn, H * (dn + dr), put(G, c, BF16), put(G, kr, BF16), ints(G, [start]), max_pos,
         put(G, uv, BF16), put(G, x["sink"]) if x["sink"] is not None else None, gate, H * dv, C.byref(p), scratch, n)
    return get(G, out, (n, H, dv), BF16)[..., :x["vdim"]]


def over_keys(G, x, start, n, dt):
    """The same with keys and values multiplied out, from the first position that the call sees."""
    H, dn, dr, dv = x["heads"], up32(x["dim"]), up32(x["rot"]), value_size(x["vdim"])
    first = max(0, start - x["window"] + 1) if x["window"] else 0
    seen = start + n - first
    kv = np.zeros((seen, H * (dn + dv)))
    for h in range(H):
        kv[:, h * dn:h * dn + x["dim"]] = x["k"][first:start + n, h, :x["dim"]]
        kv[:, H * dn + h * dv:H * dn + h * dv + x["vdim"]] = x["v"][first:start + n, h]
    q = np.zeros((n, H, dn + dr))
    q[..., :x["dim"]], q[..., dn:dn + x["rot"]] = x["q"][start:start + n, :, :x["dim"]], x["q"][start:start + n, :, x["dim"]:]
    dkv, dq, out = put(G, kv, dt), put(G, q, dt), zeros(G, (n, H, dv), dt)
    w = G.B.WindowParams()
    w.heads = w.kv_heads = H
    w.dk, w.dv, w.window, w.scale, w.dk_shared, w.k_ld, w.v_ld = dn + dr, dv, x["window"] or 2 ** 31 - 1, x["scale"], dr, kv.shape[1], kv.shape[1]
    w.first_position, w.ldg = first, H * dv
    w.k_shared = put(G, pad(x["kr"], dr)[first:start + n], dt).ptr if dr else None
    w.sink = put(G, x["sink"]).ptr if x["sink"] is not None else None
    w.gate = put(G, pad(x["gate"][start:start + n], dv), dt).ptr if x["gate"] is not None else None
    call(G, "lcu_attention_windowed", out, H * dv, dq, H * (dn + dr), dkv, dkv.ptr + H * dn * (2 if dt == BF16 else 4), start, C.byref(w), dt, n)
    return get(G, out, (n, H, dv), dt)[..., :x["vdim"]]


# heads, dim, rotated, vdim, rank, window, sink, gate
SHAPES = [(3, 20, 12, 33, 45, None, True, True), (5, 44, 0, 20, 70, 29, False, False), (16, 64, 32, 64, 128, 65, True, False),
          (1, 8, 2, 8, 10, None, False, True), (20, 96, 64, 100, 300, 64, True, True), (33, 32, 0, 32, 64, 1, False, False),
          (2, 150, 80, 200, 512, None, True, True)]
BF16_ATTENTION = 2.0 ** -6   # queries applied to the key matrix and the weighted latents are rounded once more


@pytest.mark.parametrize("shape", SHAPES, ids=lambda s: "x".join(map(str, s[:5])))
def test_attention_over_latents(gpu, shape):
    H, dim, rot, vdim, rank, window, sink, gate = shape
    x = attention_case(H + dim, H, dim, rot, vdim, rank, 210, window, sink, gate)
    for start, n in ((0, 1), (1, 1), (0, 2), (0, 17), (62, 2), (63, 1), (64, 1), (65, 5), (127, 3), (178, 32), (209, 1)):
        close(over_latents(gpu, x, start, n), expected(x, start, n), BF16, bf16=BF16_ATTENTION)
        gpu.release()
    for max_pos in (300, 5000):   # other slices of the keys
        close(over_latents(gpu, x, 209, 1, max_pos), expected(x, 209, 1), BF16, bf16=BF16_ATTENTION)
        gpu.release()


@BOTH
@pytest.mark.parametrize("shape", SHAPES, ids=lambda s: "x".join(map(str, s[:5])))
def test_attention_over_keys(gpu, dt, shape):
    H, dim, rot, vdim, rank, window, sink, gate = shape
    if up32(dim) + up32(rot) > 256:
        pytest.skip("head of more than 256")
    x = attention_case(H + dim, H, dim, rot, vdim, rank, 210, window, sink, gate)
    for start, n in ((0, 210), (0, 2), (63, 2), (100, 66), (64, 65), (208, 2)):
        close(over_keys(gpu, x, start, n, dt), expected(x, start, n), dt, bf16=2.0 ** -7)
        gpu.release()


@pytest.mark.parametrize("window", [1, 31, 64, 65, 90])
@pytest.mark.parametrize("rot", [0, 24])
def test_window_edges(gpu, window, rot):
    """One key decides the output from just inside the window and leaves no trace from just outside."""
    for dist in (window - 1, window, window + 1):
        x = attention_case(dist, 4, 48, rot, 40, 96, 200, window, False, False, far=dist)
        want = expected(x, 100, 100)
        if dist == window:         # a window one longer would have shown
            assert np.max(np.abs(expected(x, 100, 100, window + 1) - want)) > 0.5
        if dist == window - 1:     # one shorter too
            assert window == 1 or np.max(np.abs(expected(x, 100, 100, window - 1) - want)) > 0.5
        for dt in (BF16, F32):
            close(over_keys(gpu, x, 100, 100, dt), want, dt, bf16=2.0 ** -6)
        for start in (100, 127, 128, 129, 191, 192, 198):
            close(over_latents(gpu, x, start, 2), want[start - 100:start - 98], BF16, bf16=2.0 ** -5)
            close(over_latents(gpu, x, start, 1), want[start - 100:start - 99], BF16, bf16=2.0 ** -5)
        gpu.release()


@pytest.mark.parametrize("dist", [0, 1, 62, 63, 64, 65, 128, 700])
def test_far_keys(gpu, dist):
    """No window: a key `dist` tokens back among hundreds, in a prompt and in decoding."""
    T = dist + 130
    x = attention_case(dist, 3, 40, 16, 48, 72, T, None, True, False, far=dist, strength=20.0)
    start = T - 40
    want = expected(x, start, 40)
    assert np.max(np.abs(want - x["v"][start - dist:T - dist])) < 0.2     # the one key decides
    for dt in (BF16, F32):
        close(over_keys(gpu, x, start, 40, dt), want, dt, bf16=2.0 ** -6)
    for at in range(0, 40, 5):
        close(over_latents(gpu, x, start + at, 1), want[at:at + 1], BF16, bf16=2.0 ** -5)
    gpu.release()


def test_sink_takes_its_share(gpu):
    """A large sink silences a head, a small one changes nothing; it counts once whatever the number of tiles and slices."""
    for value, share in ((30.0, 0.0), (-30.0, 1.0), (6.0, None)):
        x = attention_case(5, 4, 32, 32, 64, 64, 150, None, True, False)
        x["sink"][:] = value
        plain = D.masked_attention(x["q"][110:], x["k"], x["v"], x["scale"], None, None, 110)
        want = expected(x, 110, 40)
        if share is not None:
            assert np.max(np.abs(want - share * plain)) < 1e-6
        top = np.max(np.abs(plain))
        for dt in (BF16, F32):
            close(over_keys(gpu, x, 110, 40, dt), want, dt, scale=top, bf16=2.0 ** -7)
        for n in (1, 3, 32):
            close(over_latents(gpu, x, 110, n), want[:n], BF16, scale=top, bf16=BF16_ATTENTION)
        gpu.release()


# ---- gated delta rule -----------------------------------------------------------------------------------
def padded_head(n):
    return 32 if n <= 32 else 64 if n <= 64 else 128 if n <= 128 else 256


def delta_case(seed, heads, kv, dim, vdim, T, kind):
    rng = np.random.default_rng(seed)
    q, k, v, z = (rounded(rng.standard_normal(s)) for s in ((T, kv, dim), (T, kv, dim), (T, heads, vdim), (T, heads, vdim)))
    b, a = 1.5 * rng.standard_normal((T, heads)), rng.standard_normal((T, heads))
    a_log, dt_bias = rng.standard_normal(heads) - 1, 0.5 * rng.standard_normal(heads) - 1
    if kind == "alike":      # keys that all but repeat, written with full strength and hardly any decay
        k = rounded(k[:1] + 0.05 * k)
        b, dt_bias = b + 6.0, dt_bias - 6.0
    elif kind == "forget":   # decays that underflow within a chunk
        a = a + 8.0
        a_log = a_log + 2.0
    elif kind == "keep":     # nothing is forgotten, few writes
        dt_bias, b = dt_bias - 12.0, b - 4.0
        b[0] = 5.0
    elif kind == "zeros":    # a unit vector of a zero vector is zero
        k[3::7] = 0
        q[2::5] = 0
    return dict(heads=heads, kv=kv, dim=dim, vdim=vdim, T=T, q=q, k=k, v=v, z=z, b=b, a=a, a_log=a_log, dt_bias=dt_bias,
                norm=1 + 0.3 * rng.standard_normal(vdim))


def delta_expected(x, eps):
    q, k = D.unit(x["q"]) * x["dim"] ** -0.5, D.unit(x["k"])
    f = lambda v: np.asarray(v, np.float32).astype(float)   # what the device is given
    beta, g = S.sigmoid(f(x["b"])), np.exp(-np.exp(f(x["a_log"])) * S.softplus(f(x["a"]) + f(x["dt_bias"])))
    group = x["heads"] // x["kv"]
    runs = [D.delta_rule(q[:, h // group], k[:, h // group], x["v"][:, h], g[:, h], beta[:, h]) for h in range(x["heads"])]
    o = np.stack([r[0] for r in runs], 1)
    return D.rms_norm(o, x["norm"], eps) * D.silu(x["z"]), np.stack([r[1] for r in runs]), o


def run_delta(G, x, dt, cuts, eps):
    H, kv, dk, dv = x["heads"], x["kv"], padded_head(x["dim"]), up32(x["vdim"])
    vec = [put(G, x["a_log"]), put(G, x["dt_bias"]), put(G, pad(x["norm"], dv))]
    d = G.B.DeltaParams(H, kv, dk, dv, x["dim"], x["vdim"], eps, *[v.ptr for v in vec])
    channels = 2 * kv * dk + H * dv
    ld = up64(channels)
    state, got, at = zeros(G, (H, dk, dv)), [], 0
    for n in cuts:
        s = slice(at, at + n)
        rows = np.zeros((n, ld))
        rows[:, :channels] = np.concatenate([pad(x["q"][s], dk).reshape(n, -1), pad(x["k"][s], dk).reshape(n, -1), pad(x["v"][s], dv).reshape(n, -1)], 1)
        qkv, gate, ba = put(G, rows, dt), put(G, pad(x["z"][s], dv), dt), put(G, np.concatenate([x["b"][s], x["a"][s]], 1))
        out = zeros(G, (n, H, dv), dt)
        if n == 1 and dt == BF16:
            call(G, "lcu_decode_delta_step", out, qkv, gate, ba, C.byref(d), state)
        else:
            scratch = G.dev_keep(np.full(G.L().lcu_delta_rule_scratch(C.byref(d), n) // 4, np.nan, np.float32))
            call(G, "lcu_delta_rule", out, H * dv, qkv, ld, gate, H * dv, ba, 2 * H, C.byref(d), state, scratch, dt, n)
        y = get(G, out, (n, H, dv), dt)
        assert (y[..., x["vdim"]:] == 0).all()
        got.append(y[..., :x["vdim"]])
        at += n
    return np.concatenate(got), get(G, state, (H, dk, dv))


DELTA_CUTS = [(200,), (1, 2, 61, 1, 64, 2, 65, 1, 3), (2,) * 6 + (128, 59, 1), (63, 1, 1, 1, 62, 2) + (1,) * 70]


@BOTH
@pytest.mark.parametrize("heads,kv,dim,vdim", [(2, 1, 24, 40), (6, 2, 64, 32), (3, 3, 70, 20), (4, 1, 128, 128), (2, 2, 200, 96), (8, 4, 32, 256), (1, 1, 256, 33)])
@pytest.mark.parametrize("kind", ["plain", "alike", "forget", "keep", "zeros"])
def test_delta_rule_in_portions(gpu, dt, heads, kv, dim, vdim, kind):
    x, eps = delta_case(heads * 10 + dim, heads, kv, dim, vdim, 200, kind), 1e-5
    want, last, o = delta_expected(x, eps)
    # the norm divides by the size of o: what fp32 loses against the largest o shows where o is small
    small = np.maximum(1.0, 0.03 * np.abs(o).max() / np.sqrt((o ** 2).mean(-1, keepdims=True) + eps))
    for cuts in DELTA_CUTS if kind == "plain" else DELTA_CUTS[1:3]:
        got, state = run_delta(gpu, x, dt, cuts, eps)
        top = np.max(np.abs(want))
        err = np.abs(got - want) / top / small
        assert err.max() < (1e-4 if dt == F32 else 2.0 ** -8), (cuts, err.max())
        close(state[:, :dim, :vdim], last, F32, f32=2e-5)
        assert (state[:, dim:] == 0).all() and (state[..., vdim:] == 0).all()
        gpu.release()


def test_delta_rule_remembers(gpu):
    """One write at the first token, read 3000 tokens later over hardly decaying state, in one call and token by token."""
    T, dim, vdim = 3000, 32, 32
    x = delta_case(1, 2, 1, dim, vdim, T, "keep")
    x["b"][1:] = -60.0       # nothing else is written
    x["q"][-1] = x["k"][0]
    want, last, o = delta_expected(x, 1e-5)
    assert np.abs(o[-1]).max() > 0.1
    for dt, cuts in ((F32, (T,)), (BF16, (T,)), (BF16, (1000, 1500) + (1,) * 500)):
        got, state = run_delta(gpu, x, dt, cuts, 1e-5)
        close(got[-1], want[-1], dt, f32=1e-4)
        close(state[:, :dim, :vdim], last, F32, f32=1e-4)
        gpu.release()


def test_unsupported_shapes_are_refused_before_any_launch(gpu):
    L, B = gpu.L(), gpu.B
    a = zeros(gpu, 8192).ptr
    wp = B.WindowParams(2, 2, 64, 64, 8, 0, 1.0, None, None, 64, 0, 0, 0, a)                     # nothing of the key is the head's own
    assert L.lcu_attention_windowed(a, 128, a, 128, a, a, 0, C.byref(wp), 0, 1, gpu.stream) == -2
    wp = B.WindowParams(2, 2, 64, 64, 8, 0, 1.0, None, None, 0, 0, 0, 5)                         # keys from behind the window's begin
    assert L.lcu_attention_windowed(a, 128, a, 128, a, a, 6, C.byref(wp), 0, 1, gpu.stream) == -2
    assert L.lcu_attention_windowed_decode(a, a, a, a, a, 8, C.byref(wp), a, gpu.stream) == -2   # no distance bias
    d = B.DeltaParams(3, 2, 32, 32, 32, 32, 1e-5, a, a, a)                                       # 3 heads on 2
    assert L.lcu_delta_rule(a, 96, a, 256, a, 96, a, 6, C.byref(d), a, a, 0, 1, gpu.stream) == -2
    d = B.DeltaParams(2, 2, 48, 32, 48, 32, 1e-5, a, a, a)                                       # no such padded head
    assert L.lcu_decode_delta_step(a, a, a, a, C.byref(d), a, gpu.stream) == -2
    p = B.LatentParams(2, 32, 32, 34, 32, 64, 64, 8, 1.0)                                        # more rotated dimensions than there are
    assert L.lcu_latent_queries(a, a, 128, a, C.byref(p), None, 1, gpu.stream) == -2
    p = B.LatentParams(2, 32, 0, 0, 32, 600, 640, 8, 1.0)
    assert not L.lcu_latent_attention_fits(C.byref(p))
    assert L.lcu_latent_attention(a, 64, a, a, 64, a, None, a, 8, a, None, None, 0, C.byref(p), a, 1, gpu.stream) == -2
    assert L.lcu_linear_tail(a, 64, a, 2, 64, a, a, 0, 1, 64, 64, gpu.stream) == -2              # no column is left for the tail
    gpu.release()
