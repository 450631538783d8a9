"""Plain restatement of the decoder with latent attention and the gated delta rule (Logivik) in numpy float64,
one function per mechanism.

The oracle of the tests: loops over tokens, no cache, no shared code with the product.  A model is a config (the
dict of config.json) and a dict of weight arrays under the names of the weight file.  `rnd`, where a function has it, is
applied to every activation that a model in a narrower type would store in it: what it does to the logits is what that
type's rounding alone can do.
"""
import numpy as np

from plain_stack import F, bf16_bits, bf16_values, sigmoid, softplus

UNIT_EPS = 1e-6


def exact(x):
    return x


def to_bf16(x):
    return bf16_values(bf16_bits(x)).reshape(np.shape(x)).astype(F)


def rms_norm(x, w, eps):
    x = np.asarray(x, F)
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def silu(z):
    return z * sigmoid(z)


# ---- rotation ---------------------------------------------------------------------------------------
def stretched_frequencies(dims, base, scaling):
    """(frequency of each pair, factor on cos and sin).  scaling None: base^(-2i/dims) and 1.  Otherwise pairs that
    turn often within `original` positions keep their frequency, slow ones are divided by `factor`, with a linear
    ramp between."""
    i = np.arange(dims // 2)
    f = float(base) ** (-2.0 * i / dims)
    if scaling is None:
        return f, 1.0
    turns = lambda t: dims * np.log(scaling["original"] / (2 * np.pi * t)) / (2 * np.log(base))
    lo = max(np.floor(turns(scaling["fast"])), 0)
    hi = min(np.ceil(turns(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(scaling["factor"]) + 1.0


def rotate_pairs(x, rot, first=0):
    """x [T, ..., dims] at positions first .. first + T - 1; neighbours (2i, 2i + 1) are a pair."""
    f, gain = stretched_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    out = np.array(x, F)
    for t in range(x.shape[0]):
        c, s = np.cos((first + t) * f) * gain, np.sin((first + t) * f) * gain
        u, v = x[t, ..., 0:rot["dims"]:2], x[t, ..., 1:rot["dims"]:2]
        out[t, ..., 0:rot["dims"]:2] = u * c - v * s
        out[t, ..., 1:rot["dims"]:2] = v * c + u * s
    return out


# ---- latent attention -------------------------------------------------------------------------------
def masked_attention(q, k, v, scale, size=None, sink=None, first=0):
    """q [n, H, D] at positions first .., k [T, H, D], v [T, H, E] -> [n, H, E].  size: keys 0 <= i - j < size (None: all
    before).  sink [H]: a term exp(sink) in the denominator only."""
    n, H, _ = q.shape
    out = np.zeros((n, H, v.shape[2]))
    for i in range(first, first + n):
        lo = 0 if size is None else max(0, i - size + 1)
        for h in range(H):
            s = (k[lo:i + 1, h] @ q[i - first, h]) * scale
            top = s.max() if sink is None else max(s.max(), sink[h])
            e = np.exp(s - top)
            total = e.sum() + (0.0 if sink is None else np.exp(sink[h] - top))
            out[i - first, h] = (e / total) @ v[lo:i + 1, h]
    return out


def latent_mixer(h, W, p, m, eps, rnd=exact):
    """Keys and values out of a normed latent; a rotated part shared by the heads, a sink, a gate on the output, a
    latent for the queries and a window where the layer has them."""
    T, H, D, E, R = h.shape[0], m["heads"], m["dim"], m["vdim"], m["kv_rank"]
    rd = m.get("rot_dim", 0)
    if "q_rank" in m:
        q = rnd(rnd(rms_norm(rnd(h @ W[p + "dq"].T), W[p + "dq.norm"], eps)) @ W[p + "uq"].T)
    else:
        q = rnd(h @ W[p + "q"].T)
    q = q.reshape(T, H, D + rd)
    down = rnd(h @ W[p + "dkv"].T)
    c = rnd(rms_norm(down[:, :R], W[p + "dkv.norm"], eps))
    k = rnd(c @ W[p + "uk"].T).reshape(T, H, D)
    v = rnd(c @ W[p + "uv"].T).reshape(T, H, E)
    if rd:
        q = np.concatenate([q[..., :D], rnd(rotate_pairs(q[..., D:], m["rot"]))], -1)
        shared = rnd(rotate_pairs(down[:, None, R:], m["rot"]))
        k = np.concatenate([k, np.repeat(shared, H, 1)], -1)
    o = masked_attention(q, k, v, m["scale"], m["mask"]["size"] if "mask" in m else None, W.get(p + "sink"))
    o = o.reshape(T, H * E)
    if p + "g" in W:
        o = o * sigmoid(rnd(h @ W[p + "g"].T))
    return rnd(o) @ W[p + "o"].T


# ---- gated delta rule -------------------------------------------------------------------------------
def conv_silu(z, w):
    """Causal convolution per channel of z [T, C]; the last column of w [C, taps] meets the current row."""
    T, taps = z.shape[0], w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, z.shape[1])), z])
    return silu(sum(w[:, k] * pad[k:k + T] for k in range(taps)))


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + UNIT_EPS)


def delta_rule(q, k, v, g, beta, S=None):
    """One head: q, k [T, D], v [T, E], g, beta [T] -> ([T, E], last state [D, E])."""
    S = np.zeros((k.shape[1], v.shape[1])) if S is None else S
    out = np.empty(v.shape)
    for t in range(len(g)):
        S = g[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out, S


def delta_mixer(h, W, p, m, eps, rnd=exact):
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    branch = lambda n, heads, d: rnd(conv_silu(rnd(h @ W[p + n].T), W[p + n + ".conv"])).reshape(T, heads, d)
    q, k, v = unit(branch("q", G, D)) * D ** -0.5, unit(branch("k", G, D)), branch("v", H, E)
    beta = sigmoid(h @ W[p + "b"].T)
    g = np.exp(-np.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    o = np.stack([delta_rule(q[:, i // (H // G)], k[:, i // (H // G)], v[:, i], g[:, i], beta[:, i])[0] for i in range(H)], 1)
    o = rms_norm(o, W[p + "norm"], eps) * silu(rnd(h @ W[p + "g"].T)).reshape(T, H, E)
    return rnd(o.reshape(T, H * E)) @ W[p + "o"].T


def gated_mlp(h, W, p, rnd=exact):
    return rnd(silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


# ---- the model --------------------------------------------------------------------------------------
MIXERS = {"delta": delta_mixer, "latent_attention": latent_mixer, "latent_attention_2": latent_mixer}


def forward(cfg, W, tokens, layers=None, rnd=exact):
    """Logits [T, vocab]; `layers`, a list, receives the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    norm = lambda x, name: rms_norm(x, 1.0 + W[name], eps)
    x = W["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    for l, spec in enumerate(cfg["layers"]):
        p = "l%d." % l
        x = x + norm(MIXERS[spec["type"]](rnd(x), W, p + "mix.", spec["mixer"], eps, rnd), p + "norm1")
        if spec.get("mlp"):
            x = x + norm(gated_mlp(rnd(x), W, p + "mlp.", rnd), p + "norm2")
        if layers is not None:
            layers.append(x)
    return rnd(norm(x, "final.norm")) @ W["head"].T


def tensor_shapes(cfg):
    """name -> shape of every tensor of a model with this config."""
    w, n = cfg["width"], cfg["vocab"]
    s = {"embed": (n, w), "final.norm": (w,), "head": (n, w)}
    for l, spec in enumerate(cfg["layers"]):
        p = "l%d." % l
        m, q = spec["mixer"], p + "mix."
        s[p + "norm1"] = (w,)
        H, D, E = m["heads"], m["dim"], m["vdim"]
        if spec["type"] == "delta":
            G, taps = m["kv_heads"], m["conv"]
            for name, rows in (("q", G * D), ("k", G * D), ("v", H * E)):
                s[q + name], s[q + name + ".conv"] = (rows, w), (rows, taps)
            s.update({q + "b": (H, w), q + "a": (H, w), q + "A_log": (H,), q + "dt_bias": (H,), q + "norm": (E,), q + "g": (H * E, w)})
        else:
            R, rd = m["kv_rank"], m.get("rot_dim", 0)
            if spec["type"] == "latent_attention":
                s.update({q + "q": (H * (D + rd), w), q + "sink": (H,), q + "g": (H * E, w)})
            else:
                s.update({q + "dq": (m["q_rank"], w), q + "dq.norm": (m["q_rank"],), q + "uq": (H * D, m["q_rank"])})
            s.update({q + "dkv": (R + rd, w), q + "dkv.norm": (R,), q + "uk": (H * D, R), q + "uv": (H * E, R)})
        s[q + "o"] = (w, H * E)
        if spec.get("mlp"):
            ff = spec["mlp"]["ff"]
            s.update({p + "norm2": (w,), p + "mlp.gate": (ff, w), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    return s


def random_weights(cfg, seed, gain=1.0):
    """Weights of the config, every value representable in bfloat16."""
    rng = np.random.default_rng(seed)
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        a = rng.standard_normal(shape)
        if leaf in ("norm1", "norm2") or name == "final.norm":
            a = 0.2 * a                      # stored around zero
        elif leaf == "norm":
            a = 1.0 + 0.2 * a
        elif leaf == "A_log":
            a = -1.0 + a
        elif leaf == "dt_bias":
            a = -1.0 + 0.5 * a
        elif leaf == "sink":
            a = 0.5 + a
        elif leaf == "conv":
            a = a / np.sqrt(shape[-1])
        elif leaf == "embed":
            a = a / cfg["embedding"]["scale"]
        else:
            a = a * gain / np.sqrt(shape[-1])
        W[name] = bf16_values(bf16_bits(a)).reshape(shape).astype(F)
    return W
