"""Plain restatement of the layered decoder (Rirulix) in numpy float64, one function per mechanism.

The oracle of the tests: slow loops over tokens, no cache, no shared code with the product.  A model
is a config (the dict of config.json) and a dict of weight arrays under the names of the weight file.
"""
import numpy as np

F = np.float64


def sigmoid(z):
    z = np.asarray(z, dtype=F)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def softplus(z):
    return np.logaddexp(0.0, np.asarray(z, dtype=F))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def group_rms_norm(x, w, groups, eps):
    """Equal consecutive parts of the last axis, each over its own root mean square; then times w."""
    parts = np.asarray(x, F).reshape(x.shape[:-1] + (groups, x.shape[-1] // groups))
    parts = parts / np.sqrt((parts ** 2).mean(-1, keepdims=True) + eps)
    return parts.reshape(x.shape) * w


def causal_conv(z, taps_w, bias):
    """Per-channel causal convolution of z [T, C]; column taps-1 of taps_w [C, taps] meets the current row."""
    T, C = z.shape
    taps = taps_w.shape[1]
    out = np.empty((T, C))
    for t in range(T):
        acc = np.array(bias, dtype=F)
        for k in range(taps):
            s = t - (taps - 1) + k
            if s >= 0:
                acc = acc + taps_w[:, k] * z[s]
        out[t] = acc
    return out


def block_gate(u, w, b):
    """sigmoid of a block-diagonal product: part p of u goes through square matrix w[p]."""
    parts = np.split(u, w.shape[0], axis=-1)
    return sigmoid(np.concatenate([p @ w[i].T + b[i] for i, p in enumerate(parts)], axis=-1))


def gated_linear_recurrence(u, r, i, lam):
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t with log a_t = -8 r_t softplus(lam), S before the start 0."""
    log_a = -8.0 * r * softplus(lam)
    a = np.exp(log_a)
    drive = np.sqrt(-np.expm1(2.0 * log_a)) * i * u
    S = np.zeros(u.shape[1])
    out = np.empty(u.shape)
    for t in range(u.shape[0]):
        S = a[t] * S + drive[t]
        out[t] = S
    return out


def rglru_mixer(h, W, p, cfg):
    y = gelu_tanh(h @ W[p + "y"].T + W[p + "y.b"])
    u = causal_conv(h @ W[p + "x"].T + W[p + "x.b"], W[p + "conv"], W[p + "conv.b"])
    r = block_gate(u, W[p + "ra"], W[p + "ra.b"])
    i = block_gate(u, W[p + "ri"], W[p + "ri.b"])
    return (gated_linear_recurrence(u, r, i, W[p + "lam"]) * y) @ W[p + "o"].T


def visible(i, j, size, keep_first):
    return j <= i and (i - j < size or j < keep_first)


def windowed_attention(q, k, v, scale, r1, r2, size, keep_first):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]; a head's score loses r1 ln(1 + r2 (i - j))."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        js = np.array([j for j in range(i + 1) if visible(i, j, size, keep_first)])
        for h in range(H):
            g = h // (H // G)
            s = (k[js, g] @ q[i, h]) * scale - r1[h] * np.log1p(r2[h] * (i - js))
            s = np.exp(s - s.max())
            out[i, h] = (s / s.sum()) @ v[js, g]
    return out


def mix_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def attention_mixer(h, W, p, cfg, v_first):
    """Returns the output and this layer's values as projected (before any mixing)."""
    T, H, G, D, E = h.shape[0], cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = (h @ W[p + "q"].T + W[p + "q.b"]).reshape(T, H, D)
    k = (h @ W[p + "k"].T + W[p + "k.b"]).reshape(T, G, D)
    own = (h @ W[p + "v"].T + W[p + "v.b"]).reshape(T, G, E)
    v = own
    if cfg.get("v_mix") and v_first is not None:
        v = mix_values(own, v_first, W[p + "vmix"])
    o = windowed_attention(q, k, v, cfg["scale"], W[p + "r1"], W[p + "r2"], cfg["mask"]["size"], cfg["mask"]["keep_first"])
    return o.reshape(T, H * E) @ W[p + "o"].T + W[p + "o.b"], own


def expert(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def route(z, top):
    """Indices of the `top` largest scores of one token (ties: the smaller index) and the scores."""
    s = sigmoid(z)
    order = sorted(range(len(s)), key=lambda e: (-s[e], e))[:top]
    return order, s[order]


def experts_mlp(h, W, p, cfg):
    limit = cfg["expert"]["limit"]
    out = np.zeros_like(h)
    z = h @ W[p + "router"].T
    for t in range(h.shape[0]):
        for e, w in zip(*route(z[t], cfg["router"]["top"])):
            n = "%se%d." % (p, e)
            out[t] += expert(w * h[t], W[n + "gate"], W[n + "up"], W[n + "down"], limit)
    if cfg.get("shared"):
        n = p + "shared."
        gate = sigmoid(h @ W[n + "sg"].T)
        out = out + gate * expert(h, W[n + "gate"], W[n + "up"], W[n + "down"], cfg["shared"]["limit"])
    return out


def forward(cfg, W, tokens, layers=None):
    """Logits [T, vocab]; `layers`, a list, receives the residual stream after every layer."""
    groups, eps = cfg["norm"]["groups"], cfg["norm"]["eps"]

    def norm(x, name):
        return group_rms_norm(x, W[name], groups, eps)

    tokens = np.asarray(tokens)
    x = norm(W["embed"][tokens] + W["pos"][:len(tokens)], "embed.norm")
    v_first = None
    for l, spec in enumerate(cfg["layers"]):
        p = "l%d." % l
        h = norm(x, p + "norm1")
        if spec["type"] == "rglru":
            m = rglru_mixer(h, W, p + "mix.", spec["mixer"])
        else:
            m, own = attention_mixer(h, W, p + "mix.", spec["mixer"], v_first)
            if spec["mixer"].get("v_mix") and v_first is None:
                v_first = own
        x = x + norm(m, p + "norm1b")
        if spec.get("mlp"):
            x = x + norm(experts_mlp(norm(x, p + "norm2"), W, p + "mlp.", spec["mlp"]), p + "norm2b")
        if layers is not None:
            layers.append(x)
    return norm(x, "final.norm") @ W["head"].T


# ---- weight files ---------------------------------------------------------------------------------
def bf16_bits(a):
    """float array -> uint16 bfloat16 bits, nearest even."""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_values(bits):
    return (bits.astype(np.uint32) << 16).view(np.float32)


def tensor_shapes(cfg):
    """name -> shape of every tensor of a model with this config."""
    w, v = cfg["width"], cfg["vocab"]
    s = {"embed": (v, w), "pos": (cfg["max_positions"], w), "embed.norm": (w,), "final.norm": (w,), "head": (v, w)}
    for l, spec in enumerate(cfg["layers"]):
        p = "l%d." % l
        s[p + "norm1"] = s[p + "norm1b"] = (w,)
        m, q = spec["mixer"], p + "mix."
        if spec["type"] == "rglru":
            c, b = m["width"], m["blocks"]
            s.update({q + "y": (c, w), q + "y.b": (c,), q + "x": (c, w), q + "x.b": (c,), q + "conv": (c, m["conv"]),
                      q + "conv.b": (c,), q + "lam": (c,), q + "o": (w, c)})
            for g in ("ra", "ri"):
                s[q + g], s[q + g + ".b"] = (b, c // b, c // b), (b, c // b)
        else:
            H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            s.update({q + "q": (H * D, w), q + "q.b": (H * D,), q + "k": (G * D, w), q + "k.b": (G * D,),
                      q + "v": (G * E, w), q + "v.b": (G * E,), q + "r1": (H,), q + "r2": (H,), q + "o": (w, H * E),
                      q + "o.b": (w,)})
            if m.get("v_mix"):
                s[q + "vmix"] = ()
        f = spec.get("mlp")
        if f:
            s[p + "norm2"] = s[p + "norm2b"] = (w,)
            s[p + "mlp.router"] = (f["router"]["experts"], w)
            names = [("e%d" % e, f["expert"]["ff"]) for e in range(f["router"]["experts"])]
            if f.get("shared"):
                names.append(("shared", f["shared"]["ff"]))
                s[p + "mlp.shared.sg"] = (1, w)
            for n, ff in names:
                s.update({"%smlp.%s.gate" % (p, n): (ff, w), "%smlp.%s.up" % (p, n): (ff, w), "%smlp.%s.down" % (p, n): (w, ff)})
    return s


def random_weights(cfg, seed, gain=1.0):
    """Weights of the config, every value representable in bfloat16."""
    rng = np.random.default_rng(seed)
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        a = rng.standard_normal(shape)
        if "norm" in leaf:
            a = 1.0 + 0.2 * a
        elif leaf == "lam":
            a = -1.5 + a
        elif leaf in ("r1", "r2"):
            a = np.abs(a) * (0.5 if leaf == "r1" else 0.3) + 0.05
        elif leaf == "vmix":
            a = 0.3 + 0.1 * a
        elif leaf == "b":
            a = 0.2 * a
        elif leaf == "conv":
            a = a / np.sqrt(shape[-1])
        elif leaf in ("embed", "pos"):
            a = a * (1.0 if leaf == "embed" else 0.5)
        else:
            a = a * gain / np.sqrt(shape[-1])
        W[name] = bf16_values(bf16_bits(a)).reshape(shape).astype(F)
    return W


def write_model(path, cfg, W):
    """config.json and model.safetensors (bfloat16) of a model."""
    import json
    import os
    import struct
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, at = {}, [], 0
    for name, a in W.items():
        b = bf16_bits(a).tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    text = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for b in blobs:
            f.write(b)


def read_model(path):
    """(config, weights) of a model directory."""
    import json
    import os
    import struct
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    with open(os.path.join(path, "model.safetensors"), "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        head = json.loads(f.read(n))
        data = f.read()
    W = {}
    for name, t in head.items():
        if name == "__metadata__":
            continue
        lo, hi = t["data_offsets"]
        W[name] = bf16_values(np.frombuffer(data[lo:hi], np.uint16)).reshape(t["shape"]).astype(F)
    return cfg, W
