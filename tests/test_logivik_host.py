"""Host side of Logivik, without a GPU: the plain restatement against hand-worked cases, what a wrong reading of each mechanism
would do to its logits, and the refusals of the configuration reader (which come before any device call)."""
import copy
import json
import os
import subprocess

import numpy as np
import pytest

import plain_latent_delta as D
import plain_stack as S

CFG = {"architecture": "Logivik", "vocab": 40, "width": 24, "embedding": {"scale": 2.5}, "norm": {"eps": 1e-5},
       "layers": [{"type": "latent_attention", "mlp": {"kind": "dense", "ff": 20},
                   "mixer": {"heads": 2, "dim": 6, "rot_dim": 4, "vdim": 10, "kv_rank": 7, "scale": 0.8,
                             "rot": {"dims": 4, "base": 100.0, "scaling": {"factor": 3.0, "original": 30, "fast": 4.0, "slow": 1.0}}}},
                  {"type": "delta", "mlp": None, "mixer": {"heads": 4, "kv_heads": 2, "dim": 5, "vdim": 6, "conv": 3}},
                  {"type": "latent_attention_2", "mlp": {"kind": "dense", "ff": 9},
                   "mixer": {"heads": 3, "dim": 8, "vdim": 5, "kv_rank": 9, "q_rank": 11, "scale": 1.5, "mask": {"size": 6}}}]}


def test_frequencies_by_hand():
    f, gain = D.stretched_frequencies(4, 100.0, None)
    assert np.allclose(f, [1.0, 0.1]) and gain == 1.0
    # pair 0 turns 30 / 2 pi = 4.8 times within 30 positions (kept), pair 1 about half a turn (stretched)
    f, gain = D.stretched_frequencies(4, 100.0, CFG["layers"][0]["mixer"]["rot"]["scaling"])
    lo, hi = np.floor(4 * np.log(30 / (8 * np.pi)) / (2 * np.log(100))), np.ceil(4 * np.log(30 / (2 * np.pi)) / (2 * np.log(100)))
    assert (lo, hi) == (0, 1) and np.allclose(f, [1.0, 0.1 / 3]) and np.isclose(gain, 1 + 0.1 * np.log(3))


def test_rotation_by_hand():
    rot = {"dims": 2, "base": 10.0}
    x = np.array([[1.0, 0.0, 5.0], [1.0, 0.0, 5.0]])
    assert np.allclose(D.rotate_pairs(x, rot), [[1, 0, 5], [np.cos(1), np.sin(1), 5]])
    assert np.allclose(D.rotate_pairs(x, rot, 3)[0], [np.cos(3), np.sin(3), 5])
    # scores depend on the distance only
    q, k = np.random.default_rng(0).standard_normal((2, 1, 8))
    rot = {"dims": 8, "base": 50.0}
    s = [float(D.rotate_pairs(q, rot, p + 5)[0] @ D.rotate_pairs(k, rot, p)[0]) for p in (0, 9, 400)]
    assert np.allclose(s, s[0])


def test_window_and_sink_by_hand():
    k, v = np.zeros((5, 1, 2)), np.arange(5.0).reshape(5, 1, 1)
    out = D.masked_attention(k, k, v, 1.0, size=3)[:, 0, 0]
    assert np.allclose(out, [0, 0.5, 1, 2, 3])
    out = D.masked_attention(k, k, v, 1.0, sink=np.array([np.log(2.0)]))[:, 0, 0]
    assert np.allclose(out, [0, 1 / 4, 3 / 5, 6 / 6, 10 / 7])     # two more in the denominator
    assert np.allclose(D.masked_attention(k[3:], k, v, 1.0, size=3, first=3)[:, 0, 0], [2, 3])


def test_delta_rule_by_hand():
    e = np.eye(2)
    k, v = np.stack([e[0], e[1], e[0]]), np.array([[3.0], [5.0], [7.0]])
    g, beta = np.array([1.0, 0.5, 0.5]), np.array([1.0, 1.0, 0.25])
    out, S_ = D.delta_rule(np.ones((3, 2)), k, v, g, beta)
    # 3; then 1.5 + 5; then 0.75 + 0.25 (7 - 0.75) beside 2.5
    assert np.allclose(out[:, 0], [3, 6.5, 0.75 + 0.25 * 6.25 + 2.5]) and np.allclose(S_[:, 0], [0.75 + 0.25 * 6.25, 2.5])


def test_convolution_meets_the_current_token_with_the_last_tap():
    z = np.array([[1.0], [10.0], [100.0]])
    assert np.allclose(D.conv_silu(z, np.array([[5.0, 7.0]]))[:, 0], D.silu(np.array([7.0, 75.0, 750.0])))


def test_forward_in_prefixes_agrees():
    W = D.random_weights(CFG, 4)
    t = np.random.default_rng(0).integers(0, 40, 30)
    whole = D.forward(CFG, W, t)
    assert np.allclose(D.forward(CFG, W, t[:17]), whole[:17], rtol=1e-11, atol=1e-11)


def mixer(l, **change):
    return lambda c, W: c["layers"][l]["mixer"].update(change)


def rotation(**change):
    def f(c, W):
        c["layers"][0]["mixer"]["rot"].update(change)
    return f


def weight(name, f):
    def g(c, W):
        W[name] = f(W[name])
    return g


MISTAKES = {
    "window longer": mixer(2, mask={"size": 7}), "window shorter": mixer(2, mask={"size": 5}), "scale": mixer(0, scale=0.85),
    "no stretching": rotation(scaling=None), "factor": rotation(scaling={"factor": 3.5, "original": 30, "fast": 4.0, "slow": 1.0}),
    "other ramp": rotation(scaling={"factor": 3.0, "original": 300, "fast": 4.0, "slow": 1.0}),
    "no sink": weight("l0.mix.sink", lambda a: a - 60), "sinks exchanged": weight("l0.mix.sink", lambda a: a[::-1]),
    "gate flat": weight("l0.mix.g", lambda a: 0 * a), "taps reversed": weight("l1.mix.k.conv", lambda a: a[:, ::-1]),
    "no decay": weight("l1.mix.A_log", lambda a: a - 30), "step sizes": weight("l1.mix.b", lambda a: 0 * a),
    "decay of another head": weight("l1.mix.dt_bias", lambda a: np.roll(a, 1)), "queries' norm": weight("l2.mix.dq.norm", lambda a: 0 * a + 1),
    "latent's norm": weight("l2.mix.dkv.norm", lambda a: 0 * a + 1), "norm around zero": weight("l1.norm1", lambda a: a - 1),
    "head order": weight("l2.mix.uk", lambda a: a.reshape(3, 8, 9).transpose(1, 0, 2).reshape(24, 9)),
    "eps": lambda c, W: c["norm"].update(eps=1e-2), "embedding": lambda c, W: c["embedding"].update(scale=2.4)}


@pytest.mark.parametrize("name", sorted(MISTAKES))
def test_every_mistake_shows(name):
    """Each of them moves the logits by far more than the 1e-4 to which the models on the GPU are held in fp32."""
    W = D.random_weights(CFG, 4)
    t = np.random.default_rng(1).integers(0, 40, 30)
    right = D.forward(CFG, W, t)
    cfg, W = copy.deepcopy(CFG), dict(W)
    MISTAKES[name](cfg, W)
    d = D.forward(cfg, W, t) - right
    d -= d.mean(1, keepdims=True)
    assert np.sqrt((d ** 2).mean(1)).max() / right.std() > 5e-3


BIN = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "llama.cu_amd", "bin", "trace_run")


def edited(path, value):
    cfg = copy.deepcopy(CFG)
    at = cfg
    for key in path[:-1]:
        at = at[key]
    if value is KeyError:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return cfg


M0, M1, M2 = (("layers", n, "mixer") for n in range(3))
BAD = [(("vocab",), KeyError), (("width",), 0), (("embedding",), KeyError), (("embedding", "scale"), "big"), (("norm", "eps"), None), (("layers",), {}),
       (("layers", 0, "type"), "latent_attention_3"), (("layers", 0, "mlp", "kind"), "moe"), (("layers", 0, "mlp", "ff"), 0),
       (M0 + ("rot_dim",), KeyError), (M0 + ("rot",), KeyError), (M0 + ("rot", "dims"), 3), (M0 + ("rot", "dims"), 6), (M0 + ("rot", "base"), 1.0),
       (M0 + ("rot", "scaling", "slow"), KeyError), (M0 + ("rot", "scaling", "factor"), 0), (M0 + ("kv_rank",), -1), (M0 + ("scale",), KeyError),
       (M0 + ("dim",), 300), (M0 + ("vdim",), 257), (M1 + ("kv_heads",), 3), (M1 + ("conv",), 0), (M1 + ("dim",), 257), (M1 + ("vdim",), 300),
       (M2 + ("q_rank",), KeyError), (M2 + ("mask",), KeyError), (M2 + ("mask", "size"), 0), (("width",), 20000)]


@pytest.mark.parametrize("path,value", BAD, ids=[".".join(map(str, p)) for p, _ in BAD])
def test_bad_configurations_are_refused(tmp_path, path, value):
    if not os.path.exists(BIN):
        pytest.skip("programs are not built")
    (tmp_path / "config.json").write_text(json.dumps(edited(path, value)))
    p = subprocess.run([BIN, "--model", str(tmp_path), "--dtype", "bfloat16", "--out", str(tmp_path), "--max-tokens", "8"], input="",
                       capture_output=True, text=True, timeout=60)
    assert p.returncode == 1 and "could not load the model" in p.stderr
    assert any(w in p.stderr for w in ("Invalid config.json", "unsupported model shape")), p.stderr


def test_a_good_configuration_gets_as_far_as_its_weights(tmp_path):
    if not os.path.exists(BIN):
        pytest.skip("programs are not built")
    (tmp_path / "config.json").write_text(json.dumps(CFG))
    p = subprocess.run([BIN, "--model", str(tmp_path), "--dtype", "bfloat16", "--out", str(tmp_path), "--max-tokens", "8"], input="",
                       capture_output=True, text=True, timeout=60)
    assert p.returncode == 1 and "model.safetensors" in p.stderr


def test_weight_file_round_trip(tmp_path):
    W = D.random_weights(CFG, 3)
    S.write_model(str(tmp_path / "m"), CFG, W)
    cfg, back = S.read_model(str(tmp_path / "m"))
    assert cfg == CFG and set(back) == set(W) and all((back[n] == W[n]).all() for n in W)
