"""Host side of the layered decoders, without a GPU: the plain restatement against hand-worked cases, and the
refusals of the model reader (which come before any device call)."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import plain_stack as S

CFG = {"architecture": "Rirulix", "vocab": 50, "width": 24, "max_positions": 40, "norm": {"eps": 1e-5, "groups": 3},
       "layers": [{"type": "rglru", "mixer": {"width": 20, "blocks": 2, "conv": 2},
                   "mlp": {"kind": "moe", "router": {"experts": 3, "top": 2}, "expert": {"ff": 10, "limit": 2.0},
                           "shared": {"ff": 12, "limit": 1.0}}},
                  {"type": "attention", "mlp": None,
                   "mixer": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 10, "scale": 0.4, "v_mix": False,
                             "mask": {"size": 5, "keep_first": 2}}}]}


def test_visible_keys():
    seen = [[j for j in range(10) if S.visible(i, j, 3, 2)] for i in range(6)]
    assert seen == [[0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 3, 4, 5]]
    assert [j for j in range(10) if S.visible(9, j, 3, 2)] == [0, 1, 7, 8, 9]


def test_convolution_meets_the_current_token_with_the_last_tap():
    z = np.array([[1.0], [10.0], [100.0]])
    w = np.array([[5.0, 7.0]])
    assert S.causal_conv(z, w, np.array([0.5]))[:, 0].tolist() == [7.5, 75.5, 750.5]


def test_recurrence_by_hand():
    r, i, u = np.array([[0.5], [1.0]]), np.array([[1.0], [0.25]]), np.array([[2.0], [3.0]])
    lam = np.array([-1.0])
    a = [np.exp(-8 * x * np.log1p(np.exp(-1.0))) for x in (0.5, 1.0)]
    s1 = np.sqrt(1 - a[0] ** 2) * 2.0
    s2 = a[1] * s1 + np.sqrt(1 - a[1] ** 2) * 0.25 * 3.0
    assert np.allclose(S.gated_linear_recurrence(u, r, i, lam)[:, 0], [s1, s2], rtol=1e-12)


def test_norm_of_parts():
    x = np.array([3.0, 4.0, 0.3, 0.4])
    assert np.allclose(S.group_rms_norm(x, np.ones(4), 2, 0.0), np.tile([3, 4] / np.sqrt(12.5), 2))


def test_expert_clamps_one_side_of_the_gate_and_both_of_the_up_row():
    one = np.eye(1)
    for h, g, u in ((5.0, 2.0, 2.0), (-5.0, -5.0, -2.0)):
        got = S.expert(np.array([[h]]), one, one, one, 2.0)[0, 0]
        assert np.isclose(got, g * S.sigmoid(1.702 * g) * (u + 1))


def test_route_prefers_the_larger_then_the_earlier():
    order, scores = S.route(np.array([0.1, 2.0, 2.0, -1.0, 3.0]), 3)
    assert order == [4, 1, 2] and np.allclose(scores, S.sigmoid(np.array([3.0, 2.0, 2.0])))


def test_weight_file_round_trip(tmp_path):
    W = S.random_weights(CFG, 3)
    S.write_model(str(tmp_path / "m"), CFG, W)
    cfg, back = S.read_model(str(tmp_path / "m"))
    assert cfg == CFG and set(back) == set(W)
    assert all((back[n] == W[n]).all() and back[n].shape == np.shape(W[n]) for n in W)


def test_forward_in_prefixes_agrees():
    """The plain forward pass is causal: a prefix gives the same logits."""
    W = S.random_weights(CFG, 4)
    t = np.random.default_rng(0).integers(0, 50, 20)
    whole = S.forward(CFG, W, t)
    assert np.allclose(S.forward(CFG, W, t[:13]), whole[:13], rtol=1e-12, atol=1e-12)


# The reader of config.json fails before anything touches a device; each case runs the replay program, whose
# exit status and message tell.
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


BAD = [(("architecture",), "Nobody"), (("vocab",), KeyError), (("width",), 25), (("norm", "eps"), "small"), (("norm", "groups"), 0),
       (("layers",), []), (("layers", 0, "type"), "ssm"), (("layers", 0, "mixer", "blocks"), 3), (("layers", 0, "mixer", "conv"), 0),
       (("layers", 0, "mlp", "kind"), "dense"), (("layers", 0, "mlp", "router", "top"), 4), (("layers", 0, "mlp", "expert", "limit"), KeyError),
       (("layers", 1, "mixer", "kv_heads"), 3), (("layers", 1, "mixer", "scale"), KeyError), (("layers", 1, "mixer", "mask", "size"), 2.5),
       (("layers", 1, "mixer", "mask"), KeyError), (("layers", 1, "mixer", "dim"), 300), (("layers", 0, "mlp", "router", "experts"), 1000),
       (("width",), 30000)]


@pytest.mark.parametrize("path,value", BAD, ids=[".".join(map(str, p)) for p, _ in BAD])
def test_bad_configurations_are_refused(tmp_path, path, value):
    if not os.path.exists(BIN):
        pytest.skip("programs are not built")
    os.makedirs(tmp_path / "m")
    (tmp_path / "m" / "config.json").write_text(json.dumps(edited(path, value)))
    p = subprocess.run([BIN, "--model", str(tmp_path / "m"), "--dtype", "bfloat16", "--out", str(tmp_path), "--max-tokens", "8"],
                       input="", capture_output=True, text=True, timeout=60)
    assert p.returncode == 1 and "could not load the model" in p.stderr
    assert any(w in p.stderr for w in ("Invalid config.json", "Unknown architecture", "unsupported model shape")), p.stderr


def test_malformed_files_and_arguments(tmp_path):
    if not os.path.exists(BIN):
        pytest.skip("programs are not built")
    run = lambda *a: subprocess.run([BIN, *a], input="", capture_output=True, text=True, timeout=60)
    assert run("--model", "x").returncode == 2
    assert run("--model", str(tmp_path), "--dtype", "int8", "--out", str(tmp_path)).returncode == 2
    (tmp_path / "config.json").write_text('{"architecture": "Rirulix", "vocab": 5,, }')
    p = run("--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "4")
    assert p.returncode == 1 and "Invalid config.json" in p.stderr
    (tmp_path / "config.json").write_text(json.dumps(CFG))
    p = run("--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "4")
    assert p.returncode == 1 and "model.safetensors" in p.stderr
    (tmp_path / "model.safetensors").write_bytes((1 << 40).to_bytes(8, "little") + b"{}")
    p = run("--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "4")
    assert p.returncode == 1 and "header longer than the file" in p.stderr
