"""Whole Logivik models (latent attention, the gated delta rule, dense feed-forwards) on the GPU against the plain
restatement: every layer type and order, whole prompts, portions, decoding, contexts used again, generation through the
library and the program, replay.  fp32 has to agree closely (any wrong key or lost state shows); bfloat16 within a few times what its
rounding does to the plain restatement."""
import json
import os
import subprocess

import numpy as np
import pytest

import lcu
import plain_latent_delta as D
import plain_stack as S
from layered_helpers import errors, feed

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BIN = os.path.join(ROOT, "llama.cu_amd", "bin")
P = lcu.package()


def mlp(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def far(heads, dim, rot, vdim, rank, scale, rotation, ff):
    """latent attention over everything before, with a rotated part"""
    return {"type": "latent_attention", "mlp": mlp(ff), "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
                                                                  "scale": scale, "rot": dict(rotation, dims=rot)}}


def near(heads, dim, vdim, rank, q_rank, size, scale, ff):
    """latent attention with a window"""
    return {"type": "latent_attention_2", "mlp": mlp(ff), "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank,
                                                                    "scale": scale, "mask": {"size": size}}}


def delta(heads, kv, dim, vdim, conv, ff):
    return {"type": "delta", "mlp": mlp(ff), "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def config(vocab, width, scale, eps, layers):
    return {"architecture": "Logivik", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


YARN = {"base": 5000.0, "scaling": {"factor": 4.0, "original": 100, "fast": 8.0, "slow": 1.5}}
LONG = {"base": 1e6, "scaling": {"factor": 40.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
PLAIN = {"base": 300.0}

MODELS = {
    # every size its own, none a multiple of a tile; layers differ from one another, some without a feed-forward
    "ragged": config(301, 180, 3.7, 1e-4, [
        delta(6, 2, 24, 40, 3, 50),
        near(5, 44, 20, 70, 37, 29, 0.31, 130),
        far(3, 20, 12, 33, 45, 0.4, YARN, 77),
        delta(3, 3, 70, 20, 1, 0),
        near(2, 33, 65, 20, 90, 64, 0.2, 0),
        far(7, 36, 6, 70, 100, 0.25, PLAIN, 0),
        delta(4, 1, 40, 33, 6, 31)]),
    # one head everywhere, latents of a few numbers, a window of one token
    "narrow": config(77, 64, 1.0, 1e-5, [
        far(1, 8, 2, 8, 6, 0.9, PLAIN, 16),
        near(1, 8, 8, 4, 5, 1, 1.0, 8),
        delta(1, 1, 8, 4, 2, 16)]),
    # the state alone
    "delta": config(128, 96, 9.0, 1e-6, [delta(8, 4, 128, 64, 4, 0), delta(2, 2, 32, 96, 2, 60), delta(4, 4, 16, 128, 5, 0)]),
    # attention alone, more than sixteen heads, windows at the tiles' edges
    "attention": config(512, 640, 20.0, 1e-6, [
        far(20, 64, 32, 64, 192, 0.15, LONG, 300),
        near(12, 64, 64, 128, 160, 65, 0.2, 500),
        near(17, 32, 32, 64, 64, 63, 0.25, 0)]),
    # a latent and heads too large for the kernels of few tokens: those run as prompts do
    "large": config(90, 128, 11.0, 1e-5, [
        near(2, 128, 128, 600, 70, 40, 0.12, 64),
        far(3, 160, 64, 200, 520, 0.1, YARN, 0),
        delta(2, 1, 256, 256, 4, 40)]),
}


@pytest.fixture(scope="module", params=sorted(MODELS))
def case(request, tmp_path_factory):
    P.binding.init(0)
    cfg = MODELS[request.param]
    W = D.random_weights(cfg, 11)
    path = str(tmp_path_factory.mktemp("logivik") / request.param)
    S.write_model(path, cfg, W)
    tokens = np.random.default_rng(5).integers(0, cfg["vocab"], 230)
    layers = []
    logits = D.forward(cfg, W, tokens, layers)
    rounding = errors(D.forward(cfg, W, tokens, rnd=D.to_bf16), logits)
    return dict(cfg=cfg, W=W, path=path, tokens=tokens, logits=logits, layers=layers, rounding=rounding)


def held(got, want, dt, rounding):
    """rounding: the errors that bfloat16 alone causes, over some positions."""
    e = errors(got, want)
    worst, middle = (1e-4, 2e-5) if dt == "f32" else (3 * rounding.max(), 2 * np.median(rounding))
    assert e.max() < worst and (len(e) < 20 or np.median(e) < middle), (e.argmax(), e.max(), np.median(e), rounding.max(), np.median(rounding))


CUTS = {"whole": (230,), "tokens": (1,) * 230, "twos": (2,) * 40 + (150,), "decode": (100,) + (1,) * 130,
        "portions": (3, 37, 64, 1, 2, 1, 1, 22, 2, 65, 1, 16, 15), "few": (32, 33, 31, 34, 30, 35, 35)}


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_prompts_portions_and_decoding(case, dt):
    m = P.Model(path=case["path"], dtype=dt)
    c = P.Context(m, context_len=240)
    assert (m.n_vocab, m.dim) == (case["cfg"]["vocab"], case["cfg"]["width"]) and m.max_context >= 32768
    for cuts in CUTS.values():
        held(feed(c, case["tokens"], cuts), case["logits"], dt, case["rounding"])
        assert c.tokens_left() == 10
        c.clear_tokens()
    # the residual stream after every layer
    c.record_residual()
    c.forward(case["tokens"][:50], [49])
    for l, want in enumerate(case["layers"]):
        e = np.max(np.abs(c.residual(l, 50) - want[:50])) / np.max(np.abs(want[:50]))
        assert e < (1e-5 if dt == "f32" else 0.08), (l, e)
    c.close()
    m.close()


def test_wanted_places_and_next_token(case):
    m = P.Model(path=case["path"], dtype="f32")
    c = P.Context(m, context_len=240)
    want = [7, 0, 229, 7, 100]
    tok, lg = c.forward(case["tokens"], want)
    held(lg, case["logits"][want], "f32", None)
    assert tok == case["logits"][229].argmax()
    c.clear_tokens()
    assert c.next_token(case["tokens"]) == tok
    c.close()
    m.close()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_contexts_do_not_meet(case, dt):
    """Two contexts of one model in turn, of different lengths, one of them used again after another sequence: as alone."""
    m = P.Model(path=case["path"], dtype=dt)
    a, b = P.Context(m, context_len=240), P.Context(m, context_len=64)
    t, other = case["tokens"], np.random.default_rng(9).integers(0, case["cfg"]["vocab"], 60)
    want = D.forward(case["cfg"], case["W"], other)
    rounding = np.concatenate([case["rounding"], errors(D.forward(case["cfg"], case["W"], other, rnd=D.to_bf16), want)])
    got_a, got_b = [a.forward(t[:40], range(40))[1]], [b.forward(other[:20], range(20))[1]]
    for k in range(40):
        got_a.append(a.forward(t[40 + k:41 + k], [0])[1])
        got_b.append(b.forward(other[20 + k:21 + k], [0])[1])
    held(np.concatenate(got_a), case["logits"][:80], dt, case["rounding"])
    held(np.concatenate(got_b), want, dt, rounding)
    a.clear_tokens()
    first = feed(a, other, (20,) + (1,) * 40)
    held(first, want, dt, rounding)
    a.clear_tokens()
    assert (feed(a, other, (20,) + (1,) * 40) == first).all()
    for x in (a, b, m):
        x.close()


def test_greedy_generation(case, tmp_path):
    """next_token step by step, and the generation program: the tokens of the plain restatement."""
    prompt = [int(t) for t in case["tokens"][:17]]
    seq, margin = list(prompt), []
    for _ in range(24):
        lg = D.forward(case["cfg"], case["W"], np.array(seq))[-1]
        top = np.sort(lg)[-2:]
        margin.append((top[1] - top[0]) / lg.std())
        seq.append(int(lg.argmax()))
    want = seq[17:]

    def generate(ctx):
        got, t = [], prompt
        for _ in range(24):
            got.append(ctx.next_token(t))
            t = [got[-1]]
        return got
    m = P.Model(path=case["path"], dtype="f32")
    c = P.Context(m, context_len=64)
    got = generate(c)
    close_call = next((i for i, x in enumerate(margin) if x < 1e-3), 24)
    assert close_call >= 4 and got[:close_call] == want[:close_call]
    c.close()
    m.close()
    # bfloat16 through the program: the choices agree up to the first close one
    p = subprocess.run([os.path.join(BIN, "llama_cu"), "1", case["path"], " ".join(map(str, prompt)), "24", "64"], cwd=str(tmp_path),
                       capture_output=True, text=True, timeout=120)
    assert p.returncode == 0, p.stderr
    ids = [int(x) for x in p.stdout.split("\ntokens: ")[0].splitlines()[-1].split()]
    clear = next((i for i, x in enumerate(margin) if x < 0.3), 24)
    assert len(ids) == 24 and ids[:clear] == want[:clear]
    m = P.Model(path=case["path"])
    c = P.Context(m, context_len=64, temperature=0.8)
    assert generate(c) == ids
    c.close()
    m.close()


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_replay_program(case, tmp_path, dtype):
    """bin/trace_run: portions of sequences that come one after the other, a finished one's context used again."""
    t = [int(x) for x in case["tokens"]]
    steps = [("a", t[:50], [0, 49]), ("a", t[50:51], [0]), ("a", t[51:90], []), ("a", t[90:92], [1, 0]), ("b", t[:3], [2]), ("b", t[3:70], [66, 5]),
             ("b", t[70:71], [0]), ("b", t[71:72], [0]), ("b", t[72:73], [0])]
    ends = {3: ["a"], 8: ["b"]}
    lines = [json.dumps({"step": n, "entries": [{"id": i, "tokens": x, "want": w}], "end": ends.get(n, [])}) for n, (i, x, w) in enumerate(steps)]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", case["path"], "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "100"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=120)
    assert p.returncode == 0, p.stderr
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == ["done %d" % n for n in range(len(steps))]
    at, got, want = {"a": 0, "b": 0}, [], []
    for n, (i, x, w) in enumerate(steps):
        if w:
            got.append(np.fromfile(str(tmp_path / ("%d.f32" % n)), "<f4").reshape(len(w), -1))
            want.append(case["logits"][[at[i] + k for k in w]])
        at[i] += len(x)
    held(np.concatenate(got), np.concatenate(want), "f32" if dtype == "float32" else "bf16", case["rounding"])


def test_sampling_is_reproducible(case):
    m = P.Model(path=case["path"])
    c = P.Context(m, context_len=64, temperature=1.0)

    def draw(seed):
        c.clear_tokens()
        c.sample_with_seed(seed)
        out, t = [], case["tokens"][:9]
        for _ in range(30):
            out.append(c.next_token(t))
            t = [out[-1]]
        return out
    first = draw(3)
    assert first == draw(3) and first != draw(4)
    assert all(0 <= t < m.n_vocab for t in first)
    c.close()
    m.close()


def test_incomplete_weight_files_are_refused(tmp_path):
    P.binding.init(0)
    cfg = MODELS["ragged"]
    W = D.random_weights(cfg, 1)
    for n, (name, change) in enumerate([("l0.mix.A_log", None), ("l0.mix.k.conv", lambda a: a[:, :-1]), ("l1.mix.dq.norm", None), ("l1.mix.uk", lambda a: a.T),
                                        ("l2.mix.sink", None), ("l2.mix.dkv", lambda a: a[:-1]), ("final.norm", None), ("l2.mlp.down", lambda a: a.T)]):
        broken = dict(W)
        if change is None:
            del broken[name]
        else:
            broken[name] = change(broken[name])
        S.write_model(str(tmp_path / str(n)), cfg, broken)
        with pytest.raises(P.LcuError):
            P.Model(path=str(tmp_path / str(n)))
    m = P.Model(config=cfg, seed=3)                # weights of its own
    c = P.Context(m, context_len=80)
    lg = np.concatenate([c.forward(range(70), [69])[1]] + [c.forward([5], [0])[1] for _ in range(5)])
    assert np.isfinite(lg).all() and lg.std() > 0.1
    with pytest.raises(P.LcuError):
        P.BatchContext(m, 2)
    with pytest.raises(P.LcuError):
        c.forward([1] * 6)
    c.close()
    m.close()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_prompt_longer_than_a_pass_and_long_decoding(tmp_path, dt):
    """2300 tokens in one call run in more than one pass; 700 tokens decoded one by one pass every edge of the windows, over
    scores that pick single keys."""
    P.binding.init(0)
    cfg = config(97, 96, 6.0, 1e-5, [delta(2, 1, 32, 32, 4, 0), near(2, 24, 32, 40, 48, 70, 0.8, 32), far(2, 32, 16, 32, 48, 0.7, LONG, 0),
                                     near(2, 32, 32, 32, 32, 600, 0.9, 0)])
    W = D.random_weights(cfg, 2)
    S.write_model(str(tmp_path / "m"), cfg, W)
    t = np.random.default_rng(0).integers(0, 97, 2300)
    want = D.forward(cfg, W, t)
    rounding = errors(D.forward(cfg, W, t[:1000], rnd=D.to_bf16), want[:1000])
    m = P.Model(path=str(tmp_path / "m"), dtype=dt)
    c = P.Context(m, context_len=2400)
    places = list(range(0, 2300, 7)) + [2047, 2048, 2299]
    held(c.forward(t, places)[1], want[places], dt, rounding)
    c.clear_tokens()
    c.forward(t[:300])
    held(np.concatenate([c.forward(t[k:k + 1], [0])[1] for k in range(300, 1000)]), want[300:1000], dt, rounding)
    c.close()
    m.close()
