"""Whole layered decoders on the GPU against the plain restatement: every layer type and order, whole prompts,
portions, decoding, reuse of contexts, generation through the library, the generation program and the replay
program.  fp32 has to agree closely (any wrong key, state or route shows); bfloat16 within its rounding."""
import copy
import json
import os
import subprocess

import numpy as np
import pytest

import lcu
import plain_stack as S
from layered_helpers import errors, feed

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BIN = os.path.join(ROOT, "llama.cu_amd", "bin")
P = lcu.package()


def moe(experts, top, ff, limit, shared=None, shared_limit=1.0):
    m = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}
    if shared:
        m["shared"] = {"ff": shared, "limit": shared_limit}
    return m


def rec(width, blocks, conv, mlp):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": mlp}


def att(heads, kv, dim, vdim, size, keep, scale, v_mix, mlp):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": v_mix,
                      "mask": {"size": size, "keep_first": keep}}}


def config(vocab, width, groups, eps, layers, positions=400):
    return {"architecture": "Rirulix", "vocab": vocab, "width": width, "max_positions": positions, "norm": {"eps": eps, "groups": groups},
            "layers": layers}


MODELS = {
    # every size its own, none a multiple of a tile; layers differ from one another
    "ragged": config(301, 180, 3, 1e-4, [
        att(6, 2, 20, 33, 29, 5, 0.3, False, moe(7, 3, 50, 1.5, 70, 0.8)),
        rec(84, 3, 4, moe(5, 2, 24, 0.7)),
        att(4, 4, 44, 20, 64, 0, 0.1, True, None),
        rec(150, 5, 1, None),
        att(8, 4, 36, 20, 17, 11, 0.25, True, moe(3, 3, 40, 2.0, 30, 3.0)),
        rec(66, 1, 6, moe(9, 1, 33, 1.1, 100, 1.2))]),
    # one group, one head, recurrence last, feed-forward of one expert
    "narrow": config(77, 64, 1, 1e-5, [
        att(1, 1, 8, 8, 3, 1, 0.5, True, moe(1, 1, 16, 1.0, 8)),
        rec(32, 1, 2, moe(2, 1, 8, 1.0))]),
    # recurrence only, and only of it
    "recurrent": config(128, 96, 4, 1e-6, [rec(128, 4, 3, None), rec(64, 2, 4, moe(4, 2, 20, 1.0, 20)), rec(96, 2, 2, None)]),
    # attention only, groups of norm larger than a wavefront, values wider than keys
    "attention": config(512, 640, 2, 1e-5, [
        att(16, 1, 32, 64, 100, 40, 0.2, True, moe(20, 2, 70, 1.0, 90)),
        att(12, 1, 64, 64, 33, 2, 0.15, True, moe(12, 2, 64, 0.9, 64))]),
}


def weights(cfg, seed):
    W = S.random_weights(cfg, seed)
    for name in W:
        if name.endswith(".router"):
            W[name] = S.bf16_values(S.bf16_bits(3.0 * W[name])).astype(float)   # few close calls between experts
    return W


@pytest.fixture(scope="module", params=sorted(MODELS))
def case(request, tmp_path_factory):
    P.binding.init(0)
    name = request.param
    cfg = MODELS[name]
    W = weights(cfg, 11)
    path = str(tmp_path_factory.mktemp("layered") / name)
    S.write_model(path, cfg, W)
    tokens = np.random.default_rng(5).integers(0, cfg["vocab"], 230)
    layers = []
    logits = S.forward(cfg, W, tokens, layers)
    return dict(cfg=cfg, W=W, path=path, tokens=tokens, logits=logits, layers=layers)


def held(got, want, dt):
    """fp32: every position; bfloat16: nearly all (a close call between two experts may fall either way, and the
    tokens that attend to that one feel it)."""
    e = errors(got, want)
    if dt == "f32":
        assert e.max() < 1e-4, (e.argmax(), e.max())
    else:
        assert np.quantile(e, 0.92) < 0.05 and np.median(e) < 0.015, (np.quantile(e, 0.92), np.median(e))


CUTS = {"whole": (230,), "tokens": (1,) * 230, "twos": (2,) * 40 + (150,), "decode": (100,) + (1,) * 130,
        "portions": (3, 37, 64, 1, 2, 1, 1, 22, 2, 65, 1, 16, 15)}


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_prompts_portions_and_decoding(case, dt):
    m = P.Model(path=case["path"], dtype=dt)
    c = P.Context(m, context_len=240)
    assert (m.n_vocab, m.dim, m.max_context) == (case["cfg"]["vocab"], case["cfg"]["width"], 400)
    for name, cuts in CUTS.items():
        held(feed(c, case["tokens"], cuts), case["logits"], dt)
        assert c.tokens_left() == 10
        c.clear_tokens()
    # the residual stream after every layer
    c.record_residual()
    c.forward(case["tokens"][:50], [49])
    for l, want in enumerate(case["layers"]):
        e = np.max(np.abs(c.residual(l, 50) - want[:50])) / np.max(np.abs(want[:50]))
        assert e < (1e-5 if dt == "f32" else 0.05) or (dt == "bf16" and l > 0), (l, e)
    c.close()
    m.close()


def test_wanted_places_and_next_token(case):
    """Logits at scattered places, in the order asked for and twice, do not disturb the next token."""
    m = P.Model(path=case["path"], dtype="f32")
    c = P.Context(m, context_len=240)
    want = [7, 0, 229, 7, 100]
    tok, lg = c.forward(case["tokens"], want)
    held(lg, case["logits"][want], "f32")
    assert tok == case["logits"][229].argmax()
    c.clear_tokens()
    assert c.next_token(case["tokens"]) == tok
    probs = c.probs().astype(float)
    x = case["logits"][229] / 0.9
    assert np.max(np.abs(probs - np.exp(x - x.max()) / np.exp(x - x.max()).sum())) < 1e-3
    c.close()
    m.close()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_contexts_do_not_meet(case, dt):
    """Two contexts of one model in turn, one of them used again after another sequence: as each alone."""
    m = P.Model(path=case["path"], dtype=dt)
    a, b = P.Context(m, context_len=240), P.Context(m, context_len=64)
    t = case["tokens"]
    other = np.random.default_rng(9).integers(0, case["cfg"]["vocab"], 60)
    alone = P.Context(m, context_len=240)
    want_a, want_b = feed(alone, t[:80], (40,) + (1,) * 40), None
    alone.clear_tokens()
    want_b = feed(alone, other, (20,) + (1,) * 40)
    got_a, got_b = [a.forward(t[:40], range(40))[1]], [b.forward(other[:20], range(20))[1]]
    for k in range(40):
        got_a.append(a.forward(t[40 + k:41 + k], [0])[1])
        got_b.append(b.forward(other[20 + k:21 + k], [0])[1])
    assert (np.concatenate(got_a) == want_a).all() and (np.concatenate(got_b) == want_b).all()
    a.clear_tokens()
    assert (feed(a, other, (20,) + (1,) * 40) == want_b).all()
    for x in (a, b, alone):
        x.close()
    m.close()


def greedy(cfg, W, prompt, n):
    """Tokens by the plain restatement, and how clear each choice was."""
    seq, margin = list(prompt), []
    for _ in range(n):
        lg = S.forward(cfg, W, np.array(seq))[-1]
        top = np.sort(lg)[-2:]
        margin.append((top[1] - top[0]) / lg.std())
        seq.append(int(lg.argmax()))
    return seq[len(prompt):], margin


def test_greedy_generation(case, tmp_path):
    """next_token step by step, and the generation program: the tokens of the plain restatement."""
    prompt = [int(t) for t in case["tokens"][:17]]
    want, margin = greedy(case["cfg"], case["W"], prompt, 24)
    m = P.Model(path=case["path"], dtype="f32")
    c = P.Context(m, context_len=64)
    got, t = [], prompt
    for _ in range(24):
        got.append(c.next_token(t))
        t = [got[-1]]
    assert min(margin) > 1e-3 and got == want
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
    again, t = [], prompt
    for _ in range(24):
        again.append(c.next_token(t))
        t = [again[-1]]
    assert again == ids
    c.close()
    m.close()


def test_generation_program_refuses(case, tmp_path):
    run = lambda *a: subprocess.run([os.path.join(BIN, "llama_cu"), "1", *a], cwd=str(tmp_path), capture_output=True, text=True, timeout=120)
    p = run(case["path"], "once upon a time", "4", "64")
    assert p.returncode == 1 and "token ids" in p.stderr
    p = run(case["path"], " ".join(["1"] * 70), "4", "64")
    assert p.returncode == 1 and "exceeds the context" in p.stderr


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_replay_program(case, tmp_path, dtype):
    """bin/trace_run: portions of sequences that come one after the other, a finished one's context used again."""
    t = [int(x) for x in case["tokens"]]
    steps = [("a", t[:50], [0, 49]), ("a", t[50:51], [0]), ("a", t[51:90], []), ("a", t[90:92], [1, 0]), ("b", t[:3], [2]), ("b", t[3:70], [66, 5])]
    ends = {3: ["a"], 5: ["b"]}
    lines = [json.dumps({"step": n, "entries": [{"id": i, "tokens": x, "want": w}], "end": ends.get(n, [])}) for n, (i, x, w) in enumerate(steps)]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", case["path"], "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "100"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=120)
    assert p.returncode == 0, p.stderr
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == ["done %d" % n for n in range(6)]
    at = {"a": 0, "b": 0}
    got, want = [], []
    for n, (i, x, w) in enumerate(steps):
        path = tmp_path / ("%d.f32" % n)
        if w:
            got.append(np.fromfile(str(path), "<f4").reshape(len(w), -1))
            want.append(case["logits"][[at[i] + k for k in w]])
        else:
            assert not path.exists()
        at[i] += len(x)
    e = errors(np.concatenate(got), np.concatenate(want))
    assert e.max() < (1e-4 if dtype == "float32" else 0.1)
    bad = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", case["path"], "--dtype", dtype, "--out", str(tmp_path),
                          "--max-tokens", "8"], input=lines[0] + "\n", capture_output=True, text=True, timeout=120)
    assert bad.returncode == 1 and "do not fit" in bad.stderr


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
    c.greedy()
    c.close()
    m.close()


def test_limits_are_refused(case):
    m = P.Model(path=case["path"])
    with pytest.raises(P.LcuError):
        P.Context(m, context_len=401)              # more positions than were learned
    with pytest.raises(P.LcuError):
        P.BatchContext(m, 2)
    c = P.Context(m, context_len=20)
    for tokens, want in (([0] * 21, []), ([m.n_vocab], []), ([-1], []), ([1, 2], [2]), ([1], [-1])):
        with pytest.raises(P.LcuError):
            c.forward(tokens, want)
    assert c.tokens_left() == 20                    # nothing was done
    c.forward([0] * 20)
    with pytest.raises(P.LcuError):
        c.forward([0])
    c.close()
    m.close()


def test_incomplete_weight_files_are_refused(tmp_path):
    P.binding.init(0)
    cfg = MODELS["narrow"]
    W = weights(cfg, 1)
    for n, (name, change) in enumerate([("l0.mix.q.b", None), ("l1.mix.lam", lambda a: a[:-1]), ("l0.mlp.e0.down", lambda a: a.T),
                                        ("final.norm", None), ("l0.mlp.shared.sg", None), ("pos", lambda a: a[:-1])]):
        broken = dict(W)
        if change is None:
            del broken[name]
        else:
            broken[name] = change(broken[name])
        S.write_model(str(tmp_path / str(n)), cfg, broken)
        with pytest.raises(P.LcuError):
            P.Model(path=str(tmp_path / str(n)))
    S.write_model(str(tmp_path / "mixed"), MODELS["ragged"], weights(MODELS["ragged"], 1))
    odd = copy.deepcopy(MODELS["ragged"])
    odd["layers"][4]["mixer"]["vdim"] = 21          # values of another size than the first layer's
    S.write_model(str(tmp_path / "odd"), odd, weights(odd, 1))
    with pytest.raises(P.LcuError):
        P.Model(path=str(tmp_path / "odd"))


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_prompt_longer_than_a_pass_and_long_decoding(tmp_path, dt):
    """2300 tokens in one call run in more than one pass; 700 tokens decoded one by one pass every edge of a
    window, with keys from far back that stand out."""
    P.binding.init(0)
    cfg = config(97, 96, 2, 1e-5, [rec(64, 2, 4, None), att(4, 2, 32, 32, 70, 9, 0.6, True, moe(4, 2, 16, 1.0, 16)),
                                   att(2, 2, 24, 32, 600, 2, 0.5, True, None)], positions=2400)
    W = weights(cfg, 2)
    S.write_model(str(tmp_path / "m"), cfg, W)
    t = np.random.default_rng(0).integers(0, 97, 2300)
    want = S.forward(cfg, W, t)
    m = P.Model(path=str(tmp_path / "m"), dtype=dt)
    c = P.Context(m, context_len=2400)
    places = list(range(0, 2300, 7)) + [2047, 2048, 2299]
    held(c.forward(t, places)[1], want[places], dt)
    c.clear_tokens()
    c.forward(t[:300])
    got = np.concatenate([c.forward(t[k:k + 1], [0])[1] for k in range(300, 1000)])
    held(got, want[300:1000], dt)
    c.close()
    m.close()


def test_llama_contexts_give_logits_at_any_place():
    """forward() on the fp16 family: logits of the places of one call equal those of calls that end there."""
    P.binding.init(0)
    m = P.Model(dim=256, multiple_of=64, n_heads=2, n_layers=2, n_vocab=320, weight_std=0.05, seed=1)
    a, b = P.Context(m, context_len=64), P.Context(m, context_len=64)
    t = np.random.default_rng(0).integers(0, 320, 12)
    tok, lg = a.forward(t, [11, 4, 0])
    assert tok == b.next_token(t)
    assert (lg[0] == b.logits().astype(np.float32)).all() and (a.logits() == b.logits()).all()
    for i, place in ((1, 4), (2, 0)):
        b.clear_tokens()
        b.next_token(t[:place + 1])
        assert np.max(np.abs(lg[i] - b.logits().astype(np.float32))) < 2e-2 * np.max(np.abs(lg[i]))
    for x in (a, b, m):
        x.close()
