"""What the GPU tests of the layered decoders share: device arrays of both element types, comparisons, calls in portions."""
import ctypes as C

import numpy as np
import pytest

import plain_stack as S

F32, BF16 = 1, 0
BOTH = pytest.mark.parametrize("dt", [BF16, F32], ids=["bf16", "f32"])


@pytest.fixture(scope="module")
def gpu():
    import gpu_helpers as G
    G.setup()
    stream = G.B.vp()
    G.B.check(G.L().lcu_stream_create(C.byref(stream)))
    G.stream = stream.value
    yield G
    G.release()
    G.B.check(G.L().lcu_stream_destroy(G.stream))


def rounded(a):
    """Values a bfloat16 holds, as float64 (every input here is one, so that both types see the same numbers)."""
    return S.bf16_values(S.bf16_bits(a)).reshape(np.shape(a)).astype(np.float64)


def up64(n):
    return (n + 63) // 64 * 64


def pad(a, cols):
    out = np.zeros(a.shape[:-1] + (cols,))
    out[..., :a.shape[-1]] = a
    return out


def put(G, a, dt=F32):
    return G.dev_keep(np.asarray(a, np.float32) if dt == F32 else S.bf16_bits(a).reshape(np.shape(a)))


def zeros(G, shape, dt=F32):
    return put(G, np.zeros(shape), dt)


def get(G, buf, shape, dt=F32):
    G.B.check(G.L().lcu_sync(G.stream))
    if dt == F32:
        return G.host(buf, shape, np.float32).astype(np.float64)
    return S.bf16_values(G.host(buf, shape, np.uint16)).astype(np.float64)


def get_ints(G, buf, shape):
    G.B.check(G.L().lcu_sync(G.stream))
    return G.host(buf, shape, np.int32)


def ints(G, a):
    return G.dev_keep(np.asarray(a, np.int32))


def close(got, want, dt, scale=None, f32=2e-5, bf16=2.0 ** -8):
    scale = np.max(np.abs(want)) if scale is None else scale
    err = np.max(np.abs(got - want)) / max(scale, 1e-30)
    assert err <= (f32 if dt == F32 else bf16), err


def call(G, name, *args):
    G.B.check(getattr(G.L(), name)(*[a.ptr if hasattr(a, "ptr") else a for a in args], G.stream), name)


def pack_gated(gate, up, ld):
    """Gate and up rows in blocks of 32 and 32, hidden units padded to ld."""
    out = np.zeros((2 * ld, gate.shape[1]))
    j = np.arange(gate.shape[0])
    out[j // 32 * 64 + j % 32] = gate
    out[j // 32 * 64 + j % 32 + 32] = up
    return out


# ---- whole models -----------------------------------------------------------------------------------------
def errors(got, want):
    d = got - want
    d = d - d.mean(1, keepdims=True)
    return np.sqrt((d ** 2).mean(1)) / want.std()


def feed(ctx, tokens, cuts):
    out, at = [], 0
    for n in cuts:
        out.append(ctx.forward(tokens[at:at + n], range(n))[1])
        at += n
    assert at == len(tokens)
    return np.concatenate(out)
