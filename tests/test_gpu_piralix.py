"""Piralix on the GPU against the plain implementation (tests/piralix_plain.py): mechanisms alone, whole prompts, portions,
decoding, batches, reuse of the cache, long contexts, generation through the framework's entry points."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch  # noqa: F401  (loaded before the library: both then share torch's HIP runtime)

import piralix_plain as plain
from conftest import ROOT, progress
from piralix_cases import SPECS, attention, mlstm, model, random_tensors, rglru, spec
from ritevik_cases import LIMIT, bf16_bits, bf16_values, check_rows, row_errors

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


def tokens_of(s, n, seed=0):
    return np.random.default_rng(seed + 77).integers(0, s["vocab"], n).astype(np.uint32)


def feed(m, tokens, sizes):
    """Logits [T, V] of a sequence fed from an empty cache in portions of the given sizes (the last one repeats)."""
    m.reset_cache()
    out, at, i = [], 0, 0
    while at < len(tokens):
        part = tokens[at:at + sizes[min(i, len(sizes) - 1)]]
        out.append(m.forward_cached(part.reshape(1, -1))[0])
        at, i = at + len(part), i + 1
    assert m.cache_len() == len(tokens)
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SPECS))
def test_whole_prompt_and_layer_streams(name, dtype):
    s = SPECS[name]
    bits, w = random_tensors(s, 1)
    m = model(s, bits, dtype=dtype, n_positions=200)
    t = tokens_of(s, 139)
    trace = []
    want = plain.forward(t, s, w, trace)
    check_rows(m.forward(t), want, dtype, name)
    m.reset_cache()
    got = np.concatenate([m.layer_streams(t[:50]), m.layer_streams(t[50:51]), m.layer_streams(t[51:60])], axis=1)
    assert got.shape[0] == m.layer_runs() == len(trace)
    for i, x in enumerate(trace):
        e = np.abs(got[i] - x[:60]).max() / np.abs(x).max()
        assert e <= LIMIT[dtype], f"layer run {i}: {e:.2e}"


ZERO = {"mixer": "mix.o", "mlp": "mlp.down"}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("what", ["embedding_and_head", "mlstm", "attention", "rglru", "feed_forward", "loop"])
def test_each_mechanism_alone(what, dtype):
    s = {"mlstm": spec(48, 40, [mlstm()]), "attention": spec(48, 40, [attention()]), "rglru": spec(48, 40, [rglru()]),
         "feed_forward": spec(48, 40, [rglru(ff=72, limit=0.4)]), "loop": spec(48, 40, [mlstm()], loop=dict(start=0, stop=1, times=4)),
         "embedding_and_head": spec(48, 40, [mlstm()])}[what]
    bits, w = random_tensors(s, 2)
    for k in bits:
        if any(k.endswith(ZERO[p]) for p in {"feed_forward": ["mixer"], "loop": ["mixer", "mlp"], "embedding_and_head": ["mixer", "mlp"]}.get(what, [])):
            bits[k], w[k] = np.zeros_like(bits[k]), np.zeros_like(w[k])
    m = model(s, bits, dtype=dtype, n_positions=96)
    t = tokens_of(s, 90)
    want = plain.forward(t, s, w)
    check_rows(m.forward(t), want, dtype, what)
    check_rows(feed(m, t, [70, 1]), want, dtype, what)


def to_device(dev, a):
    return torch.from_numpy(np.ascontiguousarray(a.view(np.int16) if a.dtype == np.uint16 else a)).to(dev)


@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_operator(dev, dtype):
    """The attention operator on its own, without sink and gate and with them: portions of 33, 1, 5 and 1 tokens over one cache."""
    from async_gpu_amd import _lib, ops
    H, G, D, DV, B, P, T, scale, cap = 6, 2, 32, 64, 2, 96, 40, 0.4, 7.0
    rng = np.random.default_rng(5)
    rot = dict(dims=24, base=300.0, scaling=dict(factor=3.0, original=32, fast=4.0, slow=1.0))
    cols = dict(q=H * D, k=G * D, v=G * DV, g=H * DV)
    x = rng.standard_normal((B, T, sum(cols.values()))).astype(np.float32)
    sink = rng.standard_normal(H).astype(np.float32)
    rope = ops.rope_table(P, 24, 300.0, stretch=(3.0, 32, 4.0, 1.0))
    f, grow = plain.frequencies(rot)
    table = np.stack([np.cos(np.outer(np.arange(P), f)), np.sin(np.outer(np.arange(P), f))], -1) * grow
    assert np.abs(rope.cpu().numpy() - table).max() <= 1e-6
    for with_gate in (False, True):
        want = []
        for b in range(B):  # the plain layer with identity projections in and out; a large gate is open
            w, at = {}, 0
            for n, c in cols.items():
                w[n] = np.eye(x.shape[2])[at:at + c]
                at += c
            h = x[b].astype(np.float64)
            if not with_gate:
                h = np.concatenate([h[:, :-H * DV], np.full((T, H * DV), 1e3)], 1)
            w.update(sink=sink.astype(np.float64) if with_gate else np.full(H, -1e30), o=np.eye(H * DV))
            want.append(plain.attention(h, w, dict(heads=H, kv_heads=G, dim=D, vdim=DV, scale=scale, softcap=cap, rot=rot), 0.0))
        want, bf16 = np.stack(want), dtype == "bfloat16"
        ct = torch.int16 if bf16 else torch.float32
        kc = torch.zeros((B, G, P, D), dtype=ct, device=dev)
        vc = torch.zeros((B, G, DV, _lib.cdll().agpu_grouped_kv_stride(P)), dtype=ct, device=dev)
        at = 0
        for n in (33, 1, 5, 1):
            r = to_device(dev, x[:, at:at + n].reshape(B * n, -1).copy())
            d = _lib.GroupedAttentionDesc(H, G, D, DV, 24, scale, cap, P, B, n, at, x.shape[2], 0, _lib.DTYPE_BF16 if bf16 else _lib.DTYPE_F32)
            c = np.cumsum([0] + list(cols.values()))
            out = ops.grouped_attention(d, r, r[:, c[1]:], r[:, c[2]:], r[:, c[3]:] if with_gate else None, to_device(dev, sink) if with_gate else None, rope, kc, vc)
            e = np.abs(out.cpu().numpy().reshape(B, n, -1) - want[:, at:at + n]).max() / np.abs(want).max()
            assert e <= (2e-2 if bf16 else 1e-5), (with_gate, at, n, e)
            at += n


def test_memory_operator(dev):
    """The matrix memory on its own: portions of 70, 1, 64, 2, 1 and 5 tokens over one state, against the recurrence."""
    from async_gpu_amd import _lib, ops
    H, D, DV, B, cap, T = 3, 32, 96, 2, 5.0, 143
    rng = np.random.default_rng(6)
    cols = dict(q=H * D, k=H * D, v=H * DV, i=4, f=4)  # columns padded to fours
    x = rng.standard_normal((B, T, sum(cols.values()))).astype(np.float32)
    c = dict(zip(cols, np.cumsum([0] + list(cols.values()))))
    x[:, :, c["f"]:] += 3.0
    x[:, :, c["i"]:c["f"]] *= 4.0
    want = []
    for b in range(B):
        h = x[b].astype(np.float64)
        part = lambda n, e: h[:, c[n]:c[n] + H * e].reshape(T, H, e)  # noqa: E731
        want.append(plain.matrix_memory_recurrence(part("q", D) / np.sqrt(D), part("k", D), part("v", DV), plain.soft_cap(part("i", 1)[..., 0], cap),
                                                   plain.log_sigmoid(plain.soft_cap(part("f", 1)[..., 0], cap))).reshape(T, -1))
    want = np.stack(want)
    state, norm = torch.zeros((B, H, DV, D), device=dev), torch.zeros((B, H, 2, D + 4), device=dev)
    at = 0
    for n in (70, 1, 64, 2, 1, 5):
        r = to_device(dev, x[:, at:at + n].reshape(B * n, -1).copy())
        d = _lib.MatrixMemoryDesc(H, D, DV, cap, B, n, at, x.shape[2], 0)
        out = ops.matrix_memory(d, r, *(r[:, c[t]:] for t in "kvif"), state, norm).cpu().numpy().reshape(B, n, -1)
        # a read-out whose denominator is small magnifies rounding: each against its own size
        e = np.abs(out - want[:, at:at + n]) / (np.abs(want[:, at:at + n]).max(-1, keepdims=True) + 1e-3)
        assert np.quantile(e, 0.99) <= 2e-5 and e.max() <= 1e-3, (at, n, e.max())
        at += n


def test_recurrent_unit_operator(dev):
    """The gated recurrent unit on its own: portions of 40, 2, 1 and 5 tokens over one state, batch of two."""
    from async_gpu_amd import _lib, ops
    W, blocks, N, B, T = 192, 3, 4, 2, 48
    bs = W // blocks
    rng = np.random.default_rng(7)
    x = rng.standard_normal((B, T, 2 * W)).astype(np.float32)
    f32 = lambda *s: rng.standard_normal(s).astype(np.float32)  # noqa: E731
    conv, cb, gb, lam = 0.6 * f32(W, N), f32(W), f32(blocks, 2, bs), f32(W) - 2.0
    gates = bf16_bits(rng.standard_normal((blocks, 2, bs, bs)) / 8)
    g = bf16_values(gates)
    w = {"y": np.eye(2 * W)[:W], "x": np.eye(2 * W)[W:], "y.b": 0.0, "x.b": 0.0, "conv": conv.astype(np.float64), "conv.b": cb.astype(np.float64), "ra": g[:, 0],
         "ri": g[:, 1], "ra.b": gb[:, 0].astype(np.float64), "ri.b": gb[:, 1].astype(np.float64), "lam": lam.astype(np.float64), "o": np.eye(W)}
    want = np.stack([plain.rglru(x[b].astype(np.float64), w, None, None) for b in range(B)])
    state, ring = torch.zeros((B, W), device=dev), torch.zeros((B, N, W), device=dev)
    at = 0
    for n in (40, 2, 1, 5):
        d = _lib.GatedLruDesc(W, blocks, N, B, n, at, 2 * W, 0, 0, W)
        out = ops.gated_lru(d, to_device(dev, x[:, at:at + n].reshape(B * n, -1).copy()), to_device(dev, conv), to_device(dev, cb), to_device(dev, gates),
                            to_device(dev, gb), to_device(dev, lam), state, ring)
        e = np.abs(out.cpu().numpy().reshape(B, n, -1) - want[:, at:at + n]).max() / np.abs(want).max()
        assert e <= 2e-5, (at, n, e)
        at += n


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SPECS))
def test_prompt_against_token_by_token(name, dtype):
    s = SPECS[name]
    bits, w = random_tensors(s, 3)
    m = model(s, bits, dtype=dtype, n_positions=96)
    t = tokens_of(s, 75)
    want = plain.forward(t, s, w)
    check_rows(feed(m, t, [1]), want, dtype, "token by token")
    check_rows(feed(m, t, [60, 1]), want, dtype, "prompt, then tokens")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [[2], [3, 2, 5, 4], [17, 1, 33, 2], [16], [31, 32, 1, 33], [15, 64, 1, 2], [65, 63, 3], [128, 3]])
def test_portions(sizes, dtype):
    s = SPECS["mixed"]
    bits, w = random_tensors(s, 4)
    m = model(s, bits, dtype=dtype, n_positions=140)
    t = tokens_of(s, 131)
    check_rows(feed(m, t, sizes), plain.forward(t, s, w), dtype, str(sizes))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 2, 3, 4, 5])
def test_first_tokens(n, dtype):
    """Sequences shorter than the convolution, whole and token by token."""
    s = SPECS["plain"]
    bits, w = random_tensors(s, 5)
    m = model(s, bits, dtype=dtype, n_positions=8)
    t = tokens_of(s, n, n)
    want = plain.forward(t, s, w)
    check_rows(feed(m, t, [n]), want, dtype)
    check_rows(feed(m, t, [1]), want, dtype)


# ---- attention ----

def one_attention(seed, vocab=300, no_sink=True, **kw):
    s = spec(64, vocab, [attention(**dict(dict(heads=4, kv_heads=2, dim=32, vdim=32, rot=8, base=1e6, softcap=60.0), **kw))])
    bits, w = random_tensors(s, seed)
    if no_sink:
        bits["l0.mix.sink"][:] = bf16_bits(np.float32(-20.0))
        w["l0.mix.sink"][:] = -20.0
    return s, bits, w


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_keys(dtype):
    """A sharp softmax that picks single keys anywhere in the context, at tile, chunk and split borders."""
    s, bits, w = one_attention(6, scale=1.0)
    t = tokens_of(s, 460)
    want = plain.forward(t, s, w)
    cut = plain.forward(t[200:], s, w)[-60:]  # without the first 200 keys the late rows are far off
    assert np.median(row_errors(cut, want[-60:])) > 0.2
    m = model(s, bits, dtype=dtype, n_positions=512)
    limit = {"float32": 2e-4, "bfloat16": 0.12}[dtype]
    for sizes in ([460], [400, 1], [63, 64, 65, 128, 1, 1, 1, 2]):
        e = row_errors(feed(m, t, sizes), want)
        assert np.sort(e)[int(0.98 * e.size)] <= limit and e.max() <= 3 * limit, (sizes, e.max(), int(e.argmax()))


@pytest.mark.parametrize("dtype", DTYPES)
def test_needle_at_every_distance(dtype):
    """One key that stands out at a chosen place and a query that finds it from the end of the context: every place around the
    borders of tiles (32) and splits (128), decoded alone and inside a portion."""
    s, bits, w = one_attention(7)
    d, H, G, D, R = s["width"], 4, 2, 32, 8
    hn = plain.rms_norm(w["embed"][[7, 9]], w["l0.norm1"], 1e-5)  # token 7 is the needle, token 9 asks for it
    k = (w["l0.mix.k"] @ hn[0]).reshape(G, D)
    wq = w["l0.mix.q"].reshape(H, D, d).copy()
    for h in range(H):
        wq[h, R:] += 6.0 * np.outer(k[h // 2, R:], hn[1]) / (hn[1] @ hn[1])  # the dimensions that do not turn
    bits["l0.mix.q"] = bf16_bits(wq.reshape(-1, d))
    w["l0.mix.q"] = bf16_values(bits["l0.mix.q"])
    m = model(s, bits, dtype=dtype, n_positions=400)
    base = np.random.default_rng(8).integers(10, s["vocab"], 330).astype(np.uint32)
    for place in (0, 1, 30, 31, 32, 33, 62, 63, 64, 65, 127, 128, 191, 192, 255, 256, 300, 318, 319, 320):
        t = base.copy()
        t[place], t[-1] = 7, 9
        want = plain.forward(t, s, w)[-1:]
        if place == 30:  # the needle matters
            t2 = base.copy()
            t2[-1] = 9
            assert row_errors(plain.forward(t2, s, w)[-1:], want)[0] > 0.2
        for sizes in ([330], [329, 1], [310, 20], [326, 4]):
            e = row_errors(feed(m, t, sizes)[-1:], want)[0]
            assert e <= {"float32": 2e-4, "bfloat16": 0.08}[dtype], (place, sizes, e)


@pytest.mark.parametrize("what", ["sink", "cap", "stretch", "gate", "group", "plain_rotation"])
def test_attention_constants_show(what):
    """Each constant where it matters: the plain model without it is far off, the library with it is not, in prompts and decoding."""
    kw = {"sink": dict(scale=0.05), "cap": dict(scale=1.0, softcap=2.0), "stretch": dict(rot=32, base=100.0, scale=0.6), "gate": {},
          "group": dict(heads=6, kv_heads=3, scale=0.6), "plain_rotation": dict(rot=32, base=100.0, scale=0.6, scaling=None)}[what]
    s, bits, w = one_attention(9, vocab=60, no_sink=what != "sink", **kw)
    t = tokens_of(s, 140)
    if what == "sink":
        big = np.array([3.0, -2.0, 5.0, 0.0])
        bits["l0.mix.sink"], w["l0.mix.sink"] = bf16_bits(big), bf16_values(bf16_bits(big))
    want = plain.forward(t, s, w)
    s2, w2 = copy.deepcopy(s), dict(w)
    m2 = s2["layers"][0]["mixer"]
    if what == "sink":
        w2["l0.mix.sink"] = np.full(4, -1e30)
    elif what == "cap":
        m2["softcap"] = 1e6
    elif what == "stretch":
        m2["rot"]["scaling"] = None
    elif what == "gate":
        w2["l0.mix.g"] = np.zeros_like(w["l0.mix.g"])
    elif what == "group":  # neighbours share a key head; every other head does not
        w2["l0.mix.q"] = w["l0.mix.q"].reshape(3, 2, 32, -1).swapaxes(0, 1).reshape(192, -1)
    else:
        m2["rot"]["scaling"] = dict(factor=4.0, fast=24.0, slow=1.5, original=64)
    assert np.quantile(row_errors(plain.forward(t, s2, w2), want), 0.9) > 0.1
    for dtype in DTYPES:
        m = model(s, bits, dtype=dtype, n_positions=160)
        for sizes in ([140], [1], [100, 1]):
            check_rows(feed(m, t, sizes), want, dtype, f"{dtype} {sizes}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_keys(dtype):
    """4500 keys: several chunks per split of the decode kernel, long rows of the prompt kernel."""
    s, bits, w = one_attention(13, scale=0.6, heads=2, kv_heads=1)
    t = tokens_of(s, 4506)
    want = plain.forward(t, s, w)[-6:]
    m = model(s, bits, dtype=dtype, n_positions=4608)
    m.reset_cache()
    m.forward_cached(t[:3000].reshape(1, -1), all_rows=False)
    m.forward_cached(t[3000:4500].reshape(1, -1), all_rows=False)
    got = np.concatenate([m.forward_cached(t[i:i + 1].reshape(1, -1))[0] for i in range(4500, 4506)])
    e = row_errors(got, want)
    assert e.max() <= {"float32": 2e-4, "bfloat16": 0.1}[dtype], e


def test_prompt_kernel_with_and_without_a_key_split():
    """Enough column blocks that every wave takes one of its own, against the same rows with the keys split over waves."""
    s = spec(64, 50, [attention(heads=32, kv_heads=16, dim=16, vdim=32, rot=16)])
    bits, _ = random_tensors(s, 16)
    t = np.random.default_rng(1).integers(0, 50, (5, 900)).astype(np.uint32)
    m = model(s, bits, dtype="bfloat16", n_positions=900, max_batch=5)
    m.reset_cache()
    many = m.forward_cached(t)
    for b in (0, 4):
        m.reset_cache()
        one = m.forward_cached(t[b:b + 1])[0]
        assert row_errors(many[b], one.astype(np.float64)).max() <= 2e-2


# ---- recurrent mixers ----

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("gates", ["weak_input", "strong_input", "forgetful", "steady"])
def test_memory_gates_at_their_ends(gates, dtype):
    """Log gates near their caps on both sides: the running maximum rises, falls and stays, over chunk borders and decoding."""
    s = spec(48, 60, [mlstm(heads=2, dim=24, vdim=16, cap=11.0)])
    bits, w = random_tensors(s, 14)
    for name, value in {"weak_input": {"i.b": -9.0}, "strong_input": {"i.b": 9.0}, "forgetful": {"f.b": -12.0}, "steady": {"f.b": 30.0}}[gates].items():
        bits["l0.mix." + name] = bf16_bits(np.full(2, value))
        w["l0.mix." + name] = bf16_values(bits["l0.mix." + name])
    t = tokens_of(s, 200)
    want = plain.forward(t, s, w)
    m = model(s, bits, dtype=dtype, n_positions=200)
    for sizes in ([200], [1], [63, 2, 65, 1]):
        check_rows(feed(m, t, sizes), want, dtype, f"{gates} {sizes}")


def test_memory_of_a_far_token():
    """One loud write among hundreds of faint ones (its input gate far above theirs) is read back at the end, in fp32 to rounding:
    whatever chunk or decode step it falls on."""
    s = spec(48, 60, [mlstm(heads=2, dim=24, vdim=16, cap=8.0)])
    bits, w = random_tensors(s, 15)
    hn = plain.rms_norm(w["embed"][7], w["l0.norm1"], 1e-5)
    wi = w["l0.mix.i"] + 9.0 * hn / (hn @ hn)
    bits["l0.mix.i"], bits["l0.mix.i.b"], bits["l0.mix.f.b"] = bf16_bits(wi), bf16_bits(np.full(2, -4.0)), bf16_bits(np.full(2, 8.0))
    for k in ("l0.mix.i", "l0.mix.i.b", "l0.mix.f.b"):
        w[k] = bf16_values(bits[k])
    m = model(s, bits, dtype="float32", n_positions=260)
    base = np.random.default_rng(3).integers(10, 60, 250).astype(np.uint32)
    without = plain.forward(base, s, w)[-1:]
    for place in (0, 1, 63, 64, 65, 127, 128, 200, 240, 248):
        t = base.copy()
        t[place] = 7
        want = plain.forward(t, s, w)[-1:]
        if place == 64:
            assert row_errors(without, want)[0] > 0.1
        for sizes in ([250], [245, 1], [60, 9, 1, 70, 1]):
            assert row_errors(feed(m, t, sizes)[-1:], want)[0] <= 1e-4, (place, sizes)


def test_long_decoding_keeps_the_state():
    """300 tokens decoded one at a time behind a prompt of 5 (fp32), with decays close to one."""
    s = spec(48, 60, [mlstm(heads=2, dim=24, vdim=16), rglru(width=32, blocks=2), attention(heads=2, kv_heads=1)], loop=dict(start=0, stop=2, times=2))
    bits, w = random_tensors(s, 12)
    m = model(s, bits, dtype="float32", n_positions=320)
    t = tokens_of(s, 305)
    want = plain.forward(t, s, w)
    check_rows(feed(m, t, [5, 1]), want, "float32")
    late = plain.forward(t[150:], s, w)[-20:]  # and the state matters over that distance
    assert np.median(row_errors(late, want[-20:])) > 0.02


# ---- batches, reuse, generation ----

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("B", [2, 3, 5, 17, 33])
def test_batch_against_each_alone(B, dtype):
    """Unequal requests of equal length side by side, prompt, portions and decoding, against the plain model."""
    s = SPECS["mixed"]
    bits, w = random_tensors(s, 10)
    m = model(s, bits, dtype=dtype, n_positions=96, max_batch=B)
    t = np.random.default_rng(B).integers(0, s["vocab"], (B, 90)).astype(np.uint32)
    m.reset_cache()
    got = [m.forward_cached(t[:, :70]), m.forward_cached(t[:, 70:75])] + [m.forward_cached(t[:, i:i + 1]) for i in range(75, 80)]
    got = np.concatenate(got + [m.forward_cached(t[:, 80:])], axis=1)
    for b in sorted({0, 1, B // 2, B - 1}):
        check_rows(got[b], plain.forward(t[b], s, w), dtype, f"sequence {b}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_cache_and_state_used_again(dtype):
    """A request after others (longer and shorter ones, ended at any place) equals the same request on a fresh model."""
    s = SPECS["mixed"]
    bits, _ = random_tensors(s, 11)
    m = model(s, bits, dtype=dtype, n_positions=128, max_batch=2)
    t = tokens_of(s, 50)
    first = feed(m, t, [30, 1])
    feed(m, tokens_of(s, 121, 1), [121])
    feed(m, tokens_of(s, 2, 2), [2])
    m.reset_cache()
    m.forward_cached(np.stack([tokens_of(s, 70, 3), tokens_of(s, 70, 4)]))
    assert np.array_equal(first, feed(m, t, [30, 1]))
    assert np.array_equal(first, feed(model(s, bits, dtype=dtype, n_positions=128, max_batch=2), t, [30, 1]))


def greedy_plain(s, w, prompt, n):
    """Greedy tokens of the plain model and the smallest margin between the best two logits on the way."""
    seq, margin = list(prompt), np.inf
    for _ in range(n):
        lg = plain.forward(np.array(seq), s, w)[-1]
        top = np.sort(lg)[-2:]
        margin = min(margin, top[1] - top[0])
        seq.append(int(lg.argmax()))
    return seq, margin


def test_greedy_generation_through_the_runtime():
    """generate_cached (graph replays) and generate (no cache) against the plain model; a second run, the eager path and a batch
    give the same tokens."""
    s = SPECS["mixed"]
    bits, w = random_tensors(s, 79)
    m = model(s, bits, dtype="float32", n_positions=96, max_batch=3)
    prompt = tokens_of(s, 21)
    want, margin = greedy_plain(s, w, prompt, 24)
    assert margin > 1e-3  # no near tie on the way: rounding cannot change a token
    (got,), _ = m.generate_cached(prompt, 24)
    assert list(got) == want
    assert list(m.generate(prompt, 24)) == want
    (again,), _ = m.generate_cached(prompt, 24)
    assert list(again) == want
    m.set_decode_mode(m.DECODE_EAGER)
    (eager,), _ = m.generate_cached(prompt, 24)
    assert list(eager) == want
    m.set_decode_mode(m.DECODE_AUTO)
    batch, _ = m.generate_cached(np.stack([prompt, tokens_of(s, 21, 5), prompt]), 24)
    assert list(batch[0]) == want and list(batch[2]) == want
    eos = want[30]
    (short,), _ = m.generate_cached(prompt, 24, eos=eos)
    assert list(short) == want[:want.index(eos, 21)]


def test_graph_replays_match_eager_steps():
    """Decode steps replayed as graphs, with eager work in between, leave the logits that eager steps leave."""
    s = SPECS["one_pass"]
    bits, _ = random_tensors(s, 18)
    m = model(s, bits, dtype="bfloat16", n_positions=300)
    prompt = tokens_of(s, 100)

    def run(mode):
        m.set_decode_mode(mode)
        m.reset_cache()
        m.forward_cached(prompt.reshape(1, -1), all_rows=False)
        out = []
        for n in (1, 3, 40, 5):
            m.decode_steps(1, n)
            out.append(m.last_logits()[0])
            m.ctx.sync()
        return np.array(out)
    eager = run(m.DECODE_EAGER)
    for _ in range(3):
        assert np.array_equal(run(m.DECODE_AUTO), eager)


def test_sampling_through_the_runtime():
    from async_gpu_amd import ops
    s = SPECS["one_pass"]
    bits, _ = random_tensors(s, 19)
    m = model(s, bits, dtype="float32", n_positions=64)
    prompt = tokens_of(s, 9)
    (greedy,), _ = m.generate_cached(prompt, 20)
    assert list(m.generate_cached_sampling(prompt, 20, 1, 1.0, ops.SimpleRng(3))) == list(greedy)
    a = m.generate_cached_sampling(prompt, 20, 10, 0.9, ops.SimpleRng(4))
    assert list(a) == list(m.generate_cached_sampling(prompt, 20, 10, 0.9, ops.SimpleRng(4)))
    lg = m.forward(a[:-1])  # every drawn token is one of the ten best of its step
    for i in range(len(prompt), len(a)):
        assert a[i] in np.argsort(-lg[i - 1])[:10]


def test_errors_are_raised_on_the_host():
    from async_gpu_amd import _lib, piralix, weights
    s = SPECS["one_pass"]
    bits, _ = random_tensors(s, 20)
    with pytest.raises(weights.ModelFileError, match="l1.mix.sink"):
        model(s, {k: v for k, v in bits.items() if k != "l1.mix.sink"})
    with pytest.raises(weights.ModelFileError, match="expected shape"):
        model(s, dict(bits, **{"l0.mix.ra": bits["l0.mix.ra"][:, :-1]}))
    m = model(s, bits, n_positions=16)
    with pytest.raises(_lib.AgpuError) as e:
        m.forward_cached(np.zeros((1, 17), np.uint32))
    assert e.value.code == _lib.ERR_DIM_OUT_OF_RANGE
    with pytest.raises(_lib.AgpuError) as e:
        m.set_tensor("l9.norm1", bits["l0.norm1"])
    assert e.value.code == _lib.ERR_KERNEL_NOT_FOUND
    bare = piralix.PiralixModel(piralix.PiralixConfig(s))
    with pytest.raises(_lib.AgpuError, match="embed"):
        bare.forward_cached(np.zeros((1, 1), np.uint32))
    for layer, key, value in ((0, "blocks", 3), (1, "kv_heads", 3), (1, "dim", 300), (2, "dim", 300), (2, "gate_cap", 0.0)):
        bad = copy.deepcopy(s)
        bad["layers"][layer]["mixer"][key] = value
        with pytest.raises(_lib.AgpuError, match=f"layer {layer}"):
            piralix.PiralixModel(piralix.PiralixConfig(bad))


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_runner_and_command_line(tmp_path, dtype):
    """bin/trace_run and the generation command on a model folder, through the registry."""
    from async_gpu_amd import models, weights
    s = SPECS["mixed"]
    bits, w = random_tensors(s, 21)
    (tmp_path / "model").mkdir()
    (tmp_path / "model" / "config.json").write_text(json.dumps({k: v for k, v in s.items() if v is not None}))
    weights.write_safetensors(str(tmp_path / "model" / "model.safetensors"), {k: ("BF16", v) for k, v in bits.items()})
    m = models.load_model(str(tmp_path / "model"), dtype=dtype, n_positions=64)
    a, b = tokens_of(s, 40, 1), tokens_of(s, 7, 2)
    check_rows(m.forward(a), plain.forward(a, s, w), dtype)
    m.close()
    steps = [("a", a[:20], [3, 19], []), ("a", a[20:22], [], []), ("a", a[22:39], [0, 16], []), ("a", a[39:], [0], ["a"]), ("b", b, [0, 6], ["b"])]
    text = "".join(json.dumps({"step": i, "entries": [{"id": n, "tokens": t.tolist(), "want": want}], "end": end}) + "\n"
                   for i, (n, t, want, end) in enumerate(steps))
    progress(f"trace_run {dtype}")
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "40"], input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(5)]
    want = {"a": plain.forward(a, s, w), "b": plain.forward(b, s, w)}
    start = [0, 20, 22, 39, 0]
    for i, (n, _, places, _) in enumerate(steps):
        path = tmp_path / f"{i}.f32"
        assert path.exists() == bool(places)
        if places:
            check_rows(np.fromfile(path, "<f4").reshape(len(places), -1), want[n][[start[i] + p for p in places]], dtype, f"step {i}")
    r = subprocess.run([sys.executable, os.path.join(ROOT, "async-gpu_amd", "examples", "generate.py"), str(tmp_path / "model"), "--dtype", dtype,
                        "--tokens", ",".join(map(str, b.tolist())), "--max-new-tokens", "5", "--n-positions", "32"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    out = [int(x) for x in r.stdout.splitlines()[-1].split(",")]
    assert out[:7] == b.tolist() and len(out) == 12
