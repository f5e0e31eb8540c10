"""Ritevik on the GPU against the plain implementation (tests/ritevik_plain.py): mechanisms alone, whole prompts, portions,
decoding, batches, reuse of the cache, long contexts, generation through the framework's entry points."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch  # noqa: F401  (loaded before the library: both then share torch's HIP runtime)

import ritevik_plain as plain
from conftest import ROOT, progress
from ritevik_cases import LIMIT, SPECS, bf16_bits, bf16_values, check_rows, delta, latent, model, random_tensors, row_errors, spec

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


def tokens_of(s, n, seed=0):
    return np.random.default_rng(seed + 77).integers(0, s["vocab"], n).astype(np.uint32)


def feed(m, tokens, sizes):
    """Logits [T, V] of a sequence fed from an empty cache in portions of the given sizes (the last one repeats)."""
    m.reset_cache()
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = sizes[min(i, len(sizes) - 1)]
        part = tokens[at:at + n]
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
    got = m.layer_streams(t[:50])
    assert got.shape[0] == m.layer_runs() == len(trace)
    for i, x in enumerate(trace):
        e = np.abs(got[i] - x[:50]).max() / np.abs(x).max()
        assert e <= LIMIT[dtype], f"layer run {i}: {e:.2e}"


ZERO = {"mixer": ("mix.o",), "mlp": ("mlp.down",), "side": ("side.proj",)}


def silence(bits, w, parts):
    for k in bits:
        if any(k.endswith(t) for p in parts for t in ZERO[p]):
            bits[k] = np.zeros_like(bits[k])
            w[k] = np.zeros_like(w[k])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("what", ["embedding_and_head", "latent", "delta", "feed_forward", "side", "loop"])
def test_each_mechanism_alone(what, dtype):
    s = {"latent": spec(48, 40, [latent(ff=0)]), "delta": spec(48, 40, [delta(ff=0)]), "feed_forward": spec(48, 40, [latent()]),
         "side": spec(48, 40, [latent(), delta()], side=20), "loop": spec(48, 40, [latent()], loop=dict(start=0, stop=1, times=4)),
         "embedding_and_head": spec(48, 40, [latent()])}[what]
    bits, w = random_tensors(s, 2)
    off = {"latent": (), "delta": (), "feed_forward": ("mixer",), "side": ("mixer", "mlp"), "loop": ("mixer", "mlp"), "embedding_and_head": ("mixer", "mlp")}[what]
    silence(bits, w, off)
    m = model(s, bits, dtype=dtype, n_positions=64)
    t = tokens_of(s, 60)
    check_rows(m.forward(t), plain.forward(t, s, w), dtype, what)


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_operator(dev, dtype):
    """The attention operator on its own: three calls over one cache, both forms, batch of two."""
    from async_gpu_amd import _lib, ops
    H, D, R, DV, C, B, P, eps, scale = 3, 16, 24, 32, 64, 2, 96, 1e-5, 0.3
    rng = np.random.default_rng(5)
    bf = lambda *sh: bf16_bits(rng.standard_normal(sh) / np.sqrt(sh[-1]) * 1.5)  # noqa: E731
    uk, uv = bf(H * D, C), bf(H * DV, C)
    norm, sink = rng.uniform(0.5, 1.5, C).astype(np.float32), rng.standard_normal(H).astype(np.float32)
    T = 70
    q = rng.standard_normal((B, T, H * (D + R))).astype(np.float32)
    down = rng.standard_normal((B, T, C + R)).astype(np.float32)
    eye = np.eye
    want = []
    for b in range(B):  # the plain layer with identity projections in and out
        h = np.concatenate([q[b], down[b]], 1).astype(np.float64)
        n, nq = h.shape[1], H * (D + R)
        w = {"q": eye(n)[:nq], "dkv": eye(n)[nq:], "dkv.norm": norm.astype(np.float64), "uk": bf16_values(uk), "uv": bf16_values(uv),
             "sink": sink.astype(np.float64), "o": eye(H * DV)}
        want.append(plain.latent_attention(h, w, dict(heads=H, dim=D, rot_dim=R, vdim=DV, kv_rank=C, scale=scale, rot=dict(base=500.0, dims=R)), eps))
    want = np.stack(want)
    to = lambda a: torch.from_numpy(np.ascontiguousarray(a.view(np.int16) if a.dtype == np.uint16 else a)).to(dev)  # noqa: E731
    rope = ops.rope_table(P, R, 500.0)
    bf16 = dtype == "bfloat16"
    row = _lib.cdll().agpu_latent_cache_row(C, R)
    cache = torch.zeros((B, P, row), dtype=torch.int16 if bf16 else torch.float32, device=dev)
    both = np.concatenate([q, down], 2)
    at = 0
    for n, tiled in ((33, bf16), (36, False), (1, False)):
        x = to(both[:, at:at + n].reshape(B * n, -1).copy())
        d = _lib.LatentAttentionDesc(H, D, R, R, DV, C, scale, eps, P, B, n, at, both.shape[2], 0, _lib.DTYPE_BF16 if bf16 else _lib.DTYPE_F32, int(tiled))
        out = ops.latent_attention(d, x, x[:, H * (D + R):], to(norm), to(uk), to(uv), to(sink), rope, cache)
        e = np.abs(out.cpu().numpy().reshape(B, n, -1) - want[:, at:at + n]).max() / np.abs(want).max()
        assert e <= (2e-2 if bf16 else 1e-5), (at, n, e)
        at += n


def test_delta_operator(dev):
    """The delta operator on its own: portions of 40, 2, 1 and 5 tokens over one state, batch of two, two heads per key head."""
    from async_gpu_amd import _lib, ops
    H, HK, D, DV, N, ra, rg, B, eps = 4, 2, 32, 24, 3, 32, 64, 2, 1e-5
    rng = np.random.default_rng(6)
    cols = dict(q=HK * D, k=HK * D, v=H * DV, b=H, a1=ra, g1=rg)
    T = 48
    x = {k: rng.standard_normal((B, T, n)).astype(np.float32) for k, n in cols.items()}
    a2, g2 = bf16_bits(rng.standard_normal((H * D, ra)) / 6), bf16_bits(rng.standard_normal((H * DV, rg)) / 8)
    conv = {k: (0.6 * rng.standard_normal((cols[k], N))).astype(np.float32) for k in "qkv"}
    a_log, bias = rng.uniform(-2, 0, H).astype(np.float32), rng.uniform(-5, 0, H * D).astype(np.float32)
    norm = rng.uniform(0.5, 1.5, DV).astype(np.float32)
    want = []
    for b in range(B):
        h = np.concatenate([x[k][b] for k in cols], 1).astype(np.float64)
        w, at = {}, 0
        for k, n in cols.items():
            w[k] = np.eye(h.shape[1])[at:at + n]
            at += n
        w.update({"a2": bf16_values(a2), "g2": bf16_values(g2), "A_log": a_log.astype(np.float64), "dt_bias": bias.astype(np.float64),
                  "norm": norm.astype(np.float64), "o": np.eye(H * DV)}, **{k + ".conv": v.astype(np.float64) for k, v in conv.items()})
        want.append(plain.channel_delta(h, w, dict(heads=H, kv_heads=HK, dim=D, vdim=DV), eps))
    want = np.stack(want)
    to = lambda a: torch.from_numpy(np.ascontiguousarray(a.view(np.int16) if a.dtype == np.uint16 else a)).to(dev)  # noqa: E731
    pad = {k: (n + 3) // 4 * 4 for k, n in cols.items()}
    col, ld = {}, 0
    for k in cols:
        col[k], ld = ld, ld + pad[k]
    rows = np.zeros((B, T, ld), np.float32)
    for k, n in cols.items():
        rows[:, :, col[k]:col[k] + n] = x[k]
    state = torch.zeros((B, H, DV, D), device=dev)
    ring = torch.zeros((B, N, 2 * HK * D + H * DV), device=dev)
    taps = to(np.concatenate([conv[k] for k in "qkv"]))
    at = 0
    for n in (40, 2, 1, 5):
        d = _lib.ChannelDeltaDesc(H, HK, D, DV, N, ra, rg, eps, B, n, at, ld, 0, *(col[k] for k in ("q", "k", "v", "b", "a1", "g1")))
        out = ops.channel_delta(d, to(rows[:, at:at + n].reshape(B * n, ld).copy()), taps, to(a_log), to(bias), to(a2), to(g2), to(norm), state, ring)
        e = np.abs(out.cpu().numpy().reshape(B, n, -1) - want[:, at:at + n]).max() / np.abs(want).max()
        assert e <= 2e-5, (at, n, e)
        at += n


@pytest.mark.parametrize("M,N,K", [(1, 70, 96), (3, 64, 1056), (4, 20000, 64), (7, 48, 320), (20, 130, 2080), (40, 96, 64), (130, 200, 544), (300, 8500, 96),
                                   (600, 8192, 64), (1100, 3072, 160)])
def test_dense_linear_and_gated(dev, M, N, K):
    """Every kernel the launchers choose between, fp32 and bf16 rows, with bias and residual; and the gated form."""
    from async_gpu_amd import _lib, ops
    rng = np.random.default_rng(M + N + K)
    w = bf16_bits(rng.standard_normal((N, K)) / np.sqrt(K))
    x = bf16_values(bf16_bits(rng.standard_normal((M, K)))).astype(np.float32)
    bias, res = rng.standard_normal(N).astype(np.float32), rng.standard_normal((M, N)).astype(np.float32)
    ref = x.astype(np.float64) @ bf16_values(w).T
    to = lambda a: torch.from_numpy(np.ascontiguousarray(a.view(np.int16) if a.dtype == np.uint16 else a)).to(dev)  # noqa: E731
    xd, wd = to(x), to(w)
    for dtype in (_lib.DTYPE_F32, _lib.DTYPE_BF16):
        y = ops.dense_linear(xd, wd, to(bias), to(res), dtype).cpu().numpy()
        assert np.abs(y - (ref + bias + res)).max() <= 2e-5, (dtype, np.abs(y - (ref + bias + res)).max())
        y = ops.dense_linear(xd, wd, dtype=dtype, gated=True).cpu().numpy()
        want = plain.silu(ref[:, 0::2]) * ref[:, 1::2]
        assert np.abs(y - want).max() <= 2e-5 * (1 + np.abs(want).max()), dtype


@pytest.mark.parametrize("rows,d", [(1, 8), (5, 100), (33, 1000), (3, 5000)])
def test_rms_norm(dev, rows, d):
    from async_gpu_amd import ops
    rng = np.random.default_rng(d)
    x, w = rng.standard_normal((rows, d)).astype(np.float32) * 3, rng.standard_normal(d).astype(np.float32)
    for off in (0.0, 1.0):
        y = ops.rms_norm(torch.from_numpy(x).to(dev), torch.from_numpy(w).to(dev), 1e-5, off).cpu().numpy()
        assert np.abs(y - plain.rms_norm(x.astype(np.float64), off + w.astype(np.float64), 1e-5)).max() <= 2e-5


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
@pytest.mark.parametrize("sizes", [[2], [3, 2, 5, 4], [17, 1, 33, 2], [16], [31, 32, 1, 33], [15, 64, 1, 2]])
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


def sharp_attention(seed=6, scale=2.5, heads=2):
    """One attention layer whose softmax picks single keys anywhere in the context."""
    s = spec(64, 300, [latent(heads=heads, dim=16, rot=8, vdim=32, rank=64, scale=scale, base=1e6, ff=0)])
    bits, w = random_tensors(s, seed)
    w["l0.mix.sink"][:] = 0.0
    bits["l0.mix.sink"][:] = 0
    return s, bits, w


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_keys(dtype):
    """Keys far behind the query, at tile and chunk borders, in prompts, portions and decoding."""
    s, bits, w = sharp_attention()
    t = tokens_of(s, 460)
    want = plain.forward(t, s, w)
    # the planted needle: without the first 200 keys the late rows are far off, so that a lost key cannot hide
    cut = plain.forward(t[200:], s, w)[-60:]
    assert np.median(row_errors(cut, want[-60:])) > 0.2
    m = model(s, bits, dtype=dtype, n_positions=512)
    limit = {"float32": 2e-4, "bfloat16": 0.12}[dtype]
    for sizes in ([460], [400, 1], [63, 64, 65, 128, 1, 1, 1, 2]):
        e = row_errors(feed(m, t, sizes), want)
        assert np.sort(e)[int(0.98 * e.size)] <= limit and e.max() <= 3 * limit, (sizes, e.max(), int(e.argmax()))


@pytest.mark.parametrize("dtype", DTYPES)
def test_needle_at_every_distance(dtype):
    """One key that stands out at a chosen place and a query that finds it from the end of the context: every place around the
    borders of tiles (32), chunks (64) and splits, decoded alone and inside a portion."""
    s, bits, w = sharp_attention(scale=0.2)
    d, H, D = s["width"], 2, 16
    # token 7 is the needle and token 9 asks for it: through W_q, token 9's query is 40 times the needle's key
    hn = plain.rms_norm_zero_centred(plain.rms_norm_zero_centred(w["embed"][[7, 9]], w["embed.norm"], 1e-5), w["l0.norm1"], 1e-5)
    c = plain.rms_norm(hn[:1] @ w["l0.mix.dkv"][:64].T, w["l0.mix.dkv.norm"], 1e-5)
    k = (c @ w["l0.mix.uk"].T).reshape(H, D)
    wq = w["l0.mix.q"].reshape(H, D + 8, d).copy()
    wq[:, :D] += 40.0 * k[:, :, None] * hn[1] / (hn[1] @ hn[1])
    bits["l0.mix.q"] = bf16_bits(wq.reshape(-1, d))
    w["l0.mix.q"] = bf16_values(bits["l0.mix.q"])
    m = model(s, bits, dtype=dtype, n_positions=400)
    rng = np.random.default_rng(8)
    base = rng.integers(10, s["vocab"], 330).astype(np.uint32)
    for place in (0, 1, 30, 31, 32, 33, 62, 63, 64, 65, 127, 128, 191, 192, 255, 256, 300, 318, 319, 320):
        t = base.copy()
        t[place], t[-1] = 7, 9
        want = plain.forward(t, s, w)[-1:]
        t2 = base.copy()
        t2[-1] = 9
        if place == 30:  # the needle matters
            assert row_errors(plain.forward(t2, s, w)[-1:], want)[0] > 0.2
        for sizes in ([330], [329, 1], [310, 20]):
            e = row_errors(feed(m, t, sizes)[-1:], want)[0]
            assert e <= {"float32": 2e-4, "bfloat16": 0.08}[dtype], (place, sizes, e)


def test_sink_counts_once_and_unscaled():
    s = spec(48, 40, [latent(heads=4, ff=0, scale=0.05)])
    bits, w = random_tensors(s, 9)
    big = np.array([3.0, -2.0, 5.0, 0.0])
    bits["l0.mix.sink"], w["l0.mix.sink"] = bf16_bits(big), bf16_values(bf16_bits(big))
    t = tokens_of(s, 40)
    want = plain.forward(t, s, w)
    none = dict(w)
    none["l0.mix.sink"] = np.full(4, -1e30)
    assert row_errors(plain.forward(t, s, none), want).max() > 0.1
    for dtype in DTYPES:
        m = model(s, bits, dtype=dtype, n_positions=64)
        for sizes in ([40], [1], [20, 1]):
            check_rows(feed(m, t, sizes), want, dtype, f"{dtype} {sizes}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("B", [2, 3, 5, 17, 33])
def test_batch_against_each_alone(B, dtype):
    """Unequal requests of equal length side by side, prompt, portion and decoding, against the plain model."""
    s = SPECS["mixed"]
    bits, w = random_tensors(s, 10)
    m = model(s, bits, dtype=dtype, n_positions=64, max_batch=B)
    t = np.random.default_rng(B).integers(0, s["vocab"], (B, 40)).astype(np.uint32)
    m.reset_cache()
    got = [m.forward_cached(t[:, :30]), m.forward_cached(t[:, 30:35])] + [m.forward_cached(t[:, i:i + 1]) for i in range(35, 40)]
    got = np.concatenate(got, axis=1)
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


def test_long_decoding_keeps_the_state():
    """300 tokens decoded one at a time behind a prompt of 5 (fp32), with decays close to one."""
    s = spec(48, 60, [delta(heads=2, kv_heads=1, dim=24, vdim=16, ff=0), latent(heads=2, ff=0)], loop=dict(start=0, stop=1, times=2))
    bits, w = random_tensors(s, 12)
    m = model(s, bits, dtype="float32", n_positions=320)
    t = tokens_of(s, 305)
    check_rows(feed(m, t, [5, 1]), plain.forward(t, s, w), "float32")


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_keys(dtype):
    """4500 keys: several chunks per split of the decode kernel, long rows of the tiled one."""
    s, bits, w = sharp_attention(13, scale=1.0)
    t = tokens_of(s, 4506)
    want = plain.forward(t, s, w)[-6:]
    m = model(s, bits, dtype=dtype, n_positions=4608)
    m.reset_cache()
    m.forward_cached(t[:3000].reshape(1, -1), all_rows=False)
    m.forward_cached(t[3000:4500].reshape(1, -1), all_rows=False)
    got = np.concatenate([m.forward_cached(t[i:i + 1].reshape(1, -1))[0] for i in range(4500, 4506)])
    e = row_errors(got, want)
    assert e.max() <= {"float32": 2e-4, "bfloat16": 0.1}[dtype], e


def test_wide_latent_without_matrix_kernel():
    """A latent too wide for the matrix-core decode kernel (bf16 cache, fp32 FMAs)."""
    s = spec(64, 50, [latent(heads=3, dim=16, rot=8, vdim=24, rank=900, ff=0)])
    bits, w = random_tensors(s, 14)
    m = model(s, bits, dtype="bfloat16", n_positions=128)
    t = tokens_of(s, 100)
    check_rows(feed(m, t, [40, 1, 7]), plain.forward(t, s, w), "bfloat16")


def test_wide_heads_without_tiled_kernel():
    """Heads too wide for the tiled prompt kernel take the absorbed form for prompts too."""
    s = spec(64, 50, [latent(heads=2, dim=200, rot=16, vdim=136, rank=96, ff=0)])
    bits, w = random_tensors(s, 15)
    t = tokens_of(s, 90)
    for dtype in DTYPES:
        m = model(s, bits, dtype=dtype, n_positions=128)
        check_rows(feed(m, t, [64, 1]), plain.forward(t, s, w), dtype)


def test_tiled_kernel_with_and_without_a_key_split():
    """Enough query blocks that every wave takes one of its own, against the same rows with the keys split over waves."""
    s = spec(64, 50, [latent(heads=16, dim=16, rot=16, vdim=32, rank=64, ff=0)])
    bits, _ = random_tensors(s, 16)
    t = np.random.default_rng(1).integers(0, 50, (5, 900)).astype(np.uint32)
    m = model(s, bits, dtype="bfloat16", n_positions=900, max_batch=5)
    m.reset_cache()
    many = m.forward_cached(t)
    for b in (0, 4):
        m.reset_cache()
        one = m.forward_cached(t[b:b + 1])[0]
        assert row_errors(many[b], one.astype(np.float64)).max() <= 2e-2


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
    bits, w = random_tensors(s, 17)
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
    # every drawn token is one of the ten best of its step
    lg = m.forward(a[:-1])
    for i in range(len(prompt), len(a)):
        assert a[i] in np.argsort(-lg[i - 1])[:10]


def test_errors_are_raised_on_the_host():
    from async_gpu_amd import _lib, ritevik, weights
    s = SPECS["one_pass"]
    bits, _ = random_tensors(s, 20)
    with pytest.raises(weights.ModelFileError, match="l1.mix.uk"):
        model(s, {k: v for k, v in bits.items() if k != "l1.mix.uk"})
    with pytest.raises(weights.ModelFileError, match="expected shape"):
        model(s, dict(bits, **{"embed.norm": bits["embed.norm"][:-1]}))
    m = model(s, bits, n_positions=16)
    with pytest.raises(_lib.AgpuError) as e:
        m.forward_cached(np.zeros((1, 17), np.uint32))
    assert e.value.code == _lib.ERR_DIM_OUT_OF_RANGE
    with pytest.raises(_lib.AgpuError) as e:
        m.generate_cached(np.array([s["vocab"]], np.uint32), 2)
    assert e.value.code == _lib.ERR_DIM_OUT_OF_RANGE
    with pytest.raises(_lib.AgpuError) as e:
        m.set_tensor("l9.norm1", bits["l0.norm1"])
    assert e.value.code == _lib.ERR_KERNEL_NOT_FOUND
    bare = ritevik.RitevikModel(ritevik.RitevikConfig(s, [(32, 32), None]))
    with pytest.raises(_lib.AgpuError, match="embed"):
        bare.forward_cached(np.zeros((1, 1), np.uint32))
    bad = copy.deepcopy(s)
    bad["layers"][0]["mixer"]["kv_heads"] = 3
    with pytest.raises(_lib.AgpuError):
        ritevik.RitevikModel(ritevik.RitevikConfig(bad, [(32, 32), None]))


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
