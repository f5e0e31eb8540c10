"""Synthetic inputs of the benchmark configurations (numpy, seeded; identical on every machine
with the same numpy).  Nibble packing follows nn/ops/quantize.rs:133-148."""
import numpy as np


def pack_nibbles(q):
    """q [K,N] ints in [-8,7] -> packed [K/8,N] u32 (nibble i of word kp = q[8kp+i]+8)."""
    K, N = q.shape
    assert K % 8 == 0
    u = (q.astype(np.int64) + 8).astype(np.uint32).reshape(K // 8, 8, N)
    packed = np.zeros((K // 8, N), np.uint32)
    for i in range(8):
        packed |= u[:, i, :] << np.uint32(4 * i)
    return packed


def random_int4_linear(rng, K, N, group=32, bias=False):
    """Weights: int4 uniform in [-8,7]; scales U(0.002,0.02) per (group, column)."""
    q = rng.integers(-8, 8, size=(K, N))
    packed = pack_nibbles(q)
    scales = rng.uniform(0.002, 0.02, size=((K + group - 1) // group, N)).astype(np.float32)
    b = rng.standard_normal(N).astype(np.float32) * 0.1 if bias else None
    return packed, scales, b


def config1_gemv(seed=0, M=1, K=768, N=3072, group=32):
    """Single int4 dequant-GEMV, the GPT-2 MLP fc shape."""
    rng = np.random.default_rng(seed)
    packed, scales, _ = random_int4_linear(rng, K, N, group)
    x = rng.standard_normal((M, K)).astype(np.float32)
    return dict(x=x, packed=packed, scales=scales, group=group)


def config2_gemm(seed=1, M=128, K=768, N=2304, group=32):
    """Batched int4 dequant-GEMM, the prefill QKV projection."""
    return config1_gemv(seed, M, K, N, group)


def config3_attention(seed=2, H=12, seq=1024, d_head=64):
    """Q,K,V ~ N(0,1)/sqrt(64), head-major [H,seq,64]."""
    rng = np.random.default_rng(seed)
    s = np.float32(1.0 / np.sqrt(d_head))
    q, k, v = (rng.standard_normal((H, seq, d_head)).astype(np.float32) * s for _ in range(3))
    return dict(q=q, k=k, v=v)


GPT2_SMALL = dict(n_layer=12, n_embd=768, n_head=12, vocab=50257, n_positions=1024)
GPT2_XL = dict(n_layer=48, n_embd=1600, n_head=25, vocab=50257, n_positions=1024)
GPT2_TINY = dict(n_layer=2, n_embd=128, n_head=2, vocab=503, n_positions=64)


def gpt2_fp32_weights(cfg, seed, std=0.02, nonzero_bias=False, random_ln=False):
    """Random-init GPT-2: every Linear weight, wte, wpe ~ N(0, std); LN gain 1 / bias 0 and
    Linear biases 0 unless asked otherwise.  Linear weights are Conv1D [in, out] = the int4
    [K, N] matrix (gpt2.rs:1383, 1154: the two transposes cancel)."""
    rng = np.random.default_rng(seed)
    d, ff, V, P = cfg["n_embd"], 4 * cfg["n_embd"], cfg["vocab"], cfg["n_positions"]

    def nrm(*shape):
        return (rng.standard_normal(shape, dtype=np.float32) * np.float32(std))

    def bias(n):
        return nrm(n) if nonzero_bias else np.zeros(n, np.float32)

    def ln():
        if random_ln:
            return (1.0 + 0.1 * rng.standard_normal(d)).astype(np.float32), (0.1 * rng.standard_normal(d)).astype(np.float32)
        return np.ones(d, np.float32), np.zeros(d, np.float32)

    w = dict(wte=nrm(V, d), wpe=nrm(P, d), layers=[])
    for _ in range(cfg["n_layer"]):
        g1, b1 = ln()
        g2, b2 = ln()
        w["layers"].append(dict(
            ln1_g=g1, ln1_b=b1, ln2_g=g2, ln2_b=b2,
            qkv_w=nrm(d, 3 * d), qkv_b=bias(3 * d), proj_w=nrm(d, d), proj_b=bias(d),
            fc_w=nrm(d, ff), fc_b=bias(ff), fc_proj_w=nrm(ff, d), fc_proj_b=bias(d)))
    w["lnf_g"], w["lnf_b"] = ln()
    return w


LINEAR_NAMES = ("qkv", "proj", "fc", "fc_proj")


def quantize_gpt2(weights, group, quantize_fn, lm_head_int4=True):
    """Quantize every Linear with quantize_fn(weight_t [K,N], group) -> (packed, scales).
    The tied LM head is wte^T [K=d, N=vocab]."""
    q = dict(group=group, wte=weights["wte"], wpe=weights["wpe"], lnf_g=weights["lnf_g"], lnf_b=weights["lnf_b"],
             layers=[], lm_head=None)
    for L in weights["layers"]:
        e = {k: L[k] for k in ("ln1_g", "ln1_b", "ln2_g", "ln2_b")}
        for name in LINEAR_NAMES:
            packed, scales = quantize_fn(L[name + "_w"], group)
            e[name] = (packed, scales, L[name + "_b"])
        q["layers"].append(e)
    if lm_head_int4:
        q["lm_head"] = quantize_fn(np.ascontiguousarray(weights["wte"].T), group)
    return q


def gpt2_quantized_layerwise(cfg, seed, group, quantize_fn, std=0.02, workers=8):
    """The dict of quantize_gpt2 for a random-init GPT-2 (weights, wte, wpe ~ N(0, std); LN gain 1, every bias 0),
    built one layer at a time by a pool of threads, so that a model of XL size never holds its 6 GB of fp32 weights
    at once and does not take minutes to draw.  Layer L draws from its own generator seeded (seed, L), the embeddings
    from (seed, n_layer): the values differ from gpt2_fp32_weights(cfg, seed)."""
    from concurrent.futures import ThreadPoolExecutor
    d, ff, V, P, nl = cfg["n_embd"], 4 * cfg["n_embd"], cfg["vocab"], cfg["n_positions"], cfg["n_layer"]

    def layer(L):
        rng = np.random.default_rng([seed, L])
        e = dict(ln1_g=np.ones(d, np.float32), ln1_b=np.zeros(d, np.float32), ln2_g=np.ones(d, np.float32),
                 ln2_b=np.zeros(d, np.float32))
        for name, (k, n) in zip(LINEAR_NAMES, ((d, 3 * d), (d, d), (d, ff), (ff, d))):
            w = rng.standard_normal((k, n), dtype=np.float32) * np.float32(std)
            packed, scales = quantize_fn(w, group)
            e[name] = (packed, scales, np.zeros(n, np.float32))
        return e

    with ThreadPoolExecutor(max_workers=workers) as pool:
        layers = list(pool.map(layer, range(nl)))
    rng = np.random.default_rng([seed, nl])
    wte = rng.standard_normal((V, d), dtype=np.float32) * np.float32(std)
    wpe = rng.standard_normal((P, d), dtype=np.float32) * np.float32(std)
    return dict(group=group, wte=wte, wpe=wpe, lnf_g=np.ones(d, np.float32), lnf_b=np.zeros(d, np.float32), layers=layers,
                lm_head=quantize_fn(np.ascontiguousarray(wte.T), group))


def random_prompt(cfg, seed, length, batch=None):
    rng = np.random.default_rng(seed + 1000)
    shape = (length,) if batch is None else (batch, length)
    return rng.integers(0, cfg["vocab"], size=shape).astype(np.uint32)


# Ritevik shapes of the size of a real model's layers, beside the GPT-2 of the same width and number of layer runs.
# Three delta layers per attention layer; the middle third of the small one runs twice.
def ritevik_spec(width, heads, head_dim, rot_dim, kv_rank, ff, n_layer, vocab, side_dim, loop=None):
    latent = dict(type="latent_attention", mlp=dict(kind="dense", ff=ff),
                  mixer=dict(heads=heads, dim=head_dim, rot_dim=rot_dim, vdim=head_dim, kv_rank=kv_rank, scale=(head_dim + rot_dim) ** -0.5,
                             rot=dict(base=10000.0, dims=rot_dim)))
    delta = dict(type="channel_delta", mlp=dict(kind="dense", ff=ff),
                 mixer=dict(heads=heads, kv_heads=heads, dim=head_dim, vdim=head_dim, conv=4))
    return dict(architecture="Ritevik", width=width, vocab=vocab, norm=dict(eps=1e-6), token_side=dict(dim=side_dim) if side_dim else None, loop=loop,
                layers=[latent if i % 4 == 3 else delta for i in range(n_layer)])


RITEVIK_SMALL = ritevik_spec(768, 12, 64, 32, 256, 3072, 8, 50257, 64, loop=dict(start=2, stop=6, times=2))  # 12 layer runs
RITEVIK_LARGE = ritevik_spec(2048, 16, 128, 64, 512, 8192, 24, 50257, 128)


class _Draw:
    """Random bf16 weights by name.  Matrices are cut from one pool of N(0, 1) values scaled to 1 / sqrt(K), so a model of billions of
    weights takes seconds."""

    def __init__(self, seed):
        self.rng = np.random.default_rng(seed)
        self.pool = self.rng.standard_normal(1 << 22, dtype=np.float32)
        self.out = {}

    def mat(self, name, rows, cols, gain=1.0):
        from .weights import f32_to_bf16
        n, lo = rows * cols, int(self.rng.integers(0, self.pool.size))
        base = f32_to_bf16(np.roll(self.pool, -lo)[: min(n, self.pool.size)] * np.float32(gain / np.sqrt(cols)))
        self.out[name] = ("BF16", np.resize(base, (rows, cols)))

    def vec(self, name, shape, centre=0.0, spread=0.1):
        from .weights import f32_to_bf16
        self.out[name] = ("BF16", f32_to_bf16((centre + spread * self.rng.standard_normal(shape)).astype(np.float32)))


def ritevik_tensors(spec, seed, rank=None):
    """{name: (dtype, array)} of random bf16 weights; `rank` is the low-rank size of the delta layers (default: head dim)."""
    draw = _Draw(seed)
    mat, vec, out = draw.mat, draw.vec, draw.out
    d, V, n_layer = spec["width"], spec["vocab"], len(spec["layers"])
    mat("embed", V, d, np.sqrt(d))
    vec("embed.norm", d)
    if spec.get("loop"):
        mat("loop.in", d, 2 * d)
        vec("loop.step", (spec["loop"]["times"], d))
    side = (spec.get("token_side") or {}).get("dim", 0)
    if side:
        mat("side.embed", V, n_layer * side, np.sqrt(n_layer * side))
    for i, e in enumerate(spec["layers"]):
        p, m = f"l{i}.", e["mixer"]
        H, D, DV = m["heads"], m["dim"], m["vdim"]
        vec(p + "norm1", d)
        if e["type"] == "latent_attention":
            R, Ck = m["rot_dim"], m["kv_rank"]
            mat(p + "mix.q", H * (D + R), d)
            mat(p + "mix.dkv", Ck + R, d)
            vec(p + "mix.dkv.norm", Ck, 1.0)
            mat(p + "mix.uk", H * D, Ck)
            mat(p + "mix.uv", H * DV, Ck)
            vec(p + "mix.sink", H, 0.0, 1.0)
        else:
            r = rank or D
            for t, ch in (("q", m["kv_heads"] * D), ("k", m["kv_heads"] * D), ("v", H * DV)):
                mat(p + "mix." + t, ch, d)
                vec(p + f"mix.{t}.conv", (ch, m["conv"]), 0.0, 0.6)
            mat(p + "mix.b", H, d)
            vec(p + "mix.A_log", H, 0.0, 0.5)
            vec(p + "mix.norm", DV, 1.0)
            mat(p + "mix.a1", r, d)
            mat(p + "mix.a2", H * D, r)
            vec(p + "mix.dt_bias", H * D, -2.0, 1.0)
            mat(p + "mix.g1", r, d)
            mat(p + "mix.g2", H * DV, r)
        mat(p + "mix.o", d, H * DV, 0.3)
        if e.get("mlp"):
            ff = e["mlp"]["ff"]
            mat(p + "mlp.gate", ff, d)
            mat(p + "mlp.up", ff, d)
            mat(p + "mlp.down", d, ff, 0.5)
        if side:
            mat(p + "side.gate", side, d)
            mat(p + "side.proj", d, side)
            vec(p + "side.norm", d, 0.2)
    vec("final.norm", d)
    mat("head", V, d)
    return out


def piralix_spec(width, heads, kv_heads, head_dim, memory_heads, lru_blocks, ff, n_layer, vocab, loop=None):
    """Two matrix memories, an attention and a gated recurrent layer in turn, each with a feed-forward; the memory's values take the
    full width, its keys half of it."""
    mlp = dict(kind="dense", ff=ff, limit=7.0)
    vdim = width // memory_heads
    memory = dict(type="mlstm", mlp=mlp, mixer=dict(heads=memory_heads, dim=vdim // 2, vdim=vdim, gate_cap=15.0))
    attend = dict(type="attention", mlp=mlp, mixer=dict(heads=heads, kv_heads=kv_heads, dim=head_dim, vdim=head_dim, scale=head_dim ** -0.5, softcap=30.0,
                                                        rot=dict(base=500000.0, dims=head_dim, scaling=dict(factor=4.0, fast=16.0, slow=2.0, original=8192))))
    lru = dict(type="rglru", mlp=mlp, mixer=dict(width=width, blocks=lru_blocks, conv=4))
    return dict(architecture="Piralix", width=width, vocab=vocab, norm=dict(eps=1e-6), loop=loop,
                layers=[(memory, attend, memory, lru)[i % 4] for i in range(n_layer)])


PIRALIX_SMALL = piralix_spec(768, 12, 4, 64, 6, 12, 3072, 8, 50257, loop=dict(start=2, stop=6, times=2))  # 12 layer runs
PIRALIX_LARGE = piralix_spec(2048, 16, 4, 128, 8, 16, 8192, 24, 50257)


def piralix_tensors(spec, seed):
    """{name: (dtype, array)} of random bf16 weights."""
    draw = _Draw(seed)
    mat, vec, out = draw.mat, draw.vec, draw.out
    d, V = spec["width"], spec["vocab"]
    mat("embed", V, d, np.sqrt(d))
    if spec.get("loop"):
        vec("loop.step", (spec["loop"]["times"], d))
    for i, e in enumerate(spec["layers"]):
        p, m = f"l{i}.", e["mixer"]
        q = p + "mix."
        vec(p + "norm1", d, 1.0)
        vec(p + "norm1b", d, 0.5)
        if e["type"] == "mlstm":
            H, nk, nv = m["heads"], m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for t, n in (("q", nk), ("k", nk), ("v", nv), ("g", nv), ("i", H), ("f", H)):
                mat(q + t, n, d)
            vec(q + "norm", nv, 1.0)
            vec(q + "i.b", H)
            vec(q + "f.b", H, 4.0, 1.0)
            mat(q + "o", d, nv)
        elif e["type"] == "attention":
            H, G, D, DV = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for t, n in (("q", H * D), ("k", G * D), ("v", G * DV), ("g", H * DV)):
                mat(q + t, n, d)
            vec(q + "sink", H, 0.0, 1.0)
            mat(q + "o", d, H * DV)
        else:
            W, B = m["width"], m["blocks"]
            for t in "yx":
                mat(q + t, W, d)
                vec(q + t + ".b", W)
            vec(q + "conv", (W, m["conv"]), 0.0, 0.6)
            vec(q + "conv.b", W)
            for t in ("ra", "ri"):
                mat(q + t, W, W // B)
                out[q + t] = ("BF16", out[q + t][1].reshape(B, W // B, W // B))
                vec(q + t + ".b", (B, W // B))
            vec(q + "lam", W, -4.0, 1.0)
            mat(q + "o", d, W)
        if e.get("mlp"):
            ff = e["mlp"]["ff"]
            vec(p + "norm2", d, 1.0)
            vec(p + "norm2b", d, 0.5)
            mat(p + "mlp.gate", ff, d)
            mat(p + "mlp.up", ff, d)
            mat(p + "mlp.down", d, ff)
    vec("final.norm", d, 1.0)
    return out
