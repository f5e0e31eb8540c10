"""Small Ritevik configurations and random weights for the tests."""
import numpy as np


def bf16_bits(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_values(bits):
    return (bits.astype(np.uint32) << 16).view(np.float32).astype(np.float64)


def latent(heads=3, dim=24, rot=16, vdim=40, rank=72, scale=None, base=10000.0, ff=80):
    return dict(type="latent_attention", mlp=dict(kind="dense", ff=ff) if ff else None,
                mixer=dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=rank, scale=scale or (dim + rot) ** -0.5,
                           rot=dict(base=base, dims=rot)))


def delta(heads=6, kv_heads=2, dim=20, vdim=28, conv=4, ff=104, ranks=(12, 20)):
    return dict(type="channel_delta", mlp=dict(kind="dense", ff=ff) if ff else None, ranks=ranks,
                mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv))


def spec(width, vocab, layers, loop=None, side=None, eps=1e-5):
    return dict(architecture="Ritevik", width=width, vocab=vocab, norm=dict(eps=eps), layers=layers, loop=loop,
                token_side=dict(dim=side) if side else None)


SPECS = {
    # every mechanism, sizes off the multiples of 32, layers before, in and behind the loop
    "mixed": spec(100, 131, [latent(), delta(), delta(heads=2, kv_heads=2, dim=36, vdim=12, conv=2, ff=0), latent(heads=1, dim=8, rot=24, vdim=32, rank=40, ff=48),
                             delta(heads=3, kv_heads=1, dim=16, vdim=44, conv=3, ranks=(40, 8))],
                  loop=dict(start=1, stop=4, times=3), side=12),
    # no loop, no side input, one head, five taps (more than the fast path keeps in registers), attention without feed-forward
    "plain": spec(72, 97, [delta(heads=1, kv_heads=1, dim=64, vdim=96, conv=5, ff=33, ranks=(7, 70)), latent(heads=5, dim=64, rot=32, vdim=64, rank=160, ff=0)]),
    # a loop of one pass from the first layer on, one tap, a side input wider than 32
    "one_pass": spec(64, 50, [delta(heads=4, kv_heads=4, dim=32, vdim=32, conv=1, ff=64, ranks=(32, 32)), latent(heads=4, dim=32, rot=8, vdim=16, rank=64)],
                     loop=dict(start=0, stop=2, times=1), side=40, eps=1e-6),
    # heads and ranks of a larger model: low-rank sizes above 128, more than 256 low-rank rows, 160-wide keys
    "wide": spec(160, 61, [delta(heads=2, kv_heads=1, dim=160, vdim=200, conv=4, ff=64, ranks=(150, 260)), latent(heads=18, dim=40, rot=20, vdim=72, rank=520, ff=64)],
                 loop=dict(start=1, stop=2, times=2)),
}


def random_tensors(s, seed, memory=True):
    """({name: uint16 bits}, {name: float64 values}).  memory: decays close to one, so that lost state shows late."""
    rng = np.random.default_rng(seed)
    bits = {}

    def put(name, a):
        bits[name] = bf16_bits(a)

    def mat(name, rows, cols, gain=1.0):
        put(name, rng.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def vec(name, shape, centre=0.0, spread=0.2):
        put(name, centre + spread * rng.standard_normal(shape))

    d, V, L = s["width"], s["vocab"], len(s["layers"])
    put("embed", rng.standard_normal((V, d)))
    vec("embed.norm", d)
    if s["loop"]:
        mat("loop.in", d, 2 * d)
        vec("loop.step", (s["loop"]["times"], d), spread=0.5)
    side = s["token_side"]["dim"] if s["token_side"] else 0
    if side:
        put("side.embed", rng.standard_normal((V, L * side)))
    for i, e in enumerate(s["layers"]):
        p, m = f"l{i}.", e["mixer"]
        H, D, DV = m["heads"], m["dim"], m["vdim"]
        vec(p + "norm1", d)
        if e["type"] == "latent_attention":
            R, C = m["rot_dim"], m["kv_rank"]
            mat(p + "mix.q", H * (D + R), d, 1.5)
            mat(p + "mix.dkv", C + R, d, 1.5)
            vec(p + "mix.dkv.norm", C, 1.0)
            mat(p + "mix.uk", H * D, C)
            mat(p + "mix.uv", H * DV, C)
            vec(p + "mix.sink", H, 0.5, 1.0)
        else:
            ra, rg = e["ranks"]
            for t, ch in (("q", m["kv_heads"] * D), ("k", m["kv_heads"] * D), ("v", H * DV)):
                mat(p + "mix." + t, ch, d)
                vec(p + f"mix.{t}.conv", (ch, m["conv"]), 0.0, 0.7)
            mat(p + "mix.b", H, d)
            vec(p + "mix.A_log", H, -1.0 if memory else 0.5, 0.5)
            put(p + "mix.dt_bias", rng.uniform(-7.0, -1.0, H * D) if memory else rng.uniform(-2.0, 1.0, H * D))
            mat(p + "mix.a1", ra, d)
            mat(p + "mix.a2", H * D, ra)
            mat(p + "mix.g1", rg, d)
            mat(p + "mix.g2", H * DV, rg)
            vec(p + "mix.norm", DV, 1.0)
        mat(p + "mix.o", d, H * DV)
        if e["mlp"]:
            ff = e["mlp"]["ff"]
            mat(p + "mlp.gate", ff, d)
            mat(p + "mlp.up", ff, d)
            mat(p + "mlp.down", d, ff)
        if side:
            mat(p + "side.gate", side, d)
            mat(p + "side.proj", d, side)
            vec(p + "side.norm", d, 0.4)
    vec("final.norm", d)
    mat("head", V, d)
    return bits, {k: bf16_values(v) for k, v in bits.items()}


def model(s, bits, **kw):
    """The library's model of a configuration and its bf16 bits."""
    from async_gpu_amd import ritevik
    return ritevik.RitevikModel.from_tensors(s, {k: ("BF16", v) for k, v in bits.items()}, **kw)


def row_errors(got, want):
    """Per position: rms over the vocabulary of the difference (mean taken off), over the rms of the expected logits."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    scale = np.sqrt(np.mean((want - want.mean(-1, keepdims=True)) ** 2))
    return np.sqrt(np.mean(d * d, axis=-1)) / scale


LIMIT = {"float32": 1e-4, "bfloat16": 5e-2}


def check_rows(got, want, dtype, what=""):
    """In bf16 single positions of a random model magnify the rounding: nine in ten stay within the limit, none beyond four
    times that."""
    e = row_errors(got, want)
    bf16 = dtype == "bfloat16"
    bad = e.max() > (4 if bf16 else 1) * LIMIT[dtype] or (bf16 and e.size >= 10 and np.quantile(e, 0.9) > LIMIT[dtype])
    assert np.isfinite(e).all() and not bad, \
        f"{what}: worst position {int(e.argmax())}, error {e.max():.2e}, nine in ten within {np.quantile(e, 0.9):.2e} (limit {LIMIT[dtype]:.0e})"
