"""Small Piralix configurations and random weights for the tests."""
import numpy as np

from ritevik_cases import bf16_bits, bf16_values


def ff_of(ff, limit):
    return dict(kind="dense", ff=ff, limit=limit) if ff else None


def mlstm(heads=3, dim=20, vdim=28, cap=9.0, ff=0, limit=0.8):
    return dict(type="mlstm", mlp=ff_of(ff, limit), mixer=dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap))


STRETCH = dict(factor=4.0, fast=24.0, slow=1.5, original=64)


def attention(heads=6, kv_heads=2, dim=24, vdim=40, rot=16, base=5000.0, scaling=STRETCH, scale=None, softcap=20.0, ff=0, limit=1.3):
    return dict(type="attention", mlp=ff_of(ff, limit),
                mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale or dim ** -0.5, softcap=softcap,
                           rot=dict(base=base, dims=rot, scaling=scaling)))


def rglru(width=84, blocks=3, conv=4, ff=0, limit=1.0):
    return dict(type="rglru", mlp=ff_of(ff, limit), mixer=dict(width=width, blocks=blocks, conv=conv))


def spec(width, vocab, layers, loop=None, eps=1e-5):
    return dict(architecture="Piralix", width=width, vocab=vocab, norm=dict(eps=eps), layers=layers, loop=loop)


SPECS = {
    # every mechanism, sizes off the multiples of 32, layers before, in and behind the loop
    "mixed": spec(100, 131, [attention(ff=80), mlstm(ff=56), rglru(), attention(heads=2, kv_heads=2, dim=10, vdim=12, rot=10, softcap=3.0), mlstm(heads=2, dim=36, vdim=12),
                             rglru(width=40, blocks=2, conv=2, ff=33)], loop=dict(start=1, stop=4, times=3)),
    # no loop, one block, five taps (more than the fast path keeps in registers), one head, plain rotation
    "plain": spec(72, 97, [rglru(width=50, blocks=1, conv=5), mlstm(heads=1, dim=64, vdim=96, ff=40), attention(heads=5, kv_heads=1, dim=64, vdim=64, rot=32, scaling=None)]),
    # a loop of one pass from the first layer on, one tap, more heads per key head than a tile has columns, no rotation
    "one_pass": spec(64, 50, [rglru(width=64, blocks=2, conv=1, ff=64), attention(heads=20, kv_heads=1, dim=32, vdim=16, rot=0), mlstm(heads=4, dim=32, vdim=32)],
                     loop=dict(start=0, stop=2, times=1), eps=1e-6),
    # heads and blocks of a larger model
    "wide": spec(160, 61, [mlstm(heads=2, dim=150, vdim=330), attention(heads=3, kv_heads=3, dim=160, vdim=200, rot=64, ff=64), rglru(width=600, blocks=2, ff=48)],
                 loop=dict(start=1, stop=3, times=2)),
}


def random_tensors(s, seed):
    """({name: uint16 bits}, {name: float64 values}).  Forget gates and decays lie close to one, so that lost state shows late."""
    rng = np.random.default_rng(seed)
    bits = {}

    def put(name, a):
        bits[name] = bf16_bits(a)

    def mat(name, rows, cols, gain=1.0):
        put(name, rng.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def vec(name, shape, centre=0.0, spread=0.2):
        put(name, centre + spread * rng.standard_normal(shape))

    d, V = s["width"], s["vocab"]
    put("embed", 0.4 * rng.standard_normal((V, d)))  # faint beside what the layers add: they decide the logits
    if s["loop"]:
        vec("loop.step", (s["loop"]["times"], d), spread=0.5)
    for i, e in enumerate(s["layers"]):
        p, m = f"l{i}.", e["mixer"]
        q = p + "mix."
        vec(p + "norm1", d, 1.0)
        vec(p + "norm1b", d, 1.2)
        if e["type"] == "mlstm":
            H, D, DV = m["heads"], m["dim"], m["vdim"]
            # a query leans towards its own key: the head norm would magnify the rounding of a first read-out k . q near zero
            k, n = rng.standard_normal((2, H * D, d)) / np.sqrt(d)
            put(q + "q", 0.9 * k + 1.2 * n)
            put(q + "k", k)
            mat(q + "v", H * DV, d)
            mat(q + "g", H * DV, d)
            vec(q + "norm", H * DV, 1.0)
            mat(q + "i", H, d)
            vec(q + "i.b", H, 0.0, 1.0)
            mat(q + "f", H, d)
            put(q + "f.b", rng.uniform(2.0, 7.0, H))
            mat(q + "o", d, H * DV)
        elif e["type"] == "attention":
            H, G, D, DV = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            mat(q + "q", H * D, d, 1.5)
            mat(q + "k", G * D, d, 1.5)
            mat(q + "v", G * DV, d)
            mat(q + "g", H * DV, d)
            vec(q + "sink", H, 0.5, 1.0)
            mat(q + "o", d, H * DV)
        else:
            W, B = m["width"], m["blocks"]
            for t in "yx":
                mat(q + t, W, d)
                vec(q + t + ".b", W)
            vec(q + "conv", (W, m["conv"]), 0.0, 0.7)
            vec(q + "conv.b", W)
            for t in ("ra", "ri"):
                put(q + t, rng.standard_normal((B, W // B, W // B)) / np.sqrt(W // B))
                vec(q + t + ".b", (B, W // B), spread=0.5)
            vec(q + "lam", W, -4.0, 2.0)
            mat(q + "o", d, W)
        if e["mlp"]:
            ff = e["mlp"]["ff"]
            vec(p + "norm2", d, 1.0)
            vec(p + "norm2b", d, 1.2)
            mat(p + "mlp.gate", ff, d, 1.5)
            mat(p + "mlp.up", ff, d, 1.5)
            mat(p + "mlp.down", d, ff)
    vec("final.norm", d, 1.0)
    return bits, {k: bf16_values(v) for k, v in bits.items()}


def model(s, bits, **kw):
    """The library's model of a configuration and its bf16 bits."""
    from async_gpu_amd import piralix
    return piralix.PiralixModel.from_tensors(s, {k: ("BF16", v) for k, v in bits.items()}, **kw)
