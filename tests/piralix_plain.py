"""Plain Piralix forward in numpy, one function per mechanism, token by token where a mechanism recurs.  Test
infrastructure only: it shares nothing with the library.  Everything runs in the dtype of the weights it is given
(float64 in the tests)."""
import numpy as np

from ritevik_plain import gelu_tanh, part, rms_norm, sigmoid, softplus


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


# ---- matrix memory with exponential gates ----

def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def matrix_memory_recurrence(q, k, v, i, f):
    """q, k [T, H, D], v [T, H, DV], log gates i, f [T, H] -> o [T, H, DV].  Per head: a state S [D, DV], a normaliser n [D] and
    a running maximum of the log gates that keeps the exponentials bounded."""
    T, H, D = q.shape
    o = np.zeros_like(v)
    for hd in range(H):
        S, n, m = np.zeros((D, v.shape[2]), q.dtype), np.zeros(D, q.dtype), 0.0
        for t in range(T):
            top = max(f[t, hd] + m, i[t, hd])
            keep, take = np.exp(f[t, hd] + m - top), np.exp(i[t, hd] - top)
            m = top
            S = keep * S + take * np.outer(k[t, hd], v[t, hd])
            n = keep * n + take * k[t, hd]
            o[t, hd] = (S.T @ q[t, hd]) / (max(abs(n @ q[t, hd]), np.exp(-m)) + 1e-6)
    return o


def mlstm(h, w, m, eps):
    """h [T, width] -> [T, width]; w: the mixer's tensors by short name, m: its sizes and constants."""
    T, H, D, DV, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ w["q"].T).reshape(T, H, D) / np.sqrt(D)
    k = (h @ w["k"].T).reshape(T, H, D)
    v = (h @ w["v"].T).reshape(T, H, DV)
    i = soft_cap(h @ w["i"].T + w["i.b"], cap)
    f = log_sigmoid(soft_cap(h @ w["f"].T + w["f.b"], cap))
    o = rms_norm(matrix_memory_recurrence(q, k, v, i, f), 1.0, eps).reshape(T, H * DV)
    return (o * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T


# ---- attention: grouped heads, turned pairs of neighbours, capped scores, sink, gate ----

def frequencies(rot):
    """Angle per position of every pair; with scaling, slow pairs turn `factor` times slower and a ramp lies between."""
    dims, base = rot["dims"], float(rot["base"])
    i = np.arange(dims // 2)
    f = base ** (-2.0 * i / dims)
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def pair_that_turns(t):
        return dims * np.log(s["original"] / (2.0 * np.pi * t)) / (2.0 * np.log(base))
    lo = max(np.floor(pair_that_turns(s["fast"])), 0)
    hi = min(np.ceil(pair_that_turns(s["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * np.log(s["factor"]) + 1.0


def rotate_pairs(x, positions, rot):
    """x [T, heads, dim]: dimension 2 i turns with dimension 2 i + 1 over the first rot dims; the rest stays."""
    f, stretch = frequencies(rot)
    a = (np.asarray(positions, np.float64)[:, None] * f[None, :])[:, None, :]
    c, s = np.cos(a) * stretch, np.sin(a) * stretch
    y = x.copy()
    u, v = x[..., 0:rot["dims"]:2], x[..., 1:rot["dims"]:2]
    y[..., 0:rot["dims"]:2] = u * c - v * s
    y[..., 1:rot["dims"]:2] = v * c + u * s
    return y


def attention(h, w, m, eps):
    T, H, G, D, DV = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = np.arange(T)
    q = rotate_pairs((h @ w["q"].T).reshape(T, H, D), pos, m["rot"])
    k = rotate_pairs((h @ w["k"].T).reshape(T, G, D), pos, m["rot"])
    v = (h @ w["v"].T).reshape(T, G, DV)
    out = np.zeros((T, H, DV), h.dtype)
    for hd in range(H):
        g = hd // (H // G)
        s = m["softcap"] * np.tanh((q[:, hd] @ k[:, g].T) * m["scale"] / m["softcap"])
        s = np.where(pos[None, :] <= pos[:, None], s, -np.inf)
        top = np.maximum(s.max(axis=1, keepdims=True), w["sink"][hd])
        e = np.exp(s - top)
        out[:, hd] = (e @ v[:, g]) / (e.sum(axis=1, keepdims=True) + np.exp(w["sink"][hd] - top))
    return (out.reshape(T, H * DV) * sigmoid(h @ w["g"].T)) @ w["o"].T


# ---- real-gated linear recurrent unit ----

def short_conv(x, taps, bias):
    """Causal convolution over time per channel, x [T, channels], taps [channels, n]."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, x.shape[1]), x.dtype), x])
    return bias + sum(taps[:, j] * padded[j:j + x.shape[0]] for j in range(n))


def block_linear(u, w, b):
    """u [T, width], w [blocks, out, in], b [blocks, out]: every block sees its own part of u."""
    parts = np.split(u, w.shape[0], axis=1)
    return np.concatenate([p @ w[j].T + b[j] for j, p in enumerate(parts)], axis=1)


def gated_recurrence(u, r, i, lam):
    S, out = np.zeros(u.shape[1], u.dtype), np.zeros_like(u)
    for t in range(u.shape[0]):
        log_a = -8.0 * r[t] * softplus(lam)
        S = np.exp(log_a) * S + np.sqrt(1.0 - np.exp(log_a) ** 2) * i[t] * u[t]
        out[t] = S
    return out


def rglru(h, w, m, eps):
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = short_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    r, i = sigmoid(block_linear(u, w["ra"], w["ra.b"])), sigmoid(block_linear(u, w["ri"], w["ri.b"]))
    return (gated_recurrence(u, r, i, w["lam"]) * y) @ w["o"].T


def clipped_ff(h, w, limit):
    g, u = np.minimum(h @ w["gate"].T, limit), np.clip(h @ w["up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


MIXERS = {"mlstm": mlstm, "attention": attention, "rglru": rglru}


def layer(x, i, cfg, weights):
    eps, spec, p = cfg["norm"]["eps"], cfg["layers"][i], f"l{i}."
    y = MIXERS[spec["type"]](rms_norm(x, weights[p + "norm1"], eps), part(weights, p + "mix."), spec["mixer"], eps)
    x = x + rms_norm(y, weights[p + "norm1b"], eps)
    if spec.get("mlp"):
        y = clipped_ff(rms_norm(x, weights[p + "norm2"], eps), part(weights, p + "mlp."), spec["mlp"]["limit"])
        x = x + rms_norm(y, weights[p + "norm2b"], eps)
    return x


def forward(tokens, cfg, weights, trace=None):
    """Logits [T, vocab] of one sequence; `trace` (a list) receives the residual stream after every layer run."""
    x = x0 = weights["embed"][np.asarray(tokens)]
    n, loop = len(cfg["layers"]), cfg.get("loop")
    passes = [(range(n), None)] if not loop else (
        [(range(loop["start"]), None)] + [(range(loop["start"], loop["stop"]), t) for t in range(loop["times"])] + [(range(loop["stop"], n), None)])
    for layers, step in passes:
        if step is not None:
            x = x + (x0 if step > 0 else 0.0) + weights["loop.step"][step]
        for i in layers:
            x = layer(x, i, cfg, weights)
            if trace is not None:
                trace.append(x)
    return rms_norm(x, weights["final.norm"], cfg["norm"]["eps"]) @ weights["embed"].T
