"""Plain Ritevik forward in numpy, one function per mechanism, whole sequences token by token where a mechanism
recurs.  Test infrastructure only: it shares nothing with the library.  Everything runs in the dtype of the weights
it is given (float64 in the tests)."""
import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.logaddexp(0.0, z)


def rms_norm(x, weight, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def rms_norm_zero_centred(x, weight, eps):
    return rms_norm(x, 1.0 + weight, eps)


def rotate_half(x, positions, dims, base):
    """x [T, ..., >= dims]: dimension i < dims / 2 turns with dimension i + dims / 2; the rest stays."""
    half = dims // 2
    freq = np.asarray(base, x.dtype) ** (-2.0 * np.arange(half, dtype=x.dtype) / dims)
    a = np.asarray(positions, x.dtype)[:, None] * freq[None, :]
    a = a.reshape((a.shape[0],) + (1,) * (x.ndim - 2) + (half,))
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), x[..., dims:]], axis=-1)


def latent_attention(h, w, m, eps):
    """h [T, width] -> [T, width]; w: the layer's mixer tensors by short name, m: its sizes."""
    T, H, D, R, DV, C = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = np.arange(T)
    q = (h @ w["q"].T).reshape(T, H, D + R)
    q_rot = rotate_half(q[:, :, D:], pos, m["rot"]["dims"], m["rot"]["base"])
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :C], w["dkv.norm"], eps)
    k_rot = rotate_half(down[:, C:], pos, m["rot"]["dims"], m["rot"]["base"])
    k = (c @ w["uk"].T).reshape(T, H, D)
    v = (c @ w["uv"].T).reshape(T, H, DV)
    out = np.zeros((T, H, DV), h.dtype)
    for hd in range(H):
        s = (q[:, hd, :D] @ k[:, hd].T + q_rot[:, hd] @ k_rot.T) * m["scale"]
        s = np.where(pos[None, :] <= pos[:, None], s, -np.inf)
        sink = w["sink"][hd]
        top = np.maximum(s.max(axis=1, keepdims=True), sink)
        e = np.exp(s - top)
        out[:, hd] = (e @ v[:, hd]) / (e.sum(axis=1, keepdims=True) + np.exp(sink - top))
    return out.reshape(T, H * DV) @ w["o"].T


def short_conv_silu(x, taps):
    """Causal convolution over time per channel, x [T, channels], taps [channels, n], then silu."""
    T, n = x.shape[0], taps.shape[1]
    out = np.zeros_like(x)
    for t in range(T):
        for j in range(n):
            src = t - (n - 1) + j
            if src >= 0:
                out[t] += taps[:, j] * x[src]
    return silu(out)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_recurrence(q, k, v, g, beta):
    """q, k, g [T, H, D], v [T, H, DV], beta [T, H] -> o [T, H, DV] and the state after the last token [H, D, DV]."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]), q.dtype)
    o = np.zeros_like(v)
    for t in range(T):
        for hd in range(H):
            S[hd] = g[t, hd][:, None] * S[hd]
            u = beta[t, hd] * (v[t, hd] - S[hd].T @ k[t, hd])
            S[hd] = S[hd] + np.outer(k[t, hd], u)
            o[t, hd] = S[hd].T @ q[t, hd]
    return o, S


def channel_delta(h, w, m, eps):
    T, H, HK, D, DV = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv_silu(h @ w["q"].T, w["q.conv"]).reshape(T, HK, D)
    k = short_conv_silu(h @ w["k"].T, w["k.conv"]).reshape(T, HK, D)
    v = short_conv_silu(h @ w["v"].T, w["v.conv"]).reshape(T, H, DV)
    group = np.arange(H) // (H // HK)
    q = unit(q)[:, group] * D ** -0.5
    k = unit(k)[:, group]
    beta = sigmoid(h @ w["b"].T)
    step = softplus((h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]).reshape(T, H, D)
    g = np.exp(-np.exp(w["A_log"])[None, :, None] * step)
    o, _ = delta_recurrence(q, k, v, g, beta)
    o = rms_norm(o, w["norm"], eps) * sigmoid((h @ w["g1"].T) @ w["g2"].T).reshape(T, H, DV)
    return o.reshape(T, H * DV) @ w["o"].T


def dense_ff(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def side_input(x, tokens, table_part, w, eps):
    y = (gelu_tanh(x @ w["gate"].T) * table_part[tokens]) @ w["proj"].T
    return x + rms_norm(y, w["norm"], eps)


def part(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def layer(x, tokens, i, cfg, weights):
    eps, spec = cfg["norm"]["eps"], cfg["layers"][i]
    h = rms_norm_zero_centred(x, weights[f"l{i}.norm1"], eps)
    mixer = {"latent_attention": latent_attention, "channel_delta": channel_delta}[spec["type"]]
    y = mixer(h, part(weights, f"l{i}.mix."), spec["mixer"], eps)
    if spec.get("mlp"):
        y = y + dense_ff(h, part(weights, f"l{i}.mlp."))
    x = x + y
    if cfg.get("token_side"):
        n = cfg["token_side"]["dim"]
        x = side_input(x, tokens, weights["side.embed"][:, i * n:(i + 1) * n], part(weights, f"l{i}.side."), eps)
    return x


def forward(tokens, cfg, weights, trace=None):
    """Logits [T, vocab] of one sequence; `trace` (a list) receives the residual stream after every layer run."""
    eps = cfg["norm"]["eps"]
    tokens = np.asarray(tokens)
    x = rms_norm_zero_centred(weights["embed"][tokens], weights["embed.norm"], eps)
    x0 = x

    def run(lo, hi):
        nonlocal x
        for i in range(lo, hi):
            x = layer(x, tokens, i, cfg, weights)
            if trace is not None:
                trace.append(x)

    loop = cfg.get("loop")
    n = len(cfg["layers"])
    if not loop:
        run(0, n)
    else:
        run(0, loop["start"])
        for t in range(loop["times"]):
            x = np.concatenate([x, x0], axis=1) @ weights["loop.in"].T + weights["loop.step"][t]
            run(loop["start"], loop["stop"])
        run(loop["stop"], n)
    return rms_norm_zero_centred(x, weights["final.norm"], eps) @ weights["head"].T
