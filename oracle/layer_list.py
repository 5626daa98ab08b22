"""Plain NumPy model of the decoders whose layers are listed in config.json (architecture "Girirax").

One function per mechanism, written for reading: a token loop for the recurrence, full score matrices for the
attention, everything in the floating-point type the caller passes (float64 by default).  It is what
tests/test_girirax.py and tests/test_gpu_girirax.py compare with; it shares nothing with the product: no kernels, no
cache, no chunking.

Notation: h [T, width] is what a sublayer reads, T the tokens of ONE sequence from position 0.
"""
import numpy as np


def rms_norm(x, weight, eps):
    """Root-mean-square norm over the last axis, eps inside the root; weight may be None."""
    y = x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)
    return y if weight is None else y * weight


def silu(z):
    return z / (1 + np.exp(-z))


def sigmoid(z):
    return 1 / (1 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0, z)


def gelu_tanh(z):
    return 0.5 * z * (1 + np.tanh(np.sqrt(2 / np.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(u, taps, bias):
    """Per-channel causal convolution: u [T, C], taps [C, K]; the last column multiplies the current token."""
    T, K = u.shape[0], taps.shape[1]
    padded = np.concatenate([np.zeros((K - 1, u.shape[1]), u.dtype), u])
    out = np.zeros_like(u)
    for k in range(K):
        out += padded[k:k + T] * taps[:, k]
    return out + bias


def ssd_scan(x, b, c, dt, a_log, d):
    """Selective state-space recurrence, token by token: x [T, H, P], b / c [T, G, N], dt [T, H] (after softplus),
    state [H, N, P] from zero."""
    T, H, P = x.shape
    per_group = H // b.shape[1]
    state = np.zeros((H, b.shape[2], P), x.dtype)
    y = np.zeros_like(x)
    for t in range(T):
        for h in range(H):
            g = h // per_group
            state[h] = np.exp(-np.exp(a_log[h]) * dt[t, h]) * state[h] + dt[t, h] * np.outer(b[t, g], x[t, h])
            y[t, h] = state[h].T @ c[t, g] + d[h] * x[t, h]
    return y


def gated_group_norm(y, z, weight, groups, eps):
    """The gate first, then each of `groups` equal parts by its own root mean square."""
    v = y * silu(z)
    parts = v.reshape(v.shape[0], groups, -1)
    return rms_norm(parts, None, eps).reshape(v.shape) * weight


def mamba2(h, w, m, eps):
    """m: sizes (heads, vdim, state, groups, norm_groups); w: tensors by their short names."""
    inner, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
    T = h.shape[0]
    z, xbc, dt = np.split(h @ w["in"].T, [inner, 2 * inner + 2 * gn], axis=1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, b, c = np.split(xbc, [inner, inner + gn], axis=1)
    y = ssd_scan(x.reshape(T, m["heads"], m["vdim"]), b.reshape(T, m["groups"], m["state"]),
                 c.reshape(T, m["groups"], m["state"]), softplus(dt + w["dt_bias"]), w["A_log"], w["D"])
    return gated_group_norm(y.reshape(T, inner), z, w["norm"], m["norm_groups"], eps) @ w["o"].T


def rotate_half(x, positions, base, dims):
    """x [T, H, D]: pair (i, i + dims/2) of the first `dims` dimensions turned by position * base^(-2i/dims)."""
    half = dims // 2
    freq = np.float64(base) ** (-2.0 * np.arange(half) / dims)
    angle = (positions[:, None] * freq)[:, None, :]
    cos, sin = np.cos(angle).astype(x.dtype), np.sin(angle).astype(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], axis=-1)


def causal_attention(q, k, v, scale):
    """q / k [T, H, D], v [T, H, Dv]: softmax over all keys up to the query's own position."""
    T = q.shape[0]
    scores = np.einsum("ihd,jhd->hij", q, k) * scale
    scores = np.where(np.tril(np.ones((T, T), bool)), scores, -np.inf)
    scores = np.exp(scores - scores.max(axis=-1, keepdims=True))
    return np.einsum("hij,jhd->ihd", scores / scores.sum(axis=-1, keepdims=True), v)


def latent_attention(h, w, m, eps):
    """m: sizes (heads, dim, rot_dim, vdim, kv_rank, scale, rot.base, rot.dims)."""
    T, H, D, R, V = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    pos = np.arange(T)
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).reshape(T, H, D + R)
    ckv = h @ w["dkv"].T
    c = rms_norm(ckv[:, :m["kv_rank"]], w["dkv.norm"], eps)
    rot = lambda t: rotate_half(t, pos, m["rot"]["base"], m["rot"]["dims"])
    k_rot = rot(ckv[:, None, m["kv_rank"]:])
    q = np.concatenate([q[..., :D], rot(q[..., D:])], axis=-1)
    k = np.concatenate([(c @ w["uk"].T).reshape(T, H, D), np.broadcast_to(k_rot, (T, H, R))], axis=-1)
    v = (c @ w["uv"].T).reshape(T, H, V)
    out = causal_attention(q, k, v, m["scale"]).reshape(T, H * V)
    return (out * sigmoid(h @ w["g"].T)) @ w["o"].T


def gated_mlp(h, w):
    act = gelu_tanh(h @ w["gate"].T + w["gate.b"]) * (h @ w["up"].T + w["up.b"])
    return act @ w["down"].T + w["down.b"]


MIXERS = {"mamba2": mamba2, "latent_attention": latent_attention}


def _short_names(tensors, prefix, dtype):
    return {k[len(prefix):]: v.astype(dtype) for k, v in tensors.items() if k.startswith(prefix)}


def forward(config, tensors, tokens, dtype=np.float64, trace=None):
    """Logits [T, vocab] of one sequence; tensors: name -> float array.  trace (a list) receives the residual
    stream after every layer."""
    eps, mult = config["norm"]["eps"], dtype(config["residual_mult"])
    embed = tensors["embed"].astype(dtype)
    x = embed[np.asarray(tokens)] * dtype(config["embedding"]["scale"])
    for i, layer in enumerate(config["layers"]):
        p = "l%d." % i
        mix = MIXERS[layer["type"]](x, _short_names(tensors, p + "mix.", dtype), layer["mixer"], eps)
        x = x + mult * rms_norm(mix, tensors[p + "norm1"].astype(dtype), eps)
        if layer["mlp"] is not None:
            ff = gated_mlp(x, _short_names(tensors, p + "mlp.", dtype))
            x = x + mult * rms_norm(ff, tensors[p + "norm2"].astype(dtype), eps)
        if trace is not None:
            trace.append(x.copy())
    return rms_norm(x, tensors["final.norm"].astype(dtype), eps) @ embed.T
