"""Plain NumPy models of the decoders whose layers are listed in config.json (architectures "Girirax" and "Bonatar").

One function per mechanism, written for reading: a token loop for the recurrence, full score matrices for the
attention, everything in the floating-point type the caller passes (float64 by default).  It is what
tests/test_girirax.py, tests/test_bonatar.py and their GPU counterparts compare with; it shares nothing with the
product: no kernels, no cache, no portions.

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


# ---- Bonatar: attention inside chunks with grouped heads, experts chosen by token id ----------------------------

def yarn_frequencies(base, dims, scaling):
    """Frequencies of the dims/2 rotation pairs, and the factor of cosine and sine.  scaling (factor, original, fast,
    slow) or None: pairs that turn more than `fast` times over `original` positions keep their frequency, those that
    turn less than `slow` times have it divided by factor, a ramp over the pairs lies between."""
    i = np.arange(dims // 2)
    f = np.float64(base) ** (-2.0 * i / dims)
    if scaling is None:
        return f, 1.0

    def pair_that_turns(t):
        return dims * np.log(scaling["original"] / (2 * np.pi * t)) / (2 * np.log(base))
    lo = max(np.floor(pair_that_turns(scaling["fast"])), 0)
    hi = min(np.ceil(pair_that_turns(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0, 1)
    return f / scaling["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(scaling["factor"]) + 1


def rotate_neighbours(x, positions, freq, mult):
    """x [T, H, D]: pair (2i, 2i + 1) turned by position * freq[i], cosine and sine times mult; dimensions behind the
    last pair stay."""
    angle = (positions[:, None] * freq)[:, None, :]
    cos, sin = (np.cos(angle) * mult).astype(x.dtype), (np.sin(angle) * mult).astype(x.dtype)
    y = x.copy()
    n = 2 * len(freq)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y[..., 0:n:2] = u * cos - v * sin
    y[..., 1:n:2] = v * cos + u * sin
    return y


def chunk_attention(q, k, v, scale, chunk, first=0):
    """q [N, H, D] of the positions from `first` on, k [T, G, D], v [T, G, V]: query head h reads key/value head
    h // (H // G); position i sees j <= i of its own chunk of `chunk` positions (None: of all)."""
    N, H = q.shape[:2]
    per = H // k.shape[1]
    i, j = first + np.arange(N), np.arange(len(k))
    seen = i[:, None] >= j[None, :]
    if chunk is not None:
        seen &= (i[:, None] // chunk) == (j[None, :] // chunk)
    out = np.zeros((N, H, v.shape[2]), q.dtype)
    for h in range(H):
        s = np.where(seen, (q[:, h] @ k[:, h // per].T) * scale, -np.inf)
        s = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (s / s.sum(axis=1, keepdims=True)) @ v[:, h // per]
    return out


def gated_chunk_attention(h, w, m):
    """m: sizes (heads, kv_heads, dim, vdim, scale, rot, mask.size); one gate number per head."""
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    freq, mult = yarn_frequencies(m["rot"]["base"], m["rot"]["dims"], m["rot"].get("scaling"))
    turn = lambda x: rotate_neighbours(x, np.arange(T), freq, mult)
    q, k = turn((h @ w["q"].T).reshape(T, H, D)), turn((h @ w["k"].T).reshape(T, G, D))
    out = chunk_attention(q, k, (h @ w["v"].T).reshape(T, G, V), m["scale"], m["mask"]["size"])
    return (out * sigmoid(h @ w["g"].T)[:, :, None]).reshape(T, H * V) @ w["o"].T


def square_relu_mlp(h, w):
    return np.maximum(h @ w["up"].T, 0) ** 2 @ w["down"].T


def clamped_expert(h, w, prefix, limit):
    g = np.minimum(h @ w[prefix + "gate"].T, limit)
    u = np.clip(h @ w[prefix + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1)) @ w[prefix + "down"].T


def table_routed_mlp(h, w, tokens, m):
    """Every token's experts are its row of the table, weighted equally; a shared expert runs for all."""
    table = w["table"].astype(np.int64)
    y = np.zeros_like(h)
    for t, token in enumerate(tokens):
        for e in table[token]:
            y[t] += clamped_expert(h[t:t + 1], w, "e%d." % e, m["expert"]["limit"])[0] / m["router"]["top"]
    if m.get("shared") is not None:
        y += clamped_expert(h, w, "shared.", m["shared"]["limit"])
    return y


def forward_bonatar(config, tensors, tokens, dtype=np.float64, trace=None):
    """Logits [T, vocab] of one sequence.  Norms stand in front of the sublayers, their weights around zero; a layer
    with weights_of uses another layer's tensors."""
    eps, tokens = config["norm"]["eps"], np.asarray(tokens)
    norm = lambda x, name: rms_norm(x, 1 + tensors[name].astype(dtype), eps)
    x = tensors["embed"].astype(dtype)[tokens] * dtype(config["embedding"]["scale"])
    for i, layer in enumerate(config["layers"]):
        while layer.get("weights_of") is not None:
            i = layer["weights_of"]
            layer = config["layers"][i]
        p = "l%d." % i
        x = x + gated_chunk_attention(norm(x, p + "norm1"), _short_names(tensors, p + "mix.", dtype), layer["mixer"])
        m = layer["mlp"]
        if m is not None:
            h, w = norm(x, p + "norm2"), _short_names(tensors, p + "mlp.", dtype)
            x = x + (square_relu_mlp(h, w) if m["kind"] == "dense" else table_routed_mlp(h, w, tokens, m))
        if trace is not None:
            trace.append(x.copy())
    return norm(x, "final.norm") @ tensors["head"].astype(dtype).T


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
