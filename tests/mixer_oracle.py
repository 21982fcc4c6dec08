"""A plain, slow statement of the mixed-layer decoder in float64 NumPy.

One function per mechanism, each written from its equation and free of any
code of the product path: whole sequences at once where the mathematics is
per position, one token after the other where it is a recurrence.

  x: [tokens, width], weights: dict of float64 arrays under their tensor names
"""
import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rotate_interleaved(x, positions, dims, base):
    """x [tokens, heads, dim]: dimension 2i turns with dimension 2i + 1 by the
    angle position * base^(-2i / dims); dimensions from `dims` on stay."""
    out = x.copy()
    for i in range(dims // 2):
        angle = positions * base ** (-2.0 * i / dims)
        c, s = np.cos(angle)[:, None], np.sin(angle)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


def visible_window(queries, keys, window, sinks):
    """[queries, keys] of bool: causal, and within `window` positions (the
    query's own included) or among the first `sinks`."""
    i, j = queries[:, None], keys[None, :]
    return (j <= i) & ((i - j < window) | (j < sinks))


def softmax(scores, visible):
    scores = np.where(visible, scores, -np.inf)
    weights = np.exp(scores - scores.max(axis=-1, keepdims=True))
    return weights / weights.sum(axis=-1, keepdims=True)


def mix_heads(weights, matrix):
    """weights [heads, queries, keys]: head h gets sum_g matrix[h, g] weights[g]."""
    return np.einsum("hg,gqk->hqk", matrix, weights)


def attention_core(q, k, v, queries, keys, scale, window, sinks, talk):
    """q [queries, heads, dim], k/v [keys, kv_heads, ...] at absolute positions
    `queries` / `keys`; returns [queries, heads, vdim]."""
    group = q.shape[1] // k.shape[1]
    seen = visible_window(queries, keys, window, sinks)
    weights = np.stack([softmax(q[:, h] @ k[:, h // group].T * scale, seen)
                        for h in range(q.shape[1])])
    mixed = mix_heads(weights, talk)
    return np.stack([mixed[h] @ v[:, h // group] for h in range(q.shape[1])], axis=1)


def attention_mixer(h, w, p, cfg, first_values):
    """Returns (output, this layer's unmixed values)."""
    tokens = h.shape[0]
    positions = np.arange(tokens, dtype=np.float64)
    heads, kv = cfg["heads"], cfg["kv_heads"]
    q = (h @ w[p + "q"].T).reshape(tokens, heads, cfg["dim"])
    k = (h @ w[p + "k"].T).reshape(tokens, kv, cfg["dim"])
    v = (h @ w[p + "v"].T).reshape(tokens, kv, cfg["vdim"])
    own = v
    q = rotate_interleaved(q, positions, cfg["rot"]["dims"], cfg["rot"]["base"])
    k = rotate_interleaved(k, positions, cfg["rot"]["dims"], cfg["rot"]["base"])
    if cfg["v_mix"] and first_values is not None:
        share = float(w[p + "vmix"])
        v = (1.0 - share) * v + share * first_values
    o = attention_core(q, k, v, positions, positions, cfg["scale"], cfg["mask"]["size"],
                       cfg["mask"]["keep_first"], w[p + "talk"])
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(tokens, -1) @ w[p + "o"].T, own


def delta_recurrence(r, k, v, w, a, state):
    """One head.  r/k/w/a [tokens, dim], v [tokens, dim], state [dim, dim]
    (key channel first); returns (o [tokens, dim], final state)."""
    out = np.empty_like(v)
    for t in range(r.shape[0]):
        u = k[t] / np.sqrt(np.sum(k[t] * k[t]) + 1e-6)
        state = (w[t][:, None] * state - np.outer(a[t] * u, u @ state)
                 + np.outer(k[t], v[t]))
        out[t] = state.T @ r[t]
    return out, state


def delta_mixer(h, w, p, cfg, eps):
    tokens, heads, dim = h.shape[0], cfg["heads"], cfg["dim"]
    shape = (tokens, heads, dim)
    r, k, v = ((h @ w[p + n].T).reshape(shape) for n in "rkv")
    inner = np.tanh(h @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]
    decay = np.exp(-np.exp(-0.5) * sigmoid(inner)).reshape(shape)
    rate = sigmoid(h @ w[p + "a"].T + w[p + "a.b"]).reshape(shape)
    o = np.empty(shape)
    for head in range(heads):
        o[:, head], _ = delta_recurrence(r[:, head], k[:, head], v[:, head], decay[:, head],
                                         rate[:, head], np.zeros((dim, dim)))
    o = rms(o, eps).reshape(tokens, heads * dim) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def wkv_recurrence(r, k, v, w, u, state):
    out = np.empty_like(v)
    for t in range(r.shape[0]):
        fresh = np.outer(k[t], v[t])
        out[t] = (state + u[:, None] * fresh).T @ r[t]
        state = w[t][:, None] * state + fresh
    return out, state


def shift_mix(h, previous, mu):
    """Every token's input blended with the one before it."""
    before = np.concatenate([previous[None, :], h[:-1]])
    return h + (before - h) * mu


def wkv_mixer(h, w, p, cfg, eps):
    tokens, heads, dim = h.shape[0], cfg["heads"], cfg["dim"]
    shape = (tokens, heads, dim)
    mixed = {n: shift_mix(h, np.zeros(h.shape[1]), w[p + "mu." + n]) for n in "rkvgw"}
    r, k, v = ((mixed[n] @ w[p + n].T).reshape(shape) for n in "rkv")
    gate = silu(mixed["g"] @ w[p + "g"].T)
    inner = np.tanh(mixed["w"] @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]
    decay = np.exp(-np.exp(inner)).reshape(shape)
    bonus = w[p + "u"].reshape(heads, dim)
    o = np.empty(shape)
    for head in range(heads):
        o[:, head], _ = wkv_recurrence(r[:, head], k[:, head], v[:, head], decay[:, head],
                                       bonus[head], np.zeros((dim, dim)))
    o = rms(o, eps).reshape(tokens, heads * dim) * w[p + "norm"] * gate
    return o @ w[p + "o"].T


def gated_mlp(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def forward(cfg, w, tokens):
    """Returns (logits [tokens, vocab], residual stream after every layer)."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    first_values = None
    streams = []
    for index, layer in enumerate(cfg["layers"]):
        p = "l%d." % index
        h = rms(x, eps) * w[p + "norm1"]
        mixer = layer["mixer"]
        if layer["type"] == "attention":
            change, own = attention_mixer(h, w, p + "mix.", mixer, first_values)
            if mixer["v_mix"] and first_values is None:
                first_values = own
        elif layer["type"] == "general_delta":
            change = delta_mixer(h, w, p + "mix.", mixer, eps)
        elif layer["type"] == "wkv":
            change = wkv_mixer(h, w, p + "mix.", mixer, eps)
        else:
            raise ValueError("unknown mixer " + layer["type"])
        if layer["mlp"] is not None:
            change = change + gated_mlp(rms(x, eps) * w[p + "norm2"], w, p + "mlp.")
        x = x + change
        streams.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T, np.stack(streams)
