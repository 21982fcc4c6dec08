"""A plain, slow statement of the latent-attention decoder in float64 NumPy:
latent attention (with and without a query latent, rotated keys, a window, an
output gate), gated linear attention, sublayers between two norms.

One function per mechanism, each written from its equation and free of any code
of the product path.

  x: [tokens, width], weights: dict of float64 arrays under their tensor names
"""
import math

import numpy as np


def root_mean_square_norm(x, weight, eps):
    mean = np.mean(np.square(x), axis=-1, keepdims=True)
    return x / np.sqrt(mean + eps) * weight


def logistic(x):
    """1 / (1 + exp(-x)) without overflow on either side."""
    positive = 1.0 / (1.0 + np.exp(-np.abs(x)))
    return np.where(x >= 0, positive, 1.0 - positive)


def swish(x):
    return x * logistic(x)


def frequencies(dims, base, scaling=None):
    """Angle per position of each pair, and the factor on cosine and sine."""
    out = []
    for i in range(dims // 2):
        out.append(base ** (-2.0 * i / dims))
    if scaling is None:
        return np.array(out), 1.0

    def turning(turns):
        """The dimension that turns this often over the original length."""
        return (dims * math.log(scaling["original"] / (2.0 * math.pi * turns))
                / (2.0 * math.log(base)))

    low = max(math.floor(turning(scaling["fast"])), 0)
    high = min(math.ceil(turning(scaling["slow"])), dims - 1)
    for i, plain in enumerate(out):
        ramp = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
        out[i] = plain / scaling["factor"] * ramp + plain * (1.0 - ramp)
    return np.array(out), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_halves(x, positions, rot):
    """x [tokens, ..., n]: dimension i turns with i + dims / 2; dimensions from
    rot["dims"] on stay."""
    out = x.copy()
    half = rot["dims"] // 2
    per_position, magnitude = frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    for row, position in enumerate(positions):
        for i in range(half):
            c = math.cos(position * per_position[i]) * magnitude
            s = math.sin(position * per_position[i]) * magnitude
            u, v = x[row, ..., i], x[row, ..., i + half]
            out[row, ..., i] = u * c - v * s
            out[row, ..., i + half] = v * c + u * s
    return out


def visible(tokens, window=None):
    seen = np.zeros((tokens, tokens), dtype=bool)
    for i in range(tokens):
        first = 0 if window is None else max(0, i - window + 1)
        seen[i, first:i + 1] = True
    return seen


def attend(q, k, v, scale, seen):
    """One head: q [tokens, n], k [tokens, n], v [tokens, m]."""
    scores = np.where(seen, (q @ k.T) * scale, -np.inf)
    weights = np.exp(scores - scores.max(axis=1, keepdims=True))
    return (weights / weights.sum(axis=1, keepdims=True)) @ v


def latent_mixer(h, w, p, cfg, eps):
    """Latent attention; what the configuration and the tensors name is there:
    a query latent (.dq), rotated dimensions, a window, an output gate (.g)."""
    tokens, heads, dim, vdim = h.shape[0], cfg["heads"], cfg["dim"], cfg["vdim"]
    rank, turned = cfg["kv_rank"], cfg.get("rot_dim", 0)
    if p + "dq" in w:
        latent = root_mean_square_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
        q = latent @ w[p + "uq"].T
    else:
        q = h @ w[p + "q"].T
    q = q.reshape(tokens, heads, dim + turned)
    down = h @ w[p + "dkv"].T
    c = root_mean_square_norm(down[:, :rank], w[p + "dkv.norm"], eps)
    positions = range(tokens)
    shared = down[:, rank:]
    if turned:
        shared = rotate_halves(shared, positions, cfg["rot"])
        q = np.concatenate([q[..., :dim], rotate_halves(q[..., dim:], positions, cfg["rot"])],
                           axis=-1)
    seen = visible(tokens, cfg["mask"]["size"] if cfg.get("mask") else None)
    out = []
    for head in range(heads):
        k = c @ w[p + "uk"][head * dim:(head + 1) * dim].T
        v = c @ w[p + "uv"][head * vdim:(head + 1) * vdim].T
        out.append(attend(q[:, head], np.concatenate([k, shared], axis=1), v, cfg["scale"],
                          seen))
    joined = np.concatenate(out, axis=1)
    if p + "g" in w:
        joined = joined * logistic(h @ w[p + "g"].T)
    return joined @ w[p + "o"].T


def gated_recurrence(q, k, v, alpha, state):
    """One head: the state's rows (key channels) decay, then take up k v^T; the
    token reads what is there afterwards.  Returns (o, final state)."""
    out = np.empty_like(v)
    for t in range(q.shape[0]):
        state = alpha[t][:, None] * state + np.outer(k[t], v[t])
        out[t] = state.T @ q[t]
    return out, state


def channel_decay(z, tau):
    """logistic(z) to the power 1 / tau."""
    return np.exp(-np.logaddexp(0.0, -z) / tau)


def gla_mixer(h, w, p, cfg, eps):
    tokens, heads, dim, vdim = h.shape[0], cfg["heads"], cfg["dim"], cfg["vdim"]
    q = (h @ w[p + "q"].T / math.sqrt(dim)).reshape(tokens, heads, dim)
    k = (h @ w[p + "k"].T).reshape(tokens, heads, dim)
    v = (h @ w[p + "v"].T).reshape(tokens, heads, vdim)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = channel_decay(z, cfg["tau"]).reshape(tokens, heads, dim)
    o = np.empty((tokens, heads, vdim))
    for head in range(heads):
        o[:, head], _ = gated_recurrence(q[:, head], k[:, head], v[:, head], alpha[:, head],
                                         np.zeros((dim, vdim)))
    o = root_mean_square_norm(o, w[p + "norm"], eps).reshape(tokens, heads * vdim)
    return (o * swish(h @ w[p + "g"].T)) @ w[p + "o"].T


def dense_mlp(h, w, p):
    return (swish(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


MIXERS = {"latent_attention": latent_mixer, "latent_attention_2": latent_mixer,
          "gla": gla_mixer}


def forward(cfg, w, tokens):
    """Returns (logits [tokens, vocab], residual stream after every layer)."""
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    streams = []
    for index, layer in enumerate(cfg["layers"]):
        p = "l%d." % index

        def sublayer(x, number, change):
            h = root_mean_square_norm(x, w[p + "norm%d" % number], eps)
            return x + m * root_mean_square_norm(change(h), w[p + "norm%db" % number], eps)

        mixer = MIXERS[layer["type"]]
        x = sublayer(x, 1, lambda h: mixer(h, w, p + "mix.", layer["mixer"], eps))
        if layer["mlp"] is not None:
            x = sublayer(x, 2, lambda h: dense_mlp(h, w, p + "mlp."))
        streams.append(x)
    return root_mean_square_norm(x, w["final.norm"], eps) @ w["head"].T, np.stack(streams)
