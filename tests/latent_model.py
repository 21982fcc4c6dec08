"""Small latent-attention models for tests and the benchmark: configurations and
random bf16 weights (mixed_model writes the folder they are served from)."""
import numpy as np

import mixed_model as mm


def yarn(factor, original, fast=32.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def latent(heads, dim, vdim, kv_rank, scale=None):
    """Without positions, over the whole context, with an output gate."""
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank,
                      "scale": dim ** -0.5 if scale is None else scale}}


def windowed_latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, window, base=10000.0,
                    scaling=None, scale=None):
    return {"type": "latent_attention_2",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
                      "kv_rank": kv_rank, "q_rank": q_rank, "mask": {"size": window},
                      "rot": {"dims": rot_dim, "base": base,
                              "scaling": scaling or yarn(4.0, 256)},
                      "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}}


def gla(heads, dim, vdim, tau=16.0):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def configuration(vocab, width, layers, ffs, eps=1e-5, scale=1.0, residual=0.8):
    """`ffs`: feed-forward width of every layer, 0 = none."""
    listed = []
    for layer, ff in zip(layers, ffs):
        listed.append(dict(layer, mlp={"kind": "dense", "ff": ff} if ff else None))
    return {"architecture": "Nametar", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "embedding": {"scale": scale}, "residual_mult": residual,
            "layers": listed}


def shapes(config, rank=8):
    """Tensor name -> shape; `rank` is that of the decay's low-rank product."""
    vocab, width = config["vocab"], config["width"]
    out = {"embed": (vocab, width), "final.norm": (width,), "head": (vocab, width)}
    for index, layer in enumerate(config["layers"]):
        p, m = f"l{index}.", layer["mixer"]
        heads, dim, vdim = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = out[p + "norm1b"] = (width,)
        p += "mix."
        if layer["type"] == "gla":
            out[p + "q"] = out[p + "k"] = (heads * dim, width)
            out[p + "v"] = out[p + "g"] = (heads * vdim, width)
            out[p + "a1"], out[p + "a2"] = (rank, width), (heads * dim, rank)
            out[p + "a2.b"], out[p + "norm"] = (heads * dim,), (vdim,)
        else:
            turned = m.get("rot_dim", 0)
            if layer["type"] == "latent_attention":
                out[p + "q"], out[p + "g"] = (heads * dim, width), (heads * vdim, width)
            else:
                out[p + "dq"], out[p + "dq.norm"] = (m["q_rank"], width), (m["q_rank"],)
                out[p + "uq"] = (heads * (dim + turned), m["q_rank"])
            out[p + "dkv"] = (m["kv_rank"] + turned, width)
            out[p + "dkv.norm"] = (m["kv_rank"],)
            out[p + "uk"] = (heads * dim, m["kv_rank"])
            out[p + "uv"] = (heads * vdim, m["kv_rank"])
        out[p + "o"] = (width, heads * vdim)
        if layer["mlp"]:
            p, ff = f"l{index}.", layer["mlp"]["ff"]
            out[p + "norm2"] = out[p + "norm2b"] = (width,)
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (ff, width)
            out[p + "mlp.down"] = (width, ff)
    return out


def random_weights(config, seed, rank=8):
    """float32 arrays with bf16 values; scaled so that activations stay O(1) and
    scores spread."""
    rng = np.random.default_rng(seed)
    weights = {}
    for name, shape in shapes(config, rank).items():
        last = name.rsplit(".", 1)[-1]
        if last.startswith("norm"):
            value = 1.0 + 0.2 * rng.standard_normal(shape)
        elif last == "b":
            value = 1.0 + rng.standard_normal(shape)
        elif last == "embed":
            value = rng.standard_normal(shape)
        else:
            gain = 1.6 if last in ("q", "k", "uq", "uk") else 1.0
            value = gain * rng.standard_normal(shape) / np.sqrt(shape[-1])
        weights[name] = mm.bf16(np.asarray(value, dtype=np.float32).reshape(shape))
    return weights
