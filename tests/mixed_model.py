"""Small mixed-layer models for tests and the benchmark: configurations, random
bf16 weights and the folder they are served from."""
import json
import os
import struct

import numpy as np


def bf16(array):
    """Round to bf16 (nearest even), returned as float32."""
    array = np.asarray(array, dtype=np.float32)
    if not array.flags.c_contiguous:
        array = np.ascontiguousarray(array)
    bits = array.view(np.uint32)
    bits = bits + 0x7FFF + ((bits >> 16) & 1)
    return (bits & 0xFFFF0000).view(np.float32)


def attention(heads, kv_heads, dim, vdim, window, keep, rotary=None, base=10000.0,
              scale=None, v_mix=True):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "mask": {"size": window, "keep_first": keep},
                      "rot": {"dims": dim if rotary is None else rotary, "base": base},
                      "scale": dim ** -0.5 if scale is None else scale, "v_mix": v_mix}}


def general_delta(heads, dim):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim}}


def wkv(heads, dim):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}}


def configuration(vocab, width, layers, ffs, eps=1e-5, scale=1.0):
    """`ffs`: feed-forward width of every layer, 0 = none."""
    listed = []
    for layer, ff in zip(layers, ffs):
        listed.append(dict(layer, mlp={"kind": "dense", "ff": ff} if ff else None))
    return {"architecture": "Zatupel", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": listed}


def shapes(config, rank=8):
    """Tensor name -> shape, in the order they are stored."""
    vocab, width = config["vocab"], config["width"]
    out = {"embed": (vocab, width), "final.norm": (width,), "head": (vocab, width)}
    for index, layer in enumerate(config["layers"]):
        p, m = f"l{index}.", layer["mixer"]
        out[p + "norm1"] = (width,)
        if layer["type"] == "attention":
            inner = m["heads"] * m["vdim"]
            out[p + "mix.q"] = (m["heads"] * m["dim"], width)
            out[p + "mix.k"] = (m["kv_heads"] * m["dim"], width)
            out[p + "mix.v"] = (m["kv_heads"] * m["vdim"], width)
            out[p + "mix.g"] = (m["heads"], width)
            out[p + "mix.talk"] = (m["heads"], m["heads"])
            if m["v_mix"]:
                out[p + "mix.vmix"] = ()
        else:
            inner = m["heads"] * m["dim"]
            for name in "rkvg":
                out[p + "mix." + name] = (inner, width)
            out[p + "mix.w1"] = (rank, width)
            out[p + "mix.w2"] = (inner, rank)
            out[p + "mix.w0"] = (inner,)
            out[p + "mix.norm"] = (inner,)
            if layer["type"] == "general_delta":
                out[p + "mix.a"] = (inner, width)
                out[p + "mix.a.b"] = (inner,)
            else:
                for name in "rkvgw":
                    out[p + "mix.mu." + name] = (width,)
                out[p + "mix.u"] = (m["heads"], m["dim"])
        out[p + "mix.o"] = (width, inner)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out[p + "norm2"] = (width,)
            out[p + "mlp.gate"] = (ff, width)
            out[p + "mlp.up"] = (ff, width)
            out[p + "mlp.down"] = (width, ff)
    return out


def random_weights(config, seed, rank=8):
    """float32 arrays with bf16 values; scaled so that activations stay O(1)."""
    rng = np.random.default_rng(seed)
    weights = {}
    for name, shape in shapes(config, rank).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2", "norm"):
            value = 1.0 + 0.2 * rng.standard_normal(shape)
        elif last == "w0":
            value = -3.0 + rng.standard_normal(shape)
        elif last == "b":
            value = rng.standard_normal(shape)
        elif last == "vmix":
            value = np.float64(rng.uniform(0.2, 0.8))
        elif ".mu." in name:
            value = rng.uniform(0.0, 1.0, shape)
        elif last == "u":
            value = 0.5 * rng.standard_normal(shape)
        elif last == "talk":
            value = np.eye(shape[0]) + 0.5 * rng.standard_normal(shape)
        elif last == "embed":
            value = rng.standard_normal(shape)
        else:
            gain = 1.5 if last in ("q", "k") else 1.0
            value = gain * rng.standard_normal(shape) / np.sqrt(shape[-1])
        weights[name] = bf16(np.asarray(value, dtype=np.float32).reshape(shape))
    return weights


def write_folder(path, config, weights):
    """config.json and model.safetensors (bf16)."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as out:
        json.dump(config, out)
    header, offset = {}, 0
    for name, value in weights.items():
        header[name] = {"dtype": "BF16", "shape": list(np.shape(value)),
                        "data_offsets": [offset, offset + 2 * value.size]}
        offset += 2 * value.size
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as out:
        out.write(struct.pack("<Q", len(text)))
        out.write(text)
        for value in weights.values():
            bits = np.ascontiguousarray(value, dtype=np.float32).view(np.uint32) >> 16
            out.write(bits.astype(np.uint16).tobytes())
    return str(path)


class TiledWeights(dict):
    """Weights of a large model without its memory: matrices repeat one random
    block, scaled to keep activations O(1)."""

    def __init__(self, shapes, seed):
        self.shapes = shapes
        rng = np.random.default_rng(seed)
        self.block = rng.standard_normal(1 << 20).astype(np.float32)
        super().__init__((name, None) for name in self.shapes)

    def items(self):
        for name, shape in self.shapes.items():
            yield name, self.one(name, shape)

    def values(self):
        for name, shape in self.shapes.items():
            yield self.one(name, shape)

    def one(self, name, shape):
        last = name.rsplit(".", 1)[-1]
        if len(shape) == 2 and last not in ("talk", "u"):
            flat = np.resize(self.block, int(np.prod(shape))).reshape(shape)
            return bf16(flat if last == "embed" else flat * np.float32(shape[-1] ** -0.5))
        if last == "talk":
            return bf16(np.eye(shape[0], dtype=np.float32) + 0.1)
        if last.startswith("norm"):
            return np.ones(shape, dtype=np.float32)
        if last == "w0":
            return np.full(shape, -3.0, dtype=np.float32)
        return np.full(shape, 0.5, dtype=np.float32)


def float64(weights):
    return {name: np.asarray(value, dtype=np.float64) for name, value in weights.items()}
