"""Model folders on the host: what is turned down before a device is touched."""
import json
import os
import struct

import pytest

import latent_model as lm
import mixed_model as mm
import qllm_provider as qp


def folder(tmp_path, **changes):
    config = mm.configuration(32, 16, [mm.attention(2, 1, 8, 8, 4, 0), mm.wkv(1, 8)], [16, 0])
    path = mm.write_folder(tmp_path / "m", config, mm.random_weights(config, 1))
    config.update(changes)
    for key in [key for key, value in changes.items() if value is None]:
        del config[key]
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as out:
        json.dump(config, out)
    return path


def refusal(path):
    with pytest.raises(qp.ProviderError) as caught:
        qp.Model(path, 64)
    return str(caught.value)


def test_unknown_architecture_names_it(tmp_path):
    assert "Unheard" in refusal(folder(tmp_path, architecture="Unheard"))


@pytest.mark.parametrize("key", ["architecture", "vocab", "width", "norm", "embedding",
                                 "layers"])
def test_missing_keys_are_named(tmp_path, key):
    assert key in refusal(folder(tmp_path, **{key: None}))


def test_unknown_mixer_and_feed_forward_are_named(tmp_path):
    layer = {"type": "convolution", "mixer": {"heads": 1, "dim": 8}, "mlp": None}
    assert "convolution" in refusal(folder(tmp_path, layers=[layer]))
    layer = {"type": "wkv", "mixer": {"heads": 1, "dim": 8}, "mlp": {"kind": "routed", "ff": 4}}
    assert "routed" in refusal(folder(tmp_path / "b", layers=[layer]))


def test_latent_layers_with_missing_keys(tmp_path):
    def refused(kind, key, value=None):
        layer = {"windowed": lm.windowed_latent(2, 8, 4, 8, 12, 10, 5),
                 "latent": lm.latent(2, 8, 8, 12), "gla": lm.gla(2, 8, 8)}[kind]
        config = lm.configuration(32, 16, [layer], [16])
        place = config["layers"][0]["mixer"]
        *path, last = key.split(".")
        for part in path:
            place = place[part]
        if value is None:
            del place[last]
        else:
            place[last] = value
        path = mm.write_folder(tmp_path / (kind + key), config, lm.random_weights(
            lm.configuration(32, 16, [lm.latent(2, 8, 8, 12)], [16]), 1))
        return refusal(path)

    for key in ("heads", "dim", "vdim", "kv_rank", "scale", "rot_dim", "rot", "mask.size",
                "rot.base", "rot.dims", "rot.scaling.factor", "rot.scaling.slow"):
        assert key.split(".")[-1] in refused("windowed", key), key
    assert "kv_rank" in refused("latent", "kv_rank")
    assert "tau" in refused("gla", "tau")
    assert "tau" in refused("gla", "tau", 0)


def test_broken_tensor_files(tmp_path):
    path = folder(tmp_path)
    file = os.path.join(path, "model.safetensors")
    with open(file, "rb") as source:
        data = source.read()
    length = struct.unpack("<Q", data[:8])[0]
    header = json.loads(data[8:8 + length])

    def rewrite(new_header, body=data[8 + length:]):
        text = json.dumps(new_header).encode()
        with open(file, "wb") as out:
            out.write(struct.pack("<Q", len(text)) + text + body)

    broken = json.loads(json.dumps(header))
    broken["embed"]["shape"][0] += 1
    rewrite(broken)
    assert "embed" in refusal(path)
    broken = json.loads(json.dumps(header))
    broken["embed"]["data_offsets"][1] = 1 << 40
    rewrite(broken)
    assert "embed" in refusal(path)
    with open(file, "wb") as out:
        out.write(struct.pack("<Q", 1 << 50))
    assert "header" in refusal(path)
    os.remove(file)
    assert "open" in refusal(path)


def test_neither_folder_nor_artifact(tmp_path):
    assert refusal(str(tmp_path))
