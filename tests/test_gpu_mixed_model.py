"""Whole mixed-layer models through the framework's own entry points: the model
folder, the compiled program, request slots and pages, sampling, the worker -
against the plain float64 statement."""
import os

import numpy as np
import pytest

import mixed_model as mm
import mixer_oracle as mo
import qllm_provider as qp
import worker_client as wc
from model_util import LIMIT, Case, continuation, distance, feed

pytestmark = pytest.mark.gpu


def configurations():
    return {
        # layer order, unequal sizes, layers without feed-forward, rotary on part
        # of a head, blended values that skip a layer
        "mixed": mm.configuration(
            150, 96, [mm.wkv(3, 24), mm.attention(6, 3, 40, 24, 19, 3, rotary=16, base=500.0),
                      mm.general_delta(2, 40), mm.attention(6, 3, 40, 24, 50, 0, v_mix=False),
                      mm.attention(3, 3, 48, 24, 33, 37, base=1e5, scale=0.2),
                      mm.general_delta(4, 16)],
            [70, 0, 130, 64, 96, 0], eps=1e-4, scale=0.7),
        # sizes of one, odd sizes
        "small": mm.configuration(
            33, 18, [mm.attention(1, 1, 8, 5, 1, 0, rotary=2), mm.wkv(1, 7),
                     mm.general_delta(1, 1), mm.attention(3, 1, 6, 5, 7, 1)],
            [1, 17, 0, 5], eps=1e-6, scale=2.0),
        # many heads, several query heads per key/value head, state of 128
        "wide": mm.configuration(
            260, 128, [mm.attention(32, 8, 16, 8, 64, 4), mm.general_delta(1, 128),
                       mm.attention(32, 8, 16, 8, 20, 9), mm.wkv(2, 100)],
            [256, 40, 0, 128], eps=1e-5, scale=1.0),
    }


CONFIGS = configurations()


def case_of(name, folder):
    config = CONFIGS[name]
    return Case(config, mm.random_weights(config, 11), mo.forward, folder)


@pytest.fixture(scope="module", params=list(CONFIGS))
def case(request, tmp_path_factory):
    return case_of(request.param, tmp_path_factory.mktemp(request.param))


@pytest.fixture(scope="module")
def mixed(tmp_path_factory):
    return case_of("mixed", tmp_path_factory.mktemp("one"))


def test_streams_after_every_layer(case):
    model = qp.Model(case.path, 256, kv_page_tokens=32, kv_cache_dtype="fp32")
    request = model.begin()
    layers = len(case.config["layers"])
    first, _ = model.trace_layers(request, case.tokens[:41], layers)
    second, token = model.trace_layers(request, case.tokens[41:60], layers)
    got = np.concatenate([first, second], axis=1)
    for layer in range(layers):
        assert distance(got[layer], case.streams[layer][:60]).max() < 1e-5, layer
    assert token == case.logits[59].argmax()
    model.close()


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("counts", [[210], [1], [2], [7, 3, 64], [100, 1, 1, 33, 2]],
                         ids=lambda c: "-".join(map(str, c)))
def test_logits_however_the_prompt_is_cut(case, dtype, counts):
    model = qp.Model(case.path, 256, kv_page_tokens=64, kv_cache_dtype=dtype)
    request = model.begin()
    got = feed(model, request, case.tokens, counts)
    errors = distance(got, case.logits)
    assert errors.max() < 2 * LIMIT[dtype] and errors.mean() < LIMIT[dtype], errors.max()
    model.close()


def test_batches_longer_than_the_program_takes_at_once(mixed):
    model = qp.Model(mixed.path, 256, kv_page_tokens=32, kv_cache_dtype="fp32", chunk_rows=48)
    assert model.batch_limit == 48
    request = model.begin()
    got, token = model.step(request, mixed.tokens, range(210))
    assert distance(got, mixed.logits).max() < LIMIT["fp32"]
    assert token == mixed.logits[-1].argmax()
    model.close()


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_interleaved_requests_and_slots_used_again(mixed, dtype):
    """Requests of unequal lengths take turns in their slots; each answers as
    alone, also in a slot and pages that another request has left."""
    model = qp.Model(mixed.path, 256, capacity=2, kv_page_tokens=32, kv_cache_dtype=dtype)
    rng = np.random.default_rng(8)
    other = rng.integers(0, mixed.config["vocab"], 120)
    expected = mo.forward(mixed.config, mm.float64(mixed.weights), other)[0]
    for _ in range(2):
        a, b = model.begin(), model.begin()
        with pytest.raises(qp.ProviderError, match="free request slot"):
            model.begin()
        got_a = [feed(model, a, mixed.tokens[:90], [90])]
        got_b = [feed(model, b, other[:5], [5])]
        for i in range(60):
            got_a.append(model.step(a, mixed.tokens[90 + 2 * i:92 + 2 * i], [0, 1])[0])
            got_b.append(model.step(b, other[5 + i:6 + i], [0])[0])
        assert distance(np.concatenate(got_a), mixed.logits).max() < 2 * LIMIT[dtype]
        assert distance(np.concatenate(got_b), expected[:65]).max() < 2 * LIMIT[dtype]
        model.end(b)
        c = model.begin()
        got = feed(model, c, other, [33, 1, 20])
        assert distance(got, expected).max() < 2 * LIMIT[dtype]
        model.end(c)
        model.end(a)
    model.close()


def test_long_decoding_lets_expired_pages_go(tmp_path):
    """Every layer's window is far shorter than the sequence: pages behind it
    return to the pool, those of the kept first tokens stay, and the logits are
    those of the whole sequence."""
    config = mm.configuration(64, 32, [mm.attention(2, 1, 16, 16, 40, 3),
                                       mm.general_delta(2, 8), mm.attention(4, 1, 16, 16, 24, 35),
                                       mm.wkv(1, 16)], [32, 0, 32, 0])
    weights = mm.random_weights(config, 3)
    path = mm.write_folder(tmp_path / "m", config, weights)
    tokens = np.random.default_rng(1).integers(0, 64, 500)
    want = mo.forward(config, mm.float64(weights), tokens)[0]
    for dtype in ("fp32", "bf16"):
        model = qp.Model(path, 512, kv_page_tokens=32, kv_cache_dtype=dtype)
        request = model.begin()
        got = feed(model, request, tokens[:60], [60])
        rows = [got] + [model.step(request, [t], [0])[0] for t in tokens[60:]]
        assert distance(np.concatenate(rows), want).max() < 2 * LIMIT[dtype]
        # two pages of kept tokens, those of the widest window, the current one
        assert model.telemetry("kv_allocated_pages") <= 2 + 3
        assert model.telemetry("provider_graph_launches") > 400
        model.end(request)
        model.close()


def test_context_limit_and_bad_batches(mixed):
    model = qp.Model(mixed.path, 64, kv_page_tokens=32)
    request = model.begin()
    with pytest.raises(qp.ProviderError, match="vocabulary"):
        model.step(request, [mixed.config["vocab"]])
    model.step(request, mixed.tokens[:64])
    with pytest.raises(qp.ProviderError, match="context"):
        model.step(request, mixed.tokens[64:65])
    model.end(request)
    model.close()


def test_missing_and_misshapen_tensors_are_named(tmp_path):
    config = mm.configuration(32, 16, [mm.wkv(1, 8)], [16])
    weights = mm.random_weights(config, 1)
    short = dict(weights)
    del short["l0.mix.u"]
    with pytest.raises(qp.ProviderError, match="l0.mix.u"):
        qp.Model(mm.write_folder(tmp_path / "a", config, short), 64)
    wrong = dict(weights)
    wrong["l0.mlp.up"] = weights["l0.mlp.up"][:8]
    with pytest.raises(qp.ProviderError, match="l0.mlp.up"):
        qp.Model(mm.write_folder(tmp_path / "b", config, wrong), 64)


def test_greedy_generation_through_the_worker(mixed):
    """Two requests through the worker's own loop and slots, 32-bit, equal to the
    plain statement token for token; bf16 equal to itself alone."""
    prompts = {7: mixed.tokens[:40], 9: mixed.tokens[50:53]}
    want = {}
    for request, prompt in prompts.items():
        want[request], margin = continuation(mixed, prompt, 24)
        assert margin > 1e-4
    for dtype in ("fp32", "bf16"):
        worker = wc.Worker(mixed.path, capacity=2, kv_page_tokens=32, kv_cache_dtype=dtype)
        assert worker.ready["architecture_id"] == "zatupel"
        assert worker.ready["kv_dtype"] == dtype
        alone = {}
        for request, prompt in prompts.items():
            assert worker.begin(request, 128, prompt)["type"] == "begun"
            alone[request] = [worker.next(request)["tokens"][0] for _ in range(24)]
            assert worker.ask("END", request)["type"] == "ended"
        if dtype == "fp32":
            assert alone == want
        for request, prompt in prompts.items():
            worker.begin(request, 128, prompt)
        together = {request: [] for request in prompts}
        for _ in range(24):
            reply = worker.ask("STEP", "7,0", "9,2")
            for item in reply["items"]:
                together[item["id"]] += item["tokens"]
        assert together == alone
        stats = worker.ask("STATS")
        assert stats["active_requests"] == 2 and stats["provider_graph_launches"] > 0
        for request in prompts:
            worker.ask("END", request)
        assert worker.ask("SHUTDOWN")["type"] == "shutdown"
        worker.close()


def test_sampling_follows_the_seed(mixed):
    model = qp.Model(mixed.path, 256, capacity=3, kv_page_tokens=32, kv_cache_dtype="fp32")

    def generate(**profile):
        request = model.begin(first_output_position=19, **profile)
        _, token = model.step(request, mixed.tokens[:20])
        out = [token]
        for _ in range(12):
            _, token = model.step(request, [token])
            out.append(token)
        model.end(request)
        return out

    profile = dict(temperature_ppm=1500000, top_p_ppm=950000, top_k=40)
    assert generate(seed=1, **profile) == generate(seed=1, **profile)
    assert generate(seed=1, **profile) != generate(seed=2, **profile)
    assert generate(temperature_ppm=1500000, top_k=0, seed=3) == generate(
        temperature_ppm=1500000, top_k=0, seed=3)
    greedy = generate()
    assert generate(temperature_ppm=1000000, top_k=1, seed=5) == greedy
    # a large penalty never lets a token come twice
    once = generate(presence_ppm=2000000)
    assert once[0] == greedy[0]
    model.close()


def test_trace_replay_program(mixed, tmp_path):
    import json
    import subprocess
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    lines = [
        {"step": 0, "entries": [{"id": "a", "tokens": mixed.tokens[:50].tolist(),
                                 "want": [49, 3]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": mixed.tokens[50:52].tolist(),
                                 "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": mixed.tokens[52:53].tolist(),
                                 "want": [0]}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "a", "tokens": mixed.tokens[:1].tolist(),
                                 "want": [0]}], "end": ["a"]},
    ]
    done = subprocess.run(
        [os.path.join(root, "bin", "trace_run"), "--model", mixed.path, "--dtype", "float32",
         "--out", str(tmp_path), "--max-tokens", "64"],
        input="".join(json.dumps(line) + "\n" for line in lines), capture_output=True,
        text=True, timeout=100)
    assert done.returncode == 0, done.stderr
    assert [line for line in done.stdout.splitlines() if line.startswith("done")] == [
        f"done {n}" for n in range(4)]
    assert not (tmp_path / "1.f32").exists()
    for step, places in ((0, [49, 3]), (2, [52]), (3, [0])):
        got = np.fromfile(tmp_path / f"{step}.f32", dtype="<f4").reshape(len(places), -1)
        assert distance(got, mixed.logits[places]).max() < LIMIT["fp32"]
