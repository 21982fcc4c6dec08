"""Whole latent-attention models through the framework's own entry points: the
model folder, the compiled program, request slots and pages, sampling, the
worker, the trace replay - against the plain float64 statement."""
import json
import os
import subprocess

import numpy as np
import pytest

import latent_model as lm
import latent_oracle as lo
import mixed_model as mm
import qllm_provider as qp
import worker_client as wc
from model_util import LIMIT, Case, continuation, distance, feed

pytestmark = pytest.mark.gpu


def configurations():
    return {
        # layer order, unequal sizes, feed-forwards on some layers only
        "unequal": lm.configuration(
            150, 96, [lm.windowed_latent(6, 40, 16, 24, 56, 48, 19, base=500.0),
                      lm.gla(3, 24, 40), lm.latent(5, 32, 24, 40),
                      lm.gla(2, 40, 16, tau=4.0),
                      lm.windowed_latent(3, 48, 24, 40, 72, 30, 33, base=1e5, scale=0.2)],
            [70, 130, 0, 0, 96], eps=1e-4, scale=0.7, residual=0.6),
        # sizes of one, odd sizes, factors of one (a norm over one value is its sign
        # unless the epsilon is large)
        "small": lm.configuration(
            33, 18, [lm.latent(1, 5, 3, 7), lm.gla(1, 1, 1, tau=1.0), lm.gla(3, 2, 5),
                     lm.windowed_latent(1, 6, 2, 5, 9, 4, 1, scaling=lm.yarn(1.0, 64))],
            [1, 17, 0, 5], eps=0.3, scale=1.0, residual=1.0),
        # many heads, wide latents, a window of a page
        "wide": lm.configuration(
            260, 128, [lm.windowed_latent(20, 16, 64, 24, 260, 96, 64, scaling=lm.yarn(8.0, 64)),
                       lm.gla(1, 128, 200), lm.latent(33, 8, 16, 130)],
            [256, 0, 128], scale=3.0),
    }


CONFIGS = configurations()


def agree(got, want, dtype):
    """The norms behind the sublayers enlarge what rounding does to a small output,
    so single rows stand out more than in the mean."""
    errors = distance(got, want)
    assert errors.mean() < LIMIT[dtype] and errors.max() < 4 * LIMIT[dtype], errors.max()


def case_of(name, folder):
    config = CONFIGS[name]
    return Case(config, lm.random_weights(config, 11), lo.forward, folder)


@pytest.fixture(scope="module", params=list(CONFIGS))
def case(request, tmp_path_factory):
    return case_of(request.param, tmp_path_factory.mktemp(request.param))


@pytest.fixture(scope="module")
def unequal(tmp_path_factory):
    return case_of("unequal", tmp_path_factory.mktemp("one"))


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
    agree(got, case.logits, dtype)
    model.close()


def test_batches_longer_than_the_program_takes_at_once(unequal):
    model = qp.Model(unequal.path, 256, kv_page_tokens=32, kv_cache_dtype="fp32", chunk_rows=48)
    request = model.begin()
    got, token = model.step(request, unequal.tokens, range(210))
    assert distance(got, unequal.logits).max() < LIMIT["fp32"]
    assert token == unequal.logits[-1].argmax()
    model.close()


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_interleaved_requests_and_slots_used_again(unequal, dtype):
    """Requests of unequal lengths take turns in their slots; each answers as
    alone, also in a slot and pages that another request has left."""
    model = qp.Model(unequal.path, 256, capacity=2, kv_page_tokens=32, kv_cache_dtype=dtype)
    rng = np.random.default_rng(8)
    other = rng.integers(0, unequal.config["vocab"], 120)
    expected = unequal.expect(other)[0]
    for _ in range(2):
        a, b = model.begin(), model.begin()
        got_a = [feed(model, a, unequal.tokens[:90], [90])]
        got_b = [feed(model, b, other[:5], [5])]
        for i in range(60):
            got_a.append(model.step(a, unequal.tokens[90 + 2 * i:92 + 2 * i], [0, 1])[0])
            got_b.append(model.step(b, other[5 + i:6 + i], [0])[0])
        agree(np.concatenate(got_a), unequal.logits, dtype)
        agree(np.concatenate(got_b), expected[:65], dtype)
        model.end(b)
        c = model.begin()
        got = feed(model, c, other, [33, 1, 20])
        agree(got, expected, dtype)
        model.end(c)
        model.end(a)
    model.close()


def test_workspace_grows_with_the_context_between_decoded_tokens(tmp_path):
    """A long portion after decoding: the buffers that a captured token addresses
    are replaced, and decoding goes on over them."""
    config = lm.configuration(64, 32, [lm.latent(2, 16, 16, 24),
                                       lm.windowed_latent(2, 16, 8, 16, 24, 16, 100)], [32, 0])
    case = Case(config, lm.random_weights(config, 5), lo.forward, tmp_path / "m", tokens=700)
    for dtype in ("fp32", "bf16"):
        model = qp.Model(case.path, 768, kv_page_tokens=64, kv_cache_dtype=dtype)
        request = model.begin()
        got = feed(model, request, case.tokens, [5] + [1] * 6 + [300] + [1] * 6 + [370, 1])
        agree(got, case.logits, dtype)
        model.close()


def test_long_decoding_lets_expired_pages_go(tmp_path):
    """Every attention layer's window is far shorter than the sequence: pages behind
    it return to the pool, and the logits are those of the whole sequence."""
    config = lm.configuration(64, 32, [lm.windowed_latent(2, 16, 8, 16, 24, 16, 40),
                                       lm.gla(2, 8, 12),
                                       lm.windowed_latent(4, 16, 16, 16, 20, 12, 24),
                                       lm.gla(1, 16, 8)], [32, 0, 32, 0])
    case = Case(config, lm.random_weights(config, 3), lo.forward, tmp_path / "m", tokens=500)
    for dtype in ("fp32", "bf16"):
        model = qp.Model(case.path, 512, kv_page_tokens=32, kv_cache_dtype=dtype)
        request = model.begin()
        rows = [feed(model, request, case.tokens[:60], [60])]
        rows += [model.step(request, [t], [0])[0] for t in case.tokens[60:]]
        agree(np.concatenate(rows), case.logits, dtype)
        # those of the widest window, the current one
        assert model.telemetry("kv_allocated_pages") <= 3
        assert model.telemetry("provider_graph_launches") > 400
        model.end(request)
        # the pages serve the next request
        again = model.begin()
        got = feed(model, again, case.tokens[:130], [100, 1])
        agree(got, case.logits[:130], dtype)
        model.close()


def test_missing_and_misshapen_tensors_are_named(tmp_path):
    config = lm.configuration(32, 16, [lm.windowed_latent(2, 8, 4, 8, 12, 10, 5)], [16])
    weights = lm.random_weights(config, 1)
    for index, name in enumerate(("l0.mix.uk", "l0.norm1b", "l0.mix.dq.norm", "l0.norm2b")):
        short = {key: value for key, value in weights.items() if key != name}
        with pytest.raises(qp.ProviderError, match=name):
            qp.Model(mm.write_folder(tmp_path / f"a{index}", config, short), 64)
        wrong = dict(weights)
        wrong[name] = weights[name][:-1]
        with pytest.raises(qp.ProviderError, match=name):
            qp.Model(mm.write_folder(tmp_path / f"b{index}", config, wrong), 64)


def test_greedy_generation_through_the_worker(unequal):
    """Two requests through the worker's own loop and slots, 32-bit, equal to the
    plain statement token for token; bf16 equal to itself alone."""
    prompts = {7: unequal.tokens[:40], 9: unequal.tokens[50:53]}
    want = {}
    for request, prompt in prompts.items():
        want[request], margin = continuation(unequal, prompt, 24)
        assert margin > 1e-4
    for dtype in ("fp32", "bf16"):
        worker = wc.Worker(unequal.path, capacity=2, kv_page_tokens=32, kv_cache_dtype=dtype)
        assert worker.ready["architecture_id"] == "nametar"
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


def test_trace_replay_program(unequal, tmp_path):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    tokens = unequal.tokens.tolist()
    lines = [
        {"step": 0, "entries": [{"id": "a", "tokens": tokens[:50], "want": [49, 3]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": tokens[50:52], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": tokens[52:53], "want": [0]}],
         "end": ["a"]},
        {"step": 3, "entries": [{"id": "a", "tokens": tokens[:1], "want": [0]}], "end": ["a"]},
    ]
    for dtype, limit in (("float32", LIMIT["fp32"]), ("bfloat16", 4 * LIMIT["bf16"])):
        out = tmp_path / dtype
        out.mkdir()
        done = subprocess.run(
            [os.path.join(root, "bin", "trace_run"), "--model", unequal.path, "--dtype", dtype,
             "--out", str(out), "--max-tokens", "64"],
            input="".join(json.dumps(line) + "\n" for line in lines), capture_output=True,
            text=True, timeout=100)
        assert done.returncode == 0, done.stderr
        assert [line for line in done.stdout.splitlines() if line.startswith("done")] == [
            f"done {n}" for n in range(4)]
        assert not (out / "1.f32").exists()
        for step, places in ((0, [49, 3]), (2, [52]), (3, [0])):
            got = np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(places), -1)
            assert distance(got, unequal.logits[places]).max() < limit
