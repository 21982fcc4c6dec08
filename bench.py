#!/usr/bin/env python3
"""MTP-4 verify-step benchmark on one MI355X.

A "step" is one speculative verify call of the provider (execute_exact_decode):
target pass over 1 guaranteed + 4 draft rows of a random-init 27B-class dense
FP4 decoder (64 layers, hidden 5120, 64 Q / 8 KV heads, head_dim 128, SwiGLU
17408, vocabulary 151936, binary16 scale per 16 weights) with a Q4H KV cache
prefilled to 32768 tokens, greedy target distributions and accept-longest-
prefix.  Weights and KV contents are generated on the device before the timed
region; every step starts with all inputs resident in HBM.

Prints one JSON line: tok/s over the timed steps (emitted tokens / wall time),
the HBM roofline of the dominant kernel (fused gate/up FP4 GEMM) measured with
HIP events in this process, and a CPU baseline (the oracle's port of the same
arithmetic on the host cores, bounded sample).
"""
import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, os.path.join(ROOT, "tests"))
sys.path.insert(0, os.path.join(ROOT, "quantum-llm_amd", "python"))

HBM_PEAK_GBS = 8000.0
# HBM bytes one launch of the fused gate/up kernel moves, from the FETCH_SIZE and
# WRITE_SIZE hardware counters scaled by a 256 MiB copy (summary and commands
# in profiles/hot_kernels_hbm_traffic.md); 1.01x the algorithmic bytes.
GATE_UP_TRAFFIC_BYTES = 112914399

MODEL = dict(hidden=5120, intermediate=17408, layers=64, query_heads=64, kv_heads=8,
             head_dim=128, rotary_dim=128, vocabulary=151936, rope_theta=1.0e6,
             norm_epsilon=1.0e-6, output_gated=0, qk_norm=0, zero_centered_norm=0,
             scale_scheme=1, kv_encoding=0, kv_page_tokens=256, draft_depth=4)
CONTEXT = 32768


def fp4_bytes(rows, columns):
    """codes + binary16 scale per 16 columns."""
    return rows * columns // 2 + rows * (columns // 16) * 2


def cpu_baseline(rows):
    """CPU time of one verify step on the host cores, bounded sample.

    Linears: the reference's own all-core CPU executor
    (runtime/src/cpu/fp4_host_executor.cpp, FP4 ABI-3 weights x Q8 activations,
    AVX2), compiled from its source into oracle/_ref, timed on one layer's
    SwiGLU block (gate, up, down at the benchmark shape) and scaled by weight
    bytes to the seven linears of 64 layers plus lm_head.  Attention has no CPU
    path in the reference; its share is the oracle port (double precision,
    OpenMP) timed on one layer at 32768 tokens.  When oracle/_ref is absent the
    linears fall back to the oracle port as well (kind "port")."""
    import numpy as np

    import oracle_lib as ol
    import synth

    rng = np.random.default_rng(0)
    H, I, Q, KV, d = (MODEL["hidden"], MODEL["intermediate"], MODEL["query_heads"],
                      MODEL["kv_heads"], MODEL["head_dim"])
    cores = min(64, os.cpu_count() or 1)
    if os.environ.get("OMP_NUM_THREADS"):
        cores = min(cores, int(os.environ["OMP_NUM_THREADS"]))
    layer_parameters = (Q * d * H + 2 * KV * d * H + H * Q * d + 3 * I * H)
    ffn_parameters = 3 * I * H
    head_parameters = MODEL["vocabulary"] * H

    def abi3(n, k):
        return (rng.integers(0, 256, (n, k // 2), dtype=np.uint8),
                rng.integers(124, 131, (n, k // 32), dtype=np.uint8))

    reference = ol.ref() is not None and hasattr(ol.ref(), "qref_fp4_swiglu")
    x = rng.standard_normal((rows, H)).astype(np.float32)
    if reference:
        gate, up, down = abi3(I, H), abi3(I, H), abi3(H, I)
        _, ffn_seconds = ol.reference_fp4_swiglu(gate, up, down, H, I, x, threads=cores,
                                                 bf16_intermediate=True, repeats=8)
        linear_note = ("FP4 linears: reference CPU executor (fp4_host_executor.cpp, ABI-3 "
                       "weights x Q8, AVX2) on one layer's SwiGLU block, best of 8, scaled "
                       "by weight bytes to 7 linears x 64 layers + lm_head")
    else:
        codes = rng.integers(0, 256, (I // 8, H // 2), dtype=np.uint8)
        scales = np.exp(0.5 * rng.standard_normal((I // 8, H // 16))).astype(
            np.float16).view(np.uint16)
        act = ol.bf16_round(x)
        begin = time.perf_counter()
        ol.fp4_linear_f64(codes, scales, 1, I // 8, H, act)
        ffn_seconds = (time.perf_counter() - begin) * 8 * 3
        linear_note = ("FP4 linears: oracle port (double precision) on 1/8 of one "
                       "[17408, 5120] matrix, scaled by weight bytes")
    linear_seconds = ffn_seconds * (MODEL["layers"] * layer_parameters +
                                    head_parameters) / ffn_parameters
    keys = rng.standard_normal((CONTEXT + rows - 1, KV, d)).astype(np.float32)
    values = rng.standard_normal((CONTEXT + rows - 1, KV, d)).astype(np.float32)
    pages = synth.q4h_pages(keys, values, MODEL["kv_page_tokens"])
    query = rng.standard_normal((rows, Q, d)).astype(np.float32)
    shape = ol.AttentionShape(rows, Q, KV, d, CONTEXT, MODEL["kv_page_tokens"], 0, 0)
    begin = time.perf_counter()
    ol.attention_q4h(shape, query, pages, "f64")
    attention_seconds = (time.perf_counter() - begin) * MODEL["layers"]
    step_seconds = linear_seconds + attention_seconds
    return {
        "value": 1.0 / step_seconds,
        "unit": "tok/s",
        "cores": cores,
        "kind": "reference" if reference else "port",
        "sample": (linear_note + f"; Q4H attention at {CONTEXT} tokens: the reference has "
                   "no CPU attention, so the oracle port (double precision, OpenMP) on "
                   "one layer, x 64; one step emitting 1 token"),
        "seconds_per_step": step_seconds,
        "linears_seconds_per_step": linear_seconds,
        "attention_seconds_per_step": attention_seconds,
        "linears_only_tok_s": 1.0 / linear_seconds,
    }


def measure_decode_cycle(qp, np, rows, steps, warmup, sampled=False):
    """The whole decode cycle of the same model with the proposer inside the
    provider: verify step, proposer advance over the emitted tokens, rollout of
    the next four drafts (1 + 3 proposer passes over its Q8 cache, each ending
    in the 65536-row draft head).  Random-init weights accept almost nothing,
    so a cycle emits one token; the time per cycle is what real weights would
    see as well.  `sampled`: temperature 0.7, top-p 0.95, top-k 64 instead of
    greedy (rejection sampling on the host from the rows' top-k logits, the
    proposer returning to the host after every pass)."""
    geometry = dict(MODEL)
    geometry["mtp_layers"] = 1
    needed = CONTEXT + (steps + warmup + 2) * rows + 8
    geometry["max_context"] = (needed + 255) // 256 * 256
    provider = qp.Provider(**geometry)
    provider.load_synthetic_weights(20241125)
    provider.prefill_synthetic_kv(CONTEXT, 7)
    provider.prepare_exact_decode("decode.mtp.dense-full-attention.fp4-f16-block16.exact.v2")
    if sampled:
        provider.begin_request(temperature_ppm=700000, top_p_ppm=950000, top_k=64,
                               seed=20241125)
    else:
        provider.begin_request(temperature_ppm=0)
    token, position = 1, CONTEXT
    provider.synchronize(token, position)
    emitted = 0
    begin = passes = None
    for index in range(steps + warmup):
        if index == warmup:
            provider.synchronize_stream()
            begin = time.perf_counter()
            passes = provider.telemetry("provider_mtp_passes")
        tokens, token, advanced = provider.verify(token, position, geometry["max_context"])
        position += advanced
        if index >= warmup:
            emitted += len(tokens)
    provider.synchronize_stream()
    elapsed = time.perf_counter() - begin
    report = {
        "tok_s": round(emitted / elapsed, 2),
        "ms_per_cycle": round(1000.0 * elapsed / steps, 4),
        "cycles": steps,
        "emitted_tokens": emitted,
        "proposer_passes_per_cycle": round(
            (provider.telemetry("provider_mtp_passes") - passes) / steps, 2),
        "accepted_drafts": int(provider.telemetry("provider_accepted_drafts")),
        "projected_tok_s_at_reference_acceptance_2.6667": round(
            2.6667 * steps / elapsed, 1),
    }
    provider.close()
    return report


def measure_prefill(qp, np, prompt_tokens, chunk_rows=0):
    """Prompt prefill of the same model: `prompt_tokens` synthetic tokens from
    position 0 - the linears on the tall-batch GEMM (`chunk_rows` rows at a
    time, 0 = the provider's 32768), attention in six-row batches, one launch
    per chunk - timed from the call to the prediction of the token after the
    prompt (time to first token)."""
    rng = np.random.default_rng(11)
    tokens = rng.integers(0, MODEL["vocabulary"], prompt_tokens).astype(np.uint32)

    def timed(mtp_layers):
        geometry = dict(MODEL)
        geometry["mtp_layers"] = mtp_layers
        geometry["max_context"] = (prompt_tokens + 16 + 255) // 256 * 256
        geometry["prefill_chunk_rows"] = chunk_rows
        provider = qp.Provider(**geometry)
        provider.load_synthetic_weights(20241125)
        provider.prepare_exact_decode(
            "decode.mtp.dense-full-attention.fp4-f16-block16.exact.v2")
        provider.begin_request(temperature_ppm=0)
        provider.prefill(tokens[:min(prompt_tokens, 2048)], 0)      # warm-up, allocates
        provider.synchronize_stream()
        begin = time.perf_counter()
        provider.prefill(tokens, 0)
        seconds = time.perf_counter() - begin
        provider.close()
        return seconds

    elapsed = timed(0)
    # with the proposer inside the provider: its cache is filled from the
    # prompt and the first four drafts are rolled out before prefill returns
    with_proposer = timed(1)
    H, I, Q, KV, d = (MODEL["hidden"], MODEL["intermediate"], MODEL["query_heads"],
                      MODEL["kv_heads"], MODEL["head_dim"])
    linear_flops = 2.0 * prompt_tokens * MODEL["layers"] * (
        (Q + 2 * KV) * d * H + H * Q * d + 3 * I * H)
    report = {
        "prompt_tokens": prompt_tokens,
        "seconds_to_first_token": round(elapsed, 3),
        "seconds_to_first_token_and_drafts_with_proposer": round(with_proposer, 3),
        "tok_s": round(prompt_tokens / elapsed, 1),
        "linear_tflops_if_all_time_were_linears": round(linear_flops / elapsed / 1e12, 1),
        "reference_published_ttft_s_32k_rtx3090": 39.6,
    }
    return report


def measure_long_contexts(qp, np, rows):
    """tok/s of the same 64-layer verify step with the Q4H cache prefilled to
    131072 tokens, and the exact-F16 attention kernel over 262144 tokens
    (1.07 GB of K/V per layer; 4 layers of cache, so consecutive launches read
    different memory)."""
    report = {}
    context = 131072
    steps, warmup = 10, 2
    geometry = dict(MODEL)
    geometry["max_context"] = context + (steps + warmup + 2) * rows + 256
    geometry["max_context"] = (geometry["max_context"] + 255) // 256 * 256
    provider = qp.Provider(**geometry)
    provider.load_synthetic_weights(20241125)
    provider.prefill_synthetic_kv(context, 7)
    provider.prepare_exact_decode("decode.mtp.dense-full-attention.fp4-f16-block16.exact.v2")
    provider.begin_request(temperature_ppm=0)
    rng = np.random.default_rng(2)
    token, position = 1, context
    provider.synchronize(token, position)
    emitted = 0
    begin = None
    for index in range(steps + warmup):
        if index == warmup:
            provider.synchronize_stream()
            begin = time.perf_counter()
        provider.set_drafts(rng.integers(0, MODEL["vocabulary"],
                                         MODEL["draft_depth"]).astype(np.uint32))
        tokens, token, advanced = provider.verify(token, position, geometry["max_context"])
        position += advanced
        if index >= warmup:
            emitted += len(tokens)
    provider.synchronize_stream()
    elapsed = time.perf_counter() - begin
    attention_us, _ = provider.time_kernel("attention", 2, context)
    attention_bytes = context * MODEL["kv_heads"] * 2 * (MODEL["head_dim"] // 2 + 2)
    report["q4h_131072"] = {
        "tok_s": round(emitted / elapsed, 2),
        "ms_per_step": round(1000.0 * elapsed / steps, 4),
        "projected_tok_s_at_reference_acceptance_2.6667": round(
            2.6667 * steps / elapsed, 1),
        "attention_avg_launch_us": round(attention_us, 2),
        "attention_GBps": round(attention_bytes / attention_us / 1e3, 1),
        "attention_frac": round(attention_bytes / attention_us / 1e3 / HBM_PEAK_GBS, 4),
    }
    provider.close()

    context = 262144
    geometry = dict(MODEL)
    geometry.update(layers=4, kv_encoding=1, max_context=context + 512)
    provider = qp.Provider(**geometry)
    provider.load_synthetic_weights(3)
    provider.prefill_synthetic_kv(context, 9)
    attention_us, launches = provider.time_kernel("attention", 3, context)
    attention_bytes = context * MODEL["kv_heads"] * MODEL["head_dim"] * 2 * 2
    report["f16_attention_262144"] = {
        "avg_launch_us": round(attention_us, 2),
        "launches_timed": launches,
        "algorithmic_bytes_per_launch": attention_bytes,
        "achieved_GBps": round(attention_bytes / attention_us / 1e3, 1),
        "frac": round(attention_bytes / attention_us / 1e3 / HBM_PEAK_GBS, 4),
    }
    provider.close()
    return report


# Layers of about the size of a 1B and of a 7B model, four of them: attention,
# generalised delta rule, bonus recurrence, attention.
MIXED_SIZES = {
    "width-2048": dict(width=2048, ff=5632, heads=16, kv_heads=4, recurrent_heads=32,
                       query_rank=768),
    "width-4096": dict(width=4096, ff=14336, heads=32, kv_heads=8, recurrent_heads=64,
                       query_rank=1536),
}
MIXED_WINDOW, MIXED_KEPT, MIXED_VOCABULARY = 1024, 4, 32000


def measure_folder(qp, np, config, shapes, prompt_tokens, steps, warmup):
    """Prefill and greedy decode of a model folder's design (bf16, random weights).
    Prefill: from the call to the token after the prompt.  Decode: one token after
    the other through the program, each read back by the host.  Bytes are those of
    the weights a token reads."""
    import shutil
    import tempfile

    import mixed_model as mm

    folder = tempfile.mkdtemp()
    try:
        mm.write_folder(folder, config, mm.TiledWeights(shapes, 1))
        model = qp.Model(folder, prompt_tokens + warmup + steps + 8, kv_page_tokens=256)
    finally:
        shutil.rmtree(folder, ignore_errors=True)
    tokens = np.random.default_rng(0).integers(0, config["vocab"], prompt_tokens)
    prefill = []
    for _ in range(4):                   # the first one allocates and is not counted
        request = model.begin()
        begin = time.perf_counter()
        _, token = model.step(request, tokens)
        prefill.append(time.perf_counter() - begin)
        if len(prefill) < 4:
            model.end(request)
    for index in range(warmup + steps):
        if index == warmup:
            begin = time.perf_counter()
        _, token = model.step(request, [token])
    decode = (time.perf_counter() - begin) / steps
    read = model.telemetry("provider_weight_bytes") - 2 * config["vocab"] * config["width"]
    model.close()
    return {"prefill_tok_s": round(prompt_tokens / min(prefill[1:]), 1),
            "prefill_ms": round(1e3 * min(prefill[1:]), 3),
            "decode_tok_s": round(1.0 / decode, 1),
            "decode_us_per_token": round(1e6 * decode, 1),
            "decode_weight_GBps": round(read / decode / 1e9, 1)}


def mixed_configuration(size):
    import mixed_model as mm

    attention = mm.attention(size["heads"], size["kv_heads"], 128, 128, MIXED_WINDOW,
                             MIXED_KEPT)
    layers = [attention, mm.general_delta(size["recurrent_heads"], 64),
              mm.wkv(size["recurrent_heads"], 64), attention]
    config = mm.configuration(MIXED_VOCABULARY, size["width"], layers, [size["ff"]] * 4)
    return config, mm.shapes(config, 64)


def latent_configuration(size):
    import latent_model as lm

    windowed = lm.windowed_latent(size["heads"], 128, 64, 128, 512, size["query_rank"],
                                  MIXED_WINDOW, scaling=lm.yarn(8.0, 4096))
    recurrent = lm.gla(size["recurrent_heads"] // 2, 64, 128)
    layers = [recurrent, windowed, lm.latent(size["heads"], 128, 128, 512), windowed]
    config = lm.configuration(MIXED_VOCABULARY, size["width"], layers, [size["ff"]] * 4)
    return config, lm.shapes(config, 64)


def measure_latent(qp, np, prompt_tokens, steps, warmup):
    """The latent-attention decoder beside the mixed-layer decoder with as many
    layers of the same width, feed-forward, heads, state size and vocabulary."""
    report = {}
    for name, size in MIXED_SIZES.items():
        report[name] = measure_folder(qp, np, *latent_configuration(size), prompt_tokens,
                                      steps, warmup)
        other = measure_folder(qp, np, *mixed_configuration(size), prompt_tokens, steps,
                               warmup)
        report[name].update({"mixed_" + key: value for key, value in other.items()})
    return report


def measure_mixed(qp, np, prompt_tokens, steps, warmup):
    """The mixed-layer decoder beside the dense FP4 decoder with as many layers of
    the same width, feed-forward, heads and vocabulary.  The dense decoder's one-row
    target pass is replayed back to back (its decode step is speculative)."""
    report = {}
    for name, size in MIXED_SIZES.items():
        report[name] = measure_folder(qp, np, *mixed_configuration(size), prompt_tokens,
                                      steps, warmup)
        tokens = np.random.default_rng(0).integers(0, MIXED_VOCABULARY, prompt_tokens)
        geometry = dict(MODEL)
        geometry.update(hidden=size["width"], intermediate=size["ff"], layers=4,
                        query_heads=size["heads"], kv_heads=size["kv_heads"],
                        vocabulary=MIXED_VOCABULARY, max_context=prompt_tokens + 256)
        dense = qp.Provider(**geometry)
        dense.load_synthetic_weights(3)
        dense.prepare_exact_decode(
            "decode.mtp.dense-full-attention.fp4-f16-block16.exact.v2")
        dense.begin_request(temperature_ppm=0)
        dense_prefill = []
        for _ in range(4):
            begin = time.perf_counter()
            dense.prefill(tokens.astype(np.uint32), 0)
            dense_prefill.append(time.perf_counter() - begin)
        dense.capture_target(np.array([5], np.uint32), MIXED_WINDOW)
        for index in range(warmup + steps):
            if index == warmup:
                dense.synchronize_stream()
                begin = time.perf_counter()
            dense.replay_target()
        dense.synchronize_stream()
        dense_decode = (time.perf_counter() - begin) / steps
        dense.close()
        report[name].update({
            "dense_fp4_prefill_tok_s": round(prompt_tokens / min(dense_prefill[1:]), 1),
            "dense_fp4_prefill_ms": round(1e3 * min(dense_prefill[1:]), 3),
            "dense_fp4_one_row_pass_us": round(1e6 * dense_decode, 1),
        })
    return report


def main():
    parser = argparse.ArgumentParser()
    parser.add_argument("--gpus", type=int, default=1)
    parser.add_argument("--steps", type=int, default=40)
    parser.add_argument("--warmup", type=int, default=5)
    parser.add_argument("--layers", type=int, default=MODEL["layers"],
                        help="for quick experiments only; the reported config is 64")
    parser.add_argument("--no-cpu-baseline", action="store_true")
    parser.add_argument("--skip-long-contexts", action="store_true",
                        help="skip the 131072-token step and the 262144-token F16 "
                             "attention measurements")
    parser.add_argument("--skip-decode-cycle", action="store_true",
                        help="leave out the decode cycle with the proposer (a second "
                             "provider with the MTP layer)")
    parser.add_argument("--prefill-chunk-rows", type=int, default=0,
                        help="prompt rows per pass of the tall linears (0 = the "
                             "provider's default)")
    parser.add_argument("--prefill-tokens", type=int, default=32768,
                        help="prompt length of the prefill leg (0 skips it; the "
                             "default is the context of the headline metric, for "
                             "which the reference publishes its time to first token)")
    parser.add_argument("--mixed", action="store_true",
                        help="measure the mixed-layer decoder (prefill and decode at "
                             "two sizes, beside the dense decoder) instead of the "
                             "verify step")
    parser.add_argument("--latent", action="store_true",
                        help="measure the latent-attention decoder (prefill and decode "
                             "at two sizes, beside the mixed-layer decoder) instead of "
                             "the verify step")
    parser.add_argument("--mixed-prompt-tokens", type=int, default=4096,
                        help="prompt length of --mixed and --latent")
    parser.add_argument("--calibration-copy", action="store_true",
                        help="also run one 256 MiB device copy (a kernel of known "
                             "traffic to scale hardware counters by)")
    arguments = parser.parse_args()
    if arguments.gpus != 1:
        print("bench.py: this build runs the verify step on ONE GPU only "
              f"(--gpus {arguments.gpus} is not supported; there are no collectives "
              "on this path)", file=sys.stderr)
        return 2

    import numpy as np
    import torch

    import qllm_provider as qp

    if not torch.cuda.is_available():
        print("bench.py: no GPU visible", file=sys.stderr)
        return 1
    rows = MODEL["draft_depth"] + 1
    steps, warmup = arguments.steps, arguments.warmup
    if arguments.mixed or arguments.latent:
        measure, kind, design = ((measure_latent, "latent-attention", "Nametar")
                                 if arguments.latent else
                                 (measure_mixed, "mixed-layer", "Zatupel"))
        report = measure(qp, np, arguments.mixed_prompt_tokens, steps, warmup)
        first = report["width-2048"]
        print(json.dumps({
            "metric": kind + " decoder decode tok/s", "value": first["decode_tok_s"],
            "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warmup,
            "ms_per_step": round(first["decode_us_per_token"] / 1e3, 4),
            "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
            "dtype": "bf16", "data": "synthetic", "sizes": report,
            "config": {"model": design + "-shaped, 4 layers, random weights",
                       "global_batch": 1, "seq_len": arguments.mixed_prompt_tokens,
                       "parallelism": "none"}}))
        return 0
    geometry = dict(MODEL)
    geometry["layers"] = arguments.layers
    # room for every step to advance by up to 5 positions
    needed = CONTEXT + (steps + warmup + 2) * rows + 8
    geometry["max_context"] = (needed + 255) // 256 * 256
    provider = qp.Provider(**geometry)
    provider.load_synthetic_weights(20241125)
    provider.prefill_synthetic_kv(CONTEXT, 7)
    tag = "fp4-f16-block16"
    provider.prepare_exact_decode(f"decode.mtp.dense-full-attention.{tag}.exact.v2")
    provider.begin_request(temperature_ppm=0)

    rng = np.random.default_rng(1)
    vocabulary = MODEL["vocabulary"]
    position = CONTEXT
    token = int(rng.integers(0, vocabulary))
    provider.synchronize(token, position)

    def step():
        nonlocal token, position
        drafts = rng.integers(0, vocabulary, MODEL["draft_depth"]).astype(np.uint32)
        provider.set_drafts(drafts)
        emitted, next_token, advanced = provider.verify(
            token, position, geometry["max_context"])
        token, position = next_token, position + advanced
        return len(emitted)

    for _ in range(warmup):
        step()
    provider.synchronize_stream()
    torch.cuda.synchronize()
    begin = time.perf_counter()
    emitted_tokens = 0
    for _ in range(steps):
        emitted_tokens += step()
    provider.synchronize_stream()
    torch.cuda.synchronize()
    elapsed = time.perf_counter() - begin
    ms_per_step = 1000.0 * elapsed / steps
    tokens_per_second = emitted_tokens / elapsed

    # dominant kernel: fused gate/up FP4 GEMM of the SwiGLU block
    H, I = MODEL["hidden"], MODEL["intermediate"]
    kernel_us, launches = provider.time_kernel("ffn_gate_up", 4)
    kernel_bytes = 2 * fp4_bytes(I, H) + rows * H * 2 + rows * I * 2
    achieved = kernel_bytes / kernel_us / 1e3   # GB/s
    roofline = {
        "bound": "hbm",
        "kernel": "fp4_gemm_mfma_kernel (fused gate/up, [2x17408, 5120], M=5)",
        "achieved": round(achieved, 1),
        "peak": HBM_PEAK_GBS,
        "unit": "GB/s",
        "frac": round(achieved / HBM_PEAK_GBS, 4),
        "traffic": GATE_UP_TRAFFIC_BYTES if geometry["layers"] == MODEL["layers"] else None,
        "algorithmic_bytes_per_launch": kernel_bytes,
        "avg_launch_us": round(kernel_us, 3),
        "launches_timed": launches,
    }
    other_kernels = {}
    qkv_rows = (MODEL["query_heads"] + 2 * MODEL["kv_heads"]) * MODEL["head_dim"]
    attention_width = MODEL["query_heads"] * MODEL["head_dim"]
    for name, bytes_per_launch in (
            ("qkv", fp4_bytes(qkv_rows, H) + rows * H * 2 + rows * qkv_rows * 4),
            ("attention_output", fp4_bytes(H, attention_width) + rows * attention_width * 2
             + rows * H * 4),
            ("ffn_down", fp4_bytes(H, I) + rows * I * 2 + rows * H * 4),
            ("lm_head", fp4_bytes(vocabulary, H) + rows * H * 2 + rows * vocabulary * 4),
            ("attention", CONTEXT * MODEL["kv_heads"] * 2 * (MODEL["head_dim"] // 2 + 2)
             + 2 * rows * MODEL["query_heads"] * MODEL["head_dim"] * 2)):
        us, _ = provider.time_kernel(name, 16 if name == "lm_head" else 4, CONTEXT)
        other_kernels[name] = {"avg_launch_us": round(us, 3),
                               "achieved_GBps": round(bytes_per_launch / us / 1e3, 1),
                               "frac": round(bytes_per_launch / us / 1e3 / HBM_PEAK_GBS, 4)}
    other_kernels["attention"]["launches"] = (
        "rotary + Q4H store + query quantisation + attention split in one launch, then "
        "the split combine; the separate rotary launch it replaces took 5.2 us")
    other_kernels["lm_head"]["weights"] = (
        "cold: every timed launch follows > 640 MB of other weight reads")

    # the other contexts of the metric: the same step at 131072 tokens (Q4H) and
    # the exact-F16 attention kernel at 262144 tokens, on providers of their own
    weight_bytes = provider.weight_bytes()
    accepted_drafts = int(provider.telemetry("provider_accepted_drafts"))
    long_context = {}
    decode_cycle = {}
    if arguments.layers == MODEL["layers"] and not arguments.skip_decode_cycle:
        provider.close()
        provider = None
        decode_cycle = measure_decode_cycle(qp, np, rows, min(steps, 20), min(warmup, 3))
        sampled = measure_decode_cycle(qp, np, rows, min(steps, 20), min(warmup, 3),
                                       sampled=True)
        decode_cycle["sampled_t0.7_top_p0.95_top_k64"] = {
            key: sampled[key] for key in ("tok_s", "ms_per_cycle", "emitted_tokens",
                                          "accepted_drafts")}
    if arguments.layers == MODEL["layers"] and not arguments.skip_long_contexts:
        if provider is not None:
            provider.close()
        provider = None
        long_context = measure_long_contexts(qp, np, rows)
    prefill = {}
    if arguments.layers == MODEL["layers"] and arguments.prefill_tokens > 0:
        if provider is not None:
            provider.close()
        provider = None
        prefill = measure_prefill(qp, np, arguments.prefill_tokens,
                                  arguments.prefill_chunk_rows)
    layers = geometry["layers"]
    step_bytes = (layers * (fp4_bytes(MODEL["query_heads"] * 128, H) +
                            2 * fp4_bytes(MODEL["kv_heads"] * 128, H) +
                            fp4_bytes(H, MODEL["query_heads"] * 128) +
                            2 * fp4_bytes(I, H) + fp4_bytes(H, I) +
                            CONTEXT * MODEL["kv_heads"] * 2 * 66) +
                  fp4_bytes(vocabulary, H))
    result = {
        "metric": "MTP-4 decode tok/s at 32K ctx (verify step)",
        "value": round(tokens_per_second, 2),
        "unit": "tok/s",
        "n_gpus": 1,
        "steps": steps,
        "warmup": warmup,
        "ms_per_step": round(ms_per_step, 4),
        "higher_is_better": True,
        "scaling": "weak",
        "vs_baseline": None,
        "dtype": "fp4 weights x bf16 activations, f32 accumulate",
        "data": "synthetic",
        "config": {
            "workload": ("full MTP-4 verify step, 27B-class dense FP4 decoder, "
                         f"{layers} layers, hidden 5120, 64Q/8KV heads, head_dim 128, "
                         "FFN 17408, vocab 151936, Q4H KV prefilled to 32768 tokens, "
                         "greedy acceptance, 5 rows (1 guaranteed + 4 random drafts)"),
            "context_tokens": CONTEXT,
            "rows": rows,
            "emitted_tokens": emitted_tokens,
            "accepted_drafts": accepted_drafts,
            "weight_bytes": int(weight_bytes),
            "algorithmic_bytes_per_step": int(step_bytes),
            "step_hbm_GBps": round(step_bytes / (ms_per_step * 1e-3) / 1e9, 1),
            "step_roofline_frac": round(step_bytes / (ms_per_step * 1e-3) / 1e9 /
                                        HBM_PEAK_GBS, 4),
            "reference_published_tok_s_rtx3090": 54.54,
            # the verify step alone: no proposer passes in the timed region (the
            # decode cycle below has them and carries the projection that can be
            # set next to the reference's end-to-end figure)
            "verify_only_projected_tok_s_at_reference_acceptance_2.6667": round(
                2.6667 * 1000.0 / ms_per_step, 1),
        },
        "roofline": roofline,
        "kernels": other_kernels,
    }
    if provider is not None:
        provider.close()
    if decode_cycle:
        result["decode_cycle_with_proposer"] = decode_cycle
    if long_context:
        result["long_context"] = long_context
    if prefill:
        result["prompt_prefill"] = prefill
    if arguments.calibration_copy:
        source = torch.empty(256 << 20, dtype=torch.uint8, device="cuda:0")
        target = torch.empty_like(source)
        target.copy_(source)
        torch.cuda.synchronize()
    if not arguments.no_cpu_baseline:
        result["cpu_baseline"] = cpu_baseline(rows)
    print(json.dumps(result))
    return 0


if __name__ == "__main__":
    sys.exit(main())
