#!/usr/bin/env python3
"""Decode and prefill throughput of the engine on one MI355X, Qwen3-8B layer sizes, bfloat16,
random weights.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--context 8192] [--shape 8B|14B|32B] [--layers L]

A step is one decode step of the whole batch: the step function over one token per request,
greedy choice of the next token on the device, and feeding it back.  The requests' caches are
brought to the benchmark's context length by filling their pages with random keys and values
(decode time does not depend on their content); the prefill figure is measured separately
on a 2,048-token prompt through the same step function.  One JSON line is printed.

    python bench.py --workload mixed16|concurrent32 [--shape ...] [--decode-tokens T]

runs requests through the serving loop instead (scheduler, prompt portions beside decode tokens, greedy
choice): `mixed16` is 16 requests with prompts of 128 to 4,096 random tokens in portions of 512 at the
14B shape, `concurrent32` 32 requests of 1,024 prompt tokens at the 32B shape; every request decodes
`--decode-tokens` tokens.  Its JSON line gives tokens a second over the whole run, the prompts' and the
decoded tokens' rates apart, and the time to a request's first token.

    python bench.py --design buketar|lofudra|fisanex|ligizen|vufizen|lumedra [--design-shapes 1k,2k,4k]

measures the Buketar design (latent attention, gated recurrences, routed experts, residual streams), the Lofudra
design (windowed sink attention beside retention, matrix memory, state space, norms on both sides) or the Fisanex design
(a stream normed after every sum, gated window attention with values narrower than keys over caches that layers share,
routed experts with outputs that hand the input on and a shared expert) at a few layer
sizes beside the dense decoder at equal width, layers and feed-forward products a token, or the Ligizen design (one layer
norm a layer that both sub-layers read, latent window attention with learned sinks beside chunked attention over caches
that layers share, experts weighted on their inputs, a token's own input a layer) beside the Fisanex design at equal size,
or the Vufizen design (gated, normed branches; differential attention behind a short convolution beside a matrix state that fades
by a gate a channel; routed experts in every layer) beside the Fisanex and the Lofudra design at equal width and layers, or the
Lumedra design (two norms of one stream a layer; lightning attention, latent attention and capped window attention beside first
tokens that stay, over mixed values; experts chosen inside the best groups) beside the Ligizen and the Lofudra design: prompts of `--prefill-tokens`
tokens, decode steps at `--batch` and at batch 1 through the serving loop, and every kernel's time in one prompt and one
decode step of both.  One JSON line; the default record above is not touched by it.

The reference measures the same quantities with `inferrs bench` (`inferrs/src/bench.rs:40-224`,
`Engine::bench_generate`, `inferrs/src/engine.rs:2557-2641`): synthetic prompt, stop tokens
ignored, device-synchronised wall time.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

# Qwen3-8B as its config.json gives it.
QWEN3_8B = dict(architectures=["Qwen3ForCausalLM"], model_type="qwen3", vocab_size=151936,
                hidden_size=4096, intermediate_size=12288, num_hidden_layers=36,
                num_attention_heads=32, num_key_value_heads=8, head_dim=128, rope_theta=1000000.0,
                rms_norm_eps=1e-6, tie_word_embeddings=False, max_position_embeddings=40960)
# The larger dense models of the family differ in these sizes only.
QWEN3_14B = dict(QWEN3_8B, hidden_size=5120, intermediate_size=17408, num_hidden_layers=40, num_attention_heads=40)
QWEN3_32B = dict(QWEN3_8B, hidden_size=5120, intermediate_size=25600, num_hidden_layers=64, num_attention_heads=64)
# The smallest shape is the one that the reference's defaults describe (`inferrs/src/config.rs:468-502`: width 1,024, 28 layers,
# 16 query and 8 key/value heads, feed-forward 3,072, tied embeddings); two more small ones between it and the 8B shape.
QWEN3_0_6B = dict(QWEN3_8B, hidden_size=1024, intermediate_size=3072, num_hidden_layers=28, num_attention_heads=16,
                  tie_word_embeddings=True)
QWEN3_1_7B = dict(QWEN3_0_6B, hidden_size=2048, intermediate_size=6144)
QWEN3_4B = dict(QWEN3_0_6B, hidden_size=2560, intermediate_size=9728, num_hidden_layers=36, num_attention_heads=32)
SHAPES = {"0.6B": QWEN3_0_6B, "1.7B": QWEN3_1_7B, "4B": QWEN3_4B, "8B": QWEN3_8B, "14B": QWEN3_14B, "32B": QWEN3_32B}
PEAK_HBM_GBS = 8000.0
PEAK_FLOPS = {"bf16": 2.5e15, "fp32": 157.3e12}
PREFILL_TOKENS = 2048
PAGE = 16


def matmul_params(c) -> int:
    """Weights of one layer's matrix products."""
    h, d = c["hidden_size"], c["head_dim"]
    qkv = (c["num_attention_heads"] + 2 * c["num_key_value_heads"]) * d * h
    return qkv + c["num_attention_heads"] * d * h + 3 * h * c["intermediate_size"]


def prefill_flops(c, t: int, rows_of_logits: int = 1) -> float:
    linear = 2.0 * t * matmul_params(c) * c["num_hidden_layers"]
    # causal scores and weighted values: 2 products of t(t+1)/2 x head_dim per query head
    attn = 4.0 * (t * (t + 1) / 2) * c["head_dim"] * c["num_attention_heads"] * c["num_hidden_layers"]
    return linear + attn + 2.0 * rows_of_logits * c["vocab_size"] * c["hidden_size"]


def decode_bytes(c, batch: int, context: float, esize: int = 2) -> float:
    """What one decode step has to read: every weight it uses once, and the cache of the live requests."""
    weights = (matmul_params(c) + 2 * c["hidden_size"] + 2 * c["head_dim"]) * c["num_hidden_layers"]
    weights += c["vocab_size"] * c["hidden_size"] + c["hidden_size"]          # logits head, final norm
    kv = 2 * c["num_key_value_heads"] * c["head_dim"] * c["num_hidden_layers"] * context * batch
    return float(weights * esize + kv * esize + batch * c["hidden_size"] * esize)


def fill_storage(engine) -> None:
    """Random keys and values in every page of the cache (decode time does not depend on their content)."""
    import torch
    gen = torch.Generator(device=engine.device).manual_seed(1)
    for arr in engine.storage.arrays:
        flat = arr.view(-1)
        step = 1 << 28
        for i in range(0, flat.numel(), step):
            part = flat[i:i + step]
            part.copy_(torch.randn(part.numel(), generator=gen, device=engine.device, dtype=torch.float32)
                       .mul_(0.5).to(arr.dtype))


def fill_context(engine, ids, context: int) -> None:
    """Gives each request `context` cached tokens without running them: pages are reserved (they hold the
    random keys and values of `fill_storage`)."""
    for sid in ids:
        engine.add_request(sid)
        if not engine.cache.reserve(sid, context):
            raise RuntimeError("the cache pool is too small for the benchmark's context")
        engine.cache.commit(sid, context)


def time_decode(engine, batch: int, context: int, steps: int, warmup: int, decode_run: int = 8, sampled: bool = False):
    """(seconds for `steps` steps, mean context length during them).  The steps go through the
    serving loop: scheduler, step function, greedy choice on the device; with `sampled` the choice is a draw
    with the reference's default parameters (temperature 0.7, top_k 50, top_p 0.9, repetition penalty 1.1
    over 64 tokens: `inferrs/src/main.rs:144-154`, `inferrs/src/sampler.rs:96-97`) and a fixed seed."""
    import torch
    from inferrs_amd.engine import GenerationLoop
    from inferrs_amd.engine.scheduler import Request
    from inferrs_amd.sampling import SamplingParams
    start_len = context - steps - warmup
    loop = GenerationLoop(engine, max_batch_size=batch, max_tokens_per_step=max(batch, 16), decode_run=decode_run)
    if sampled:
        params = SamplingParams(max_tokens=steps + warmup + 8, bypass_stop_tokens=True, seed=7)
    else:
        params = SamplingParams.greedy(max_tokens=steps + warmup + 8, bypass_stop_tokens=True)
    ids = [f"d{i}" for i in range(batch)]
    # the requests enter as if their contexts had been run: random keys and values, and one generated token
    fill_context(engine, ids, start_len)
    for i, sid in enumerate(ids):
        loop.scheduler.adopt(Request(sid, [1] * start_len, params, output=[1 + i]))
    done_steps = 0
    while done_steps < warmup:
        loop.step(max_steps=warmup - done_steps)
        done_steps = loop.steps
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    while loop.steps < warmup + steps:
        loop.step(max_steps=warmup + steps - loop.steps)
    torch.cuda.synchronize()
    elapsed = time.perf_counter() - t0
    for sid in ids:
        if engine.has_request(sid):
            engine.end_request(sid)
    return elapsed, start_len + warmup + (steps - 1) / 2.0


def time_prefill(engine, n_tokens: int, runs: int, vocab: int):
    """Seconds of each of `runs` prefills of one prompt of `n_tokens` tokens, after three that are not counted: a shape's
    first steps run eagerly and, where the host is their bound, the third is captured into a graph (prompts of up to
    `Engine.GRAPH_MAX_TOKENS` tokens), so the counted runs are what a repeated shape settles at (the reference's own
    bench counts five runs after one warm-up, `inferrs/src/bench.rs:27-33`)."""
    import torch
    from inferrs_amd.engine import Entry
    g = torch.Generator().manual_seed(2)
    prompt = torch.randint(0, vocab, (n_tokens,), generator=g).tolist()
    times = []
    for r in range(runs + 3):
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        engine.step([Entry("p", prompt, [n_tokens - 1])])
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        engine.end_request("p")
        if r > 2:
            times.append(dt)
    return times


def mean_std(values):
    m = sum(values) / len(values)
    var = sum((v - m) ** 2 for v in values) / max(len(values) - 1, 1)
    return m, var ** 0.5


def measured_roofs(engine):
    """(GB/s of a pure streaming read over at least 4 GB, TFLOP/s of a large bfloat16 product through the vendor's
    GEMM): what this GPU gives in practice, beside the published peaks."""
    import torch
    from inferrs_amd import ops
    src = max(engine.storage.arrays, key=lambda a: a.numel() * a.element_size()).view(-1)
    want = 8 << 30
    n = min(src.numel(), want // src.element_size()) // 64 * 64
    if n * src.element_size() < (4 << 30):                  # a small cache: a buffer of its own
        src = torch.empty(4 << 30, dtype=torch.uint8, device=engine.device).random_(0, 255)
        n = src.numel()
    part = src[:n]
    best = None
    for blocks in (8192, 16384, 65536):
        for _ in range(3):
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            ops.stream_read(part, blocks)
            b.record()
            torch.cuda.synchronize()
            gbs = n * part.element_size() / (a.elapsed_time(b) * 1e-3) / 1e9
            best = gbs if best is None else max(best, gbs)
    m = 8192
    x = torch.randn(m, m, device=engine.device, dtype=torch.bfloat16)
    w = torch.randn(m, m, device=engine.device, dtype=torch.bfloat16)
    torch.nn.functional.linear(x, w)
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(10):
        torch.nn.functional.linear(x, w)
    b.record()
    torch.cuda.synchronize()
    tflops = 10 * 2.0 * m ** 3 / (a.elapsed_time(b) * 1e-3) / 1e12
    return best, tflops


def kernel_breakdown(engine, batch: int, context: int, prefill_tokens: int, vocab: int):
    """Microseconds by kernel entry point for one decode step (batch, context) and one prefill, each kernel call
    bracketed by events (eager steps, no graph; an event pair adds a few microseconds to a short kernel)."""
    import torch
    from inferrs_amd import ops
    from inferrs_amd.engine import Entry
    out = {}
    ids = [f"k{i}" for i in range(batch)]
    fill_context(engine, ids, context - 4)
    graphs, engine.use_graphs = engine.use_graphs, False
    try:
        entries = [Entry(sid, [1 + i], [0]) for i, sid in enumerate(ids)]
        engine.step(entries)                                   # once without the timer
        with ops.KernelTimer() as timer:
            engine.step(entries)
        out["decode"] = timer.summary()
        for sid in ids:
            engine.end_request(sid)
        g = torch.Generator().manual_seed(3)
        prompt = torch.randint(0, vocab, (prefill_tokens,), generator=g).tolist()
        engine.step([Entry("kp", prompt, [prefill_tokens - 1])])
        engine.end_request("kp")
        with ops.KernelTimer() as timer:
            engine.step([Entry("kp", prompt, [prefill_tokens - 1])])
        out["prefill"] = timer.summary()
        engine.end_request("kp")
    finally:
        engine.use_graphs = graphs
    return {phase: {name: {"calls": calls, "us": round(us, 1)} for name, (calls, us) in sorted(table.items(), key=lambda kv: -kv[1][1])}
            for phase, table in out.items()}


def host_gap(engine, entries_of, repeats: int = 3):
    """One eager step as the host sees it: (wall milliseconds from the call to the synchronised end, milliseconds of
    the same step's kernels replayed from a captured graph, kernel calls of the step).  What is between the two is the
    host: Python between the kernel calls, where the GPU waits for the next launch.  `entries_of()` sets the step's
    requests up and returns (entries, clean-up)."""
    import torch
    from inferrs_amd import ops
    graphs, engine.use_graphs = engine.use_graphs, False
    try:
        walls = []
        for _ in range(repeats + 1):
            entries, cleanup = entries_of()
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            engine.step(entries)
            torch.cuda.synchronize()
            walls.append(time.perf_counter() - t0)
            cleanup()
        # the same step's kernels without the host between them: captured once, replayed
        entries, cleanup = entries_of()
        for e in entries:
            if not engine.has_request(e.seq_id):
                engine.add_request(e.seq_id)
        if not engine.cache.ensure_reserved([(e.seq_id, len(e.tokens)) for e in entries]):
            raise RuntimeError("the cache pool is too small for this step")
        ctx = engine.builder.build([(e.seq_id, e.tokens, e.want) for e in entries])
        with ops.KernelTimer() as timer:
            engine.model.forward(ctx, engine.storage)
        n_calls = sum(calls for calls, _us in timer.summary().values())
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):
            engine.model.forward(ctx, engine.storage)
        replays = []
        for _ in range(repeats + 1):
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            graph.replay()
            b.record()
            torch.cuda.synchronize()
            replays.append(a.elapsed_time(b))
        del graph
        cleanup()
    finally:
        engine.use_graphs = graphs
    return min(walls[1:]) * 1e3, min(replays[1:]), n_calls


WORKLOADS = {
    # name: (shape, requests, shortest prompt, longest prompt, portion, decode tokens)
    "mixed16": ("14B", 16, 128, 4096, 512, 128),
    "concurrent32": ("32B", 32, 1024, 1024, 1024, 256),
}


def run_workload(engine, lengths, portion: int, decode_tokens: int, budget: int, vocab: int, seed: int, row_multiple: int = 256):
    """All requests arrive at once and run to their last token.  Returns (seconds, seconds to each
    request's first token, loop steps, seconds until the last prompt was through)."""
    import torch
    from inferrs_amd.engine import GenerationLoop
    from inferrs_amd.sampling import SamplingParams
    loop = GenerationLoop(engine, max_batch_size=len(lengths), max_tokens_per_step=budget, prefill_chunk=portion,
                          row_multiple=row_multiple)
    g = torch.Generator().manual_seed(seed)
    params = SamplingParams.greedy(max_tokens=decode_tokens, bypass_stop_tokens=True)
    requests = [loop.add(torch.randint(0, vocab, (n,), generator=g).tolist(), params) for n in lengths]
    first = {}
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    while loop.scheduler.has_work():
        loop.step()
        now = time.perf_counter() - t0          # (a step's tokens are on the host when it returns)
        for r in requests:
            if r.output and r.request_id not in first:
                first[r.request_id] = now
    torch.cuda.synchronize()
    elapsed = time.perf_counter() - t0
    if any(len(r.output) != decode_tokens for r in requests):
        raise RuntimeError("a request ended early")
    return elapsed, [first[r.request_id] for r in requests], loop.steps, max(first.values())


def workload_main(args, raw, engine_factory) -> int:
    import random
    _, n_req, lo, hi, portion, _ = WORKLOADS[args.workload]
    rnd = random.Random(0)
    lengths = [rnd.randint(lo, hi) for _ in range(n_req)]
    decode_tokens = args.decode_tokens
    budget = max(2048, portion)
    pages = sum(-(-(n + decode_tokens + 1) // PAGE) + 1 for n in lengths) + 8
    note(f"{args.workload}: {n_req} requests, {sum(lengths)} prompt tokens, {decode_tokens} decoded tokens each")
    engine = engine_factory(pages, n_req + 1)
    run_workload(engine, lengths, portion, min(decode_tokens, 16), budget, raw["vocab_size"], seed=1, row_multiple=args.row_multiple)      # warm-up
    runs = [run_workload(engine, lengths, portion, decode_tokens, budget, raw["vocab_size"], seed=2 + i, row_multiple=args.row_multiple)
            for i in range(max(1, args.steps if args.steps < 16 else 3))]
    elapsed, firsts, steps, prompts_done = min(runs, key=lambda r: r[0])
    p_tok, d_tok = sum(lengths), n_req * decode_tokens
    print(json.dumps({
        "metric": f"tokens/s of the serving loop, workload {args.workload} (Qwen3-{args.shape})",
        "value": round((p_tok + d_tok) / elapsed, 1), "unit": "tok/s", "n_gpus": 1, "runs": len(runs),
        "seconds": round(elapsed, 4), "higher_is_better": True, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
        "data": "synthetic: random-init weights, uniform-random token ids, stop tokens ignored",
        "config": {"model": f"Qwen3-{args.shape} shape", "layers": args.layers, "requests": n_req,
                   "prompt_tokens": p_tok, "shortest_prompt": min(lengths), "longest_prompt": max(lengths),
                   "portion": portion, "tokens_per_step": budget, "decode_tokens": decode_tokens, "kv_page_size": PAGE,
                   "row_multiple": args.row_multiple},
        "loop_steps": steps,
        "first_token_s": {"mean": round(sum(firsts) / len(firsts), 4), "max": round(max(firsts), 4)},
        # until the last request has its first token the steps are mostly prompt portions, after it only decode steps
        "prompt_phase": {"seconds": round(prompts_done, 4), "prompt_tok_s": round(p_tok / prompts_done, 1)},
        "decode_phase": {"seconds": round(elapsed - prompts_done, 4),
                         "tok_s": round(n_req * (decode_tokens - 1) / max(elapsed - prompts_done, 1e-9), 1)},
    }))
    return 0


# ---- the Buketar design beside the dense decoder at equal size (`--design buketar`) ---------------------------
# Layer sizes in the range of real models of its kind: latent attention with a cached row of 256 (latent 192 + 64
# rotated), recurrent blocks as wide as the model, 32 small experts of which a token runs 4.  The dense twin has the
# same width and number of layers, as many attention heads of size 128 as fill the width, and a feed-forward as large
# as the experts that a token runs (top x ff), so that a token costs about the same products in both.
def buketar_shape(width: int, layers: int, heads: int, experts: int, top: int, ff: int, vocab: int = 32768):
    att = {"type": "latent_attention",
           "mixer": {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 192, "scale": 192 ** -0.5,
                     "rot": {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}}
    rec = {"type": "rglru", "mixer": {"width": width, "blocks": max(1, width // 256), "conv": 4}}
    mlp = {"kind": "moe", "expert": {"ff": ff, "limit": 7.0}, "router": {"experts": experts, "top": top, "scale": 1.0}}
    pattern = [rec, rec, att]
    return {"architecture": "Buketar", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "streams": 2,
            "logit_softcap": 30.0, "layers": [dict(pattern[i % 3], mlp=mlp) for i in range(layers)]}


BUKETAR_SHAPES = {"1k": dict(width=1024, layers=12, heads=8, experts=32, top=4, ff=768),
                  "2k": dict(width=2048, layers=12, heads=16, experts=32, top=4, ff=1536),
                  "4k": dict(width=4096, layers=6, heads=32, experts=32, top=4, ff=3072)}


def dense_twin(b: dict, vocab: int = 32768) -> dict:
    return dict(QWEN3_8B, vocab_size=vocab, hidden_size=b["width"], intermediate_size=b["top"] * b["ff"],
                num_hidden_layers=b["layers"], num_attention_heads=b["width"] // 128, num_key_value_heads=max(1, b["width"] // 512),
                tie_word_embeddings=False)


# what a kernel of the new design moves or multiplies at least, against the memory or the matrix roof: entry point ->
# the like kernel of the dense decoder that it is compared with
LIKE_KERNEL = {"streams_step": "add_rmsnorm", "latent_prep": "qk_rope_kv", "head_product": "vendor_gemm",
               "experts_gate_up": "vendor_gemm", "experts_down": "vendor_gemm", "rglru_scan": "add_rmsnorm",
               "conv_step": "add_rmsnorm", "route": "rmsnorm", "route_plan": "rmsnorm", "softcap": "rmsnorm"}


# ---- the Lofudra design beside the dense decoder at equal size (`--design lofudra`) ---------------------------
# Layer sizes in the range of real models of its mixers: a state space of 2 x width inner features in heads of 64 with a
# state of 128; windowed attention in heads of 128 (a window of 1,024) beside a retention of as many heads with keys of
# 64 and values of 128; a matrix memory in heads of 128 x 256; a feed-forward of 4 x width.  The dense twin has the same
# width and number of layers, as many attention heads of size 128 as fill the width, and a gated feed-forward of the
# same products a token (2/3 of the size, three matrices for two).
def lofudra_shape(width: int, layers: int, vocab: int = 32768):
    heads = width // 128
    ssm = {"type": "mamba2", "mixer": {"heads": 2 * width // 64, "vdim": 64, "state": 128, "groups": 1, "conv": 4, "norm_groups": 1}}
    par = {"type": "parallel",
           "mixer": {"left": {"heads": heads, "kv_heads": max(1, heads // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                              "mask": {"size": 1024}, "rot": {"base": 500000.0, "dims": 128}},
                     "right": {"heads": heads, "dim": 64, "vdim": 128, "decay": [1.0 - 2.0 ** (-5 - 5 * i / max(heads - 1, 1)) for i in range(heads)]},
                     "left_scale": 1.0, "right_scale": 1.0}}
    mem = {"type": "mlstm", "mixer": {"heads": max(1, width // 256), "dim": 128, "vdim": 256, "gate_cap": 15.0}}
    pattern = [ssm, par, mem]
    return {"architecture": "Lofudra", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
            "layers": [dict(pattern[i % 3], mlp={"kind": "dense", "ff": 4 * width}) for i in range(layers)]}


LOFUDRA_SHAPES = {"1k": dict(width=1024, layers=12), "2k": dict(width=2048, layers=12), "4k": dict(width=4096, layers=6)}


def lofudra_twin(b: dict, vocab: int = 32768) -> dict:
    return dict(QWEN3_8B, vocab_size=vocab, hidden_size=b["width"], intermediate_size=8 * b["width"] // 3 // 128 * 128,
                num_hidden_layers=b["layers"], num_attention_heads=b["width"] // 128, num_key_value_heads=max(1, b["width"] // 512),
                tie_word_embeddings=False)


LOFUDRA_LIKE_KERNEL = {"sandwich_step": "add_rmsnorm", "activation": "gate_mul", "conv_act_step": "add_rmsnorm",
                       "group_norm_gate": "rmsnorm", "exp_gates": "rmsnorm", "step_gates": "rmsnorm",
                       "linear_scan": "attention_mfma", "linear_scan_chunked": "attention_mfma"}


# ---- the Fisanex design beside the dense decoder at equal size (`--design fisanex`) ---------------------------
# Layer sizes in the range of real models of its kind: heads with keys of 128 and values of 64 over a window of 1,024, a
# quarter as many key heads, half of a head turning; every other layer reads the keys and values of the layer before it
# and has routed experts (32 and 4 outputs that hand the input on, 4 a token, a shared expert of twice their size)
# where the layers with keys of their own have a gated feed-forward of 3 x width.  The dense twin has the same width and
# number of layers, as many attention heads of size 128, and a gated feed-forward of 3 x width in every layer.
def fisanex_shape(width: int, layers: int, vocab: int = 32768):
    heads = width // 128
    mixer = {"heads": heads, "kv_heads": max(1, heads // 4), "dim": 128, "vdim": 64, "scale": 128 ** -0.5,
             "mask": {"size": 1024}, "rot": {"base": 500000.0, "dims": 64}}
    ff = 3 * width // 4 // 64 * 64
    moe = {"kind": "moe", "router": {"experts": 32, "identity": 4, "top": 4}, "expert": {"ff": ff, "limit": 7.0},
           "shared": {"ff": 2 * ff, "limit": 7.0}}
    out = []
    for i in range(layers):
        if i % 2 == 0:
            out.append({"type": "attention", "mixer": dict(mixer), "mlp": {"kind": "dense", "ff": 3 * width}})
        else:
            out.append({"type": "attention", "mixer": dict(mixer, kv_from=i - 1), "mlp": moe})
    return {"architecture": "Fisanex", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "postln_alpha": 2.0,
            "embedding": {"scale": 8.0}, "logit_scale": 0.5, "layers": out}


FISANEX_SHAPES = {"1k": dict(width=1024, layers=12), "2k": dict(width=2048, layers=12), "4k": dict(width=4096, layers=6)}


def fisanex_twin(b: dict, vocab: int = 32768) -> dict:
    return dict(QWEN3_8B, vocab_size=vocab, hidden_size=b["width"], intermediate_size=3 * b["width"],
                num_hidden_layers=b["layers"], num_attention_heads=b["width"] // 128, num_key_value_heads=max(1, b["width"] // 512),
                tie_word_embeddings=True)


FISANEX_LIKE_KERNEL = {"postnorm_step": "add_rmsnorm", "qk_rope_kv_strided": "qk_rope_kv", "sigmoid_gate": "gate_mul",
                       "clamped_gate_mul": "gate_mul", "embed_gather_scaled": "embed_gather", "scale": "rmsnorm",
                       "experts_gate_up": "vendor_gemm", "experts_down": "vendor_gemm", "route": "rmsnorm",
                       "route_plan": "rmsnorm", "attention_mfma": "attention_mfma"}


# ---- the Ligizen design beside the Fisanex design at equal size (`--design ligizen`) ---------------------------
# Layer sizes in the range of real models of its kind.  Even layers: latent attention with a cached row of 256 (latent 192 +
# 64 turned, neighbours paired), heads of 64 + 64 with values of 64, queries through a row of width / 2, a window of 1,024,
# learned sinks, and a gated feed-forward of 3 x width.  Odd layers: attention with keys and values of 128 over a quarter as
# many key heads in chunks of 1,024, half of a head turning with stretched frequencies, every second of them reading the
# keys and values of the one before it, and routed experts (32, 4 a token, a shared expert of twice their size behind its
# gate).  A token's own input of 256 in every layer.  The twin is the Fisanex design at the same width and layers (its
# closest relative in this package: gated attention over shared caches, the same experts and shared expert).
def ligizen_shape(width: int, layers: int, vocab: int = 32768):
    heads = width // 128
    lat = {"heads": heads, "dim": 64, "rot_dim": 64, "vdim": 64, "q_rank": width // 2, "kv_rank": 192, "scale": 128 ** -0.5,
           "mask": {"size": 1024}, "rot": {"base": 10000.0, "dims": 64}}
    att = {"heads": heads, "kv_heads": max(1, heads // 4), "dim": 128, "vdim": 128, "scale": 0.09, "mask": {"size": 1024},
           "rot": {"base": 500000.0, "dims": 64, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    ff = 3 * width // 4 // 64 * 64
    moe = {"kind": "moe", "router": {"experts": 32, "top": 4}, "expert": {"ff": ff, "limit": 7.0}, "shared": {"ff": 2 * ff, "limit": 7.0}}
    out = []
    for i in range(layers):
        if i % 2 == 0:
            out.append({"type": "latent_attention", "mixer": dict(lat), "mlp": {"kind": "dense", "ff": 3 * width}})
        else:
            out.append({"type": "attention", "mixer": dict(att, kv_from=i - 2) if i % 4 == 3 else dict(att), "mlp": moe})
    return {"architecture": "Ligizen", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 8.0},
            "logit_softcap": 30.0, "token_side": {"dim": 256}, "layers": out}


def ligizen_twin(b: dict, vocab: int = 32768) -> dict:
    return fisanex_shape(b["width"], b["layers"], vocab)


LIGIZEN_LIKE_KERNEL = {"parallel_step": "postnorm_step", "qk_rope_kv_strided": "qk_rope_kv_strided", "sigmoid_gate": "sigmoid_gate",
                       "latent_prep": "qk_rope_kv_strided", "head_product": "vendor_gemm", "gate_rows": "clamped_gate_mul",
                       "experts_gate_up": "experts_gate_up", "experts_down": "experts_down", "route": "route",
                       "route_plan": "route_plan", "attention_mfma": "attention_mfma", "rmsnorm": "postnorm_step",
                       "softcap": "scale", "embed_gather": "embed_gather_scaled"}


# ---- the Vufizen design beside the Fisanex and the Lofudra design at equal size (`--design vufizen`) -------------
# Layer sizes in the range of real models of its kind.  Even layers: differential attention with maps of 64 (keys of 128 a
# head), values of 128 and a quarter as many key heads, a convolution of four taps; odd layers: the fading matrix state in
# heads of 128 x 128; every layer routed experts (32, 4 a token) with a shared expert of twice their size behind its gate.
# The twins are the package's closest relatives: the Fisanex design (grouped attention with keys of 128, the same experts in
# every other layer) and the Lofudra design (recurrences with a matrix state a head in every layer).
def vufizen_shape(width: int, layers: int, vocab: int = 32768):
    heads, ff = width // 128, 3 * width // 4 // 64 * 64
    att = {"type": "attention", "mixer": {"heads": heads, "kv_heads": max(1, heads // 4), "dim": 64, "vdim": 128, "scale": 0.125,
                                          "conv": 4, "diff": 0.5, "rot": {"base": 500000.0, "dims": 64}}}
    rec = {"type": "hgrn2", "mixer": {"heads": heads, "dim": 128, "vdim": 128}}
    mlp = {"kind": "moe", "router": {"experts": 32, "top": 4}, "expert": {"ff": ff}, "shared": {"ff": 2 * ff}}
    return {"architecture": "Vufizen", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
            "layers": [dict(att if i % 2 == 0 else rec, mlp=mlp) for i in range(layers)]}


def vufizen_twins(b: dict, vocab: int = 32768) -> dict:
    return {"fisanex": fisanex_shape(b["width"], b["layers"], vocab), "lofudra": lofudra_shape(b["width"], b["layers"], vocab)}


VUFIZEN_LIKE_KERNEL = {"branch_step": "postnorm_step", "conv_qkv": "qk_rope_kv_strided", "differ_norm": "sigmoid_gate",
                       "fading_scan": "linear_scan", "group_norm_gate": "group_norm_gate", "experts_gate_up": "experts_gate_up",
                       "experts_down": "experts_down", "route": "route", "route_plan": "route_plan",
                       "attention_mfma": "attention_mfma", "gate_mul": "clamped_gate_mul", "parallel_step": "postnorm_step"}


# ---- the Lumedra design beside the Ligizen and the Lofudra design at equal size (`--design lumedra`) --------------
# Layer sizes in the range of real models of its kind, three layers in turn: lightning attention in heads of 128 x 128 with a
# clamped feed-forward of 3 x width; latent attention with a cached row of 256 (latent 192 + 64 turned), heads of 64 + 64 with
# values of 64, queries through a row of width / 2, every earlier key; attention with keys and values of 128 over a quarter as
# many key heads, a window of 1,024 beside four first tokens, capped scores, mixed values; the last two with routed experts
# (32 in eight groups of which four stay, 4 a token, a shared expert of twice their size).  The twins are the package's
# closest relatives: the Ligizen design (latent and grouped attention side by side, the same experts in every other layer, one
# norm for both sub-layers) and the Lofudra design (recurrences with a matrix state a head in every layer).
def lumedra_shape(width: int, layers: int, vocab: int = 32768):
    heads, ff = width // 128, 3 * width // 4 // 64 * 64
    rec = {"type": "lightning", "mixer": {"heads": heads, "dim": 128, "vdim": 128,
                                          "decay": [1.0 - 2.0 ** (-5 - 5 * i / max(heads - 1, 1)) for i in range(heads)]},
           "mlp": {"kind": "dense", "ff": 3 * width, "limit": 7.0}}
    moe = {"kind": "moe", "router": {"experts": 32, "top": 4, "scale": 2.5, "groups": {"count": 8, "keep": 4}}, "expert": {"ff": ff},
           "shared": {"ff": 2 * ff}}
    lat = {"type": "latent_attention", "mixer": {"heads": heads, "dim": 64, "rot_dim": 64, "vdim": 64, "q_rank": width // 2, "kv_rank": 192,
                                                 "scale": 128 ** -0.5, "rot": {"base": 10000.0, "dims": 64}}, "mlp": moe}
    att = {"type": "attention", "mixer": {"heads": heads, "kv_heads": max(1, heads // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                                          "softcap": 50.0, "mask": {"size": 1024, "keep_first": 4}, "v_mix": True}, "mlp": moe}
    pattern = [rec, lat, att]
    return {"architecture": "Lumedra", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "layers": [pattern[i % 3] for i in range(layers)]}


def lumedra_twins(b: dict, vocab: int = 32768) -> dict:
    return {"ligizen": ligizen_shape(b["width"], b["layers"], vocab), "lofudra": lofudra_shape(b["width"], b["layers"], vocab)}


LUMEDRA_LIKE_KERNEL = {"parallel_step": "parallel_step", "qk_rope_kv_strided": "qk_rope_kv_strided", "latent_prep": "latent_prep",
                       "head_product": "head_product", "norm_slice": "norm_slice", "attention_mfma": "attention_mfma",
                       "linear_scan": "linear_scan", "group_norm_gate": "group_norm_gate", "clamped_gate_mul": "activation",
                       "gate_mul": "clamped_gate_mul", "experts_gate_up": "experts_gate_up", "experts_down": "experts_down",
                       "route": "route", "route_plan": "route_plan"}


def design_main(args) -> int:
    """Prefill and decode throughput of a design at a few layer sizes beside the dense decoder (or the designs that
    are closer to it) at equal size (random weights), and the time of every kernel of one prefill and one decode step of each."""
    import torch
    from inferrs_amd.config import Qwen3Config
    from inferrs_amd.config.buketar import BuketarConfig
    from inferrs_amd.config.fisanex import FisanexConfig
    from inferrs_amd.config.lofudra import LofudraConfig
    from inferrs_amd.engine import Engine
    batch, context, prompt = args.batch, min(args.context, 2048), args.prefill_tokens
    records = {}
    twin_label, twin_cls, twin_vocab = "dense", Qwen3Config, "vocab_size"
    twins_of = None                              # raw -> {label: raw} where a design stands beside several others
    if args.design == "lumedra":
        from inferrs_amd.config.ligizen import LigizenConfig
        from inferrs_amd.config.lumedra import LumedraConfig
        shapes, shape_of, config_cls, like = FISANEX_SHAPES, lumedra_shape, LumedraConfig, LUMEDRA_LIKE_KERNEL
        title, beside = "Lumedra", "Ligizen and Lofudra at equal width and layers"
        twins_of, twin_classes = lumedra_twins, {"ligizen": LigizenConfig, "lofudra": LofudraConfig}
    elif args.design == "vufizen":
        from inferrs_amd.config.vufizen import VufizenConfig
        shapes, shape_of, config_cls, like = FISANEX_SHAPES, vufizen_shape, VufizenConfig, VUFIZEN_LIKE_KERNEL
        title, beside = "Vufizen", "Fisanex and Lofudra at equal width and layers"
        twins_of, twin_classes = vufizen_twins, {"fisanex": FisanexConfig, "lofudra": LofudraConfig}
    elif args.design == "ligizen":
        from inferrs_amd.config.ligizen import LigizenConfig
        shapes, shape_of, twin_of, config_cls, like = FISANEX_SHAPES, ligizen_shape, ligizen_twin, LigizenConfig, LIGIZEN_LIKE_KERNEL
        title, beside = "Ligizen", "Fisanex at equal width and layers"
        twin_label, twin_cls, twin_vocab = "fisanex", FisanexConfig, "vocab"
    elif args.design == "fisanex":
        shapes, shape_of, twin_of, config_cls, like = FISANEX_SHAPES, fisanex_shape, fisanex_twin, FisanexConfig, FISANEX_LIKE_KERNEL
        title, beside = "Fisanex", "Qwen3 dense at equal width and layers, heads of 128 and a feed-forward of 3 x width"
    elif args.design == "lofudra":
        shapes, shape_of, twin_of, config_cls, like = LOFUDRA_SHAPES, lofudra_shape, lofudra_twin, LofudraConfig, LOFUDRA_LIKE_KERNEL
        title, beside = "Lofudra", "Qwen3 dense at equal width, layers and feed-forward products a token"
    else:
        shapes, shape_of, twin_of, config_cls, like = BUKETAR_SHAPES, buketar_shape, dense_twin, BuketarConfig, LIKE_KERNEL
        title, beside = "Buketar", "Qwen3 dense at equal width, layers and feed-forward products a token"
    for name in (args.design_shapes.split(",") if args.design_shapes else sorted(shapes)):
        b = shapes[name]
        raw_new = shape_of(**b)
        if twins_of is not None:
            beside_it = [(label, twin_classes[label].from_dict(raw), raw["vocab"]) for label, raw in twins_of(b).items()]
        else:
            raw_old = twin_of(b)
            beside_it = [(twin_label, twin_cls.from_dict(raw_old), raw_old[twin_vocab])]
        rec = {}
        for label, config, vocab in [(args.design, config_cls.from_dict(raw_new), raw_new["vocab"])] + beside_it:
            pages = batch * (-(-context // PAGE) + 1) + -(-prompt // PAGE) + 8
            note(f"{name} {label}: random weights, {pages} pages")
            engine = Engine.from_random(config, seed=0, dtype=args.dtype, page_size=PAGE, num_pages=pages, max_seqs=batch + 1)
            fill_storage(engine)
            times = time_prefill(engine, prompt, args.runs, vocab)
            p_mean, p_std = mean_std(times)
            elapsed, _ = time_decode(engine, batch, context, args.steps, args.warmup, decode_run=args.decode_run)
            one, _ = time_decode(engine, 1, context, args.steps, args.warmup, decode_run=args.decode_run)
            rec[label] = {"weights_gb": round(engine.model.weight_bytes() / 1e9, 3),
                          "prefill_tok_s": round(prompt / p_mean, 1), "prefill_ms": round(p_mean * 1e3, 3),
                          f"decode_b{batch}_tok_s": round(batch * args.steps / elapsed, 1),
                          f"decode_b{batch}_ms_per_step": round(elapsed / args.steps * 1e3, 3),
                          "decode_b1_tok_s": round(args.steps / one, 1),
                          "kernels": kernel_breakdown(engine, batch, context, prompt, vocab)}
            del engine
            torch.cuda.empty_cache()
        records[name] = rec
    print(json.dumps({"metric": "design_throughput", "design": title, "beside": beside, "dtype": args.dtype, "data": "synthetic", "batch": batch, "context": context,
                      "prefill_tokens": prompt, "steps": args.steps, "warmup": args.warmup, "like_kernel": like,
                      "shapes": records}))
    return 0


def note(msg: str) -> None:
    """Progress goes to stderr; the one JSON line is all that stdout carries."""
    print(f"[bench] {msg}", file=sys.stderr, flush=True)


def main() -> int:
    ap = argparse.ArgumentParser(description=__doc__.split("\n\n")[0])
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=8192)
    ap.add_argument("--shape", default=None, choices=sorted(SHAPES), help="layer sizes of this Qwen3 model (8B)")
    ap.add_argument("--workload", default=None, choices=sorted(WORKLOADS),
                    help="run requests through the serving loop instead of timing decode steps")
    ap.add_argument("--decode-tokens", type=int, default=None, help="tokens every request of a workload decodes")
    ap.add_argument("--layers", type=int, default=None,
                    help="run fewer layers than the model has (recorded in the config)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--no-points", action="store_true", help="skip batch 1 and 64 and the prefill")
    ap.add_argument("--sampled", action="store_true",
                    help="the timed steps draw with the reference's default sampling parameters instead of the arg max (for profiles)")
    ap.add_argument("--prefill-only", action="store_true", help="time the prefill alone (for profiles)")
    ap.add_argument("--prefill-tokens", type=int, default=PREFILL_TOKENS, help="length of the prompt of the prefill")
    ap.add_argument("--runs", type=int, default=5, help="times the decode steps and the prefill are measured (mean and deviation)")
    ap.add_argument("--no-extra-points", dest="extra_points", action="store_false",
                    help="only batch 1 and 64 and the prefill beside the headline (no further batches and contexts, "
                         "no per-kernel times, no 32-bit path)")
    ap.add_argument("--row-multiple", type=int, default=256,
                    help="workloads: cut prompt portions so that a step's tokens are a multiple of this (0: off)")
    ap.add_argument("--decode-run", type=int, default=8,
                    help="decode steps that the serving loop queues on the GPU at once (1: one at a time)")
    ap.add_argument("--design", default=None, choices=["buketar", "lofudra", "fisanex", "ligizen", "vufizen", "lumedra"],
                    help="instead of the headline: prefill and decode throughput of this design at a few layer sizes "
                         "beside the dense decoder (ligizen: beside the Fisanex design; vufizen: beside the Fisanex and the Lofudra design; lumedra: beside the Ligizen and the Lofudra design) "
                         "at equal size, with every kernel's time")
    ap.add_argument("--design-shapes", default=None, help="with --design: the sizes to run, with commas (default: all)")
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported")
        return 2

    if args.design:
        return design_main(args)

    import torch
    from inferrs_amd.config import Qwen3Config
    from inferrs_amd.engine import Engine

    if args.shape is None:
        args.shape = WORKLOADS[args.workload][0] if args.workload else "8B"
    full_layers = SHAPES[args.shape]["num_hidden_layers"]
    if args.layers is None:
        args.layers = full_layers
    raw = dict(SHAPES[args.shape], num_hidden_layers=args.layers)
    config = Qwen3Config.from_dict(raw)
    dtype_key = "bf16" if args.dtype == "bfloat16" else "fp32"
    esize = 2 if args.dtype == "bfloat16" else 4
    if args.workload:
        if args.decode_tokens is None:
            args.decode_tokens = WORKLOADS[args.workload][5]
        note(f"random weights of {args.layers} layers")
        return workload_main(args, raw, lambda pages, seqs: Engine.from_random(
            config, seed=0, dtype=args.dtype, page_size=PAGE, num_pages=pages, max_seqs=seqs))
    points_batches = [] if args.no_points or args.prefill_only else [1, 64]
    # a point whose cache would not fit beside the weights is left out (batch 64 at a context of 32 k and more)
    per_token = 2 * raw["num_key_value_heads"] * raw["head_dim"] * args.layers * esize
    weights = (matmul_params(raw) * args.layers + 2 * raw["vocab_size"] * raw["hidden_size"]) * esize
    room = 0.9 * torch.cuda.get_device_properties(0).total_memory - weights
    for b in list(points_batches):
        if b * (args.context + PAGE) * per_token > room:
            note(f"batch {b} at context {args.context} does not fit this GPU's memory: point left out")
            points_batches.remove(b)
    biggest = max([args.batch] + points_batches)
    num_pages = biggest * (-(-args.context // PAGE) + 1) + 8
    note(f"random weights of {args.layers} layers and a cache of {num_pages} pages")
    engine = Engine.from_random(config, seed=0, dtype=args.dtype, page_size=PAGE, num_pages=num_pages,
                                max_seqs=biggest + 1)
    fill_storage(engine)
    vocab = raw["vocab_size"]

    def prefill_record(tokens: int, runs: int, roof_tflops=None):
        times = time_prefill(engine, tokens, runs, vocab)
        mean, std = mean_std(times)
        flops = prefill_flops(raw, tokens)
        rec = {"value": round(tokens / mean, 1), "tokens": tokens, "ms": round(mean * 1e3, 3),
               "frac": round(flops / mean / PEAK_FLOPS[dtype_key], 4), "runs": len(times),
               "ms_std": round(std * 1e3, 3), "ms_best": round(min(times) * 1e3, 3)}
        if roof_tflops:
            rec["measured_peak_tflops"] = round(roof_tflops, 1)
            rec["frac_of_measured"] = round(flops / mean / (roof_tflops * 1e12), 4)
        return rec

    if args.prefill_only:
        print(json.dumps({"prefill": prefill_record(args.prefill_tokens, max(1, args.steps))}))
        return 0
    note(f"decode at batch {args.batch}, context {args.context}: {args.warmup} + {args.steps} steps, {args.runs} times")
    elapsed, mean_ctx = time_decode(engine, args.batch, args.context, args.steps, args.warmup, args.decode_run, args.sampled)
    ms_per_step = elapsed / args.steps * 1e3
    value = args.batch * args.steps / elapsed
    nbytes = decode_bytes(raw, args.batch, mean_ctx, esize)
    achieved = nbytes / (elapsed / args.steps) / 1e9
    # the same K steps again, for the spread (the reference's bench: warm-up, then runs, mean and standard
    # deviation, inferrs/src/bench.rs:159-173,226-248); the headline stays the first K steps
    repeats = [ms_per_step] + [time_decode(engine, args.batch, args.context, args.steps, args.warmup, args.decode_run, args.sampled)[0]
                               / args.steps * 1e3 for _ in range(max(0, args.runs - 1))]
    rep_mean, rep_std = mean_std(repeats)

    record = {
        "metric": f"decode tok/s at batch {args.batch}, context {args.context} (Qwen3-{args.shape})", "value": round(value, 2), "unit": "tok/s",
        "n_gpus": 1, "steps": args.steps, "warmup": args.warmup, "ms_per_step": round(ms_per_step, 4),
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": dtype_key,
        "data": "synthetic: random-init weights, uniform-random token ids, cache pages of the context "
                "filled with random keys and values",
        "config": {
            "model": f"Qwen3-{args.shape} shape", "global_batch": args.batch, "seq_len": args.context,
            "parallelism": "single GPU", "layers": args.layers, "layers_of_model": full_layers,
            "hidden_size": raw["hidden_size"], "intermediate_size": raw["intermediate_size"],
            "num_attention_heads": raw["num_attention_heads"], "num_key_value_heads": raw["num_key_value_heads"],
            "head_dim": raw["head_dim"], "vocab_size": raw["vocab_size"], "rope_theta": raw["rope_theta"],
            "rms_norm_eps": raw["rms_norm_eps"], "tie_word_embeddings": raw["tie_word_embeddings"],
            "kv_page_size": PAGE, "prefill_tokens": args.prefill_tokens,
        },
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": PEAK_HBM_GBS, "unit": "GB/s",
                     "frac": round(achieved / PEAK_HBM_GBS, 4)},
        "decode_runs": {"runs": len(repeats), "ms_per_step_mean": round(rep_mean, 4), "ms_per_step_std": round(rep_std, 4),
                        "tok_s_mean": round(args.batch / rep_mean * 1e3, 2)},
    }
    if not args.no_points:
        note("measured roofs: a streaming read and a large bfloat16 product")
        read_gbs, gemm_tflops = measured_roofs(engine)
        record["roofline"]["measured_peak"] = round(read_gbs, 1)
        record["roofline"]["frac_of_measured"] = round(achieved / read_gbs, 4)
        points = {}

        def decode_point(name: str, b: int, context: int, sampled: bool = False):
            steps = max(8, args.steps // 2)
            note(f"decode at batch {b}, context {context}: {steps} steps" + (", default sampling parameters" if sampled else ""))
            el, ctx_mean = time_decode(engine, b, context, steps, min(args.warmup, 4), args.decode_run, sampled)
            points[name] = round(b * steps / el, 2)
            fractions[name] = round(decode_bytes(raw, b, ctx_mean, esize) / (el / steps) / 1e9 / PEAK_HBM_GBS, 4)

        fractions = {}
        for b in points_batches:
            decode_point(f"decode_b{b}", b, args.context)
        if args.extra_points:
            for b in (16, 32):
                if b <= biggest:
                    decode_point(f"decode_b{b}", b, args.context)
            long_ctx = 4 * args.context
            if args.batch * (long_ctx // PAGE + 1) + 8 <= num_pages and long_ctx <= raw["max_position_embeddings"]:
                decode_point(f"decode_b{args.batch}_ctx{long_ctx}", args.batch, long_ctx)
        record["points"] = points
        record["points_hbm_frac"] = fractions
        note(f"prefill of {args.prefill_tokens} tokens")
        record["prefill"] = prefill_record(args.prefill_tokens, args.runs, gemm_tflops)
        # the time to a request's first token through the serving loop (scheduler, step, choice, copy to the host)
        from inferrs_amd.engine import GenerationLoop
        from inferrs_amd.sampling import SamplingParams
        g = torch.Generator().manual_seed(4)
        prompt = torch.randint(0, vocab, (args.prefill_tokens,), generator=g).tolist()
        firsts = []
        for _ in range(3):
            loop = GenerationLoop(engine, max_batch_size=1, max_tokens_per_step=args.prefill_tokens)
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            loop.add(prompt, SamplingParams.greedy(max_tokens=1, bypass_stop_tokens=True))
            loop.run()
            firsts.append(time.perf_counter() - t0)
        record["prefill"]["first_token_ms"] = round(min(firsts) * 1e3, 3)
        if args.extra_points:
            # shorter contexts and prompts, where a step is short and the host's share of it largest: the reference's
            # own bench times a prompt of 128 tokens (inferrs/src/bench.rs:35-37)
            for context in (512, 2048):
                if context < args.context:
                    for b in sorted(set([1, args.batch] + ([64] if 64 in points_batches else []))):
                        decode_point(f"decode_b{b}_ctx{context}", b, context)
            # the same steps when every request draws with the reference's default parameters instead of the arg max
            if 2048 < args.context:
                decode_point(f"decode_b{args.batch}_ctx2048_sampled", args.batch, 2048, sampled=True)
            for tokens in (128, 512):
                if tokens < args.prefill_tokens:
                    rec = prefill_record(tokens, 3)
                    points[f"prefill_{tokens}"] = rec["value"]
                    fractions[f"prefill_{tokens}_mfma"] = rec["frac"]
            # eager steps as the host sees them: wall time against the sum of the kernels' own times
            from inferrs_amd.engine import Entry
            note("eager steps: wall time against the kernels' times")
            gp = torch.Generator().manual_seed(5)
            portion = torch.randint(0, vocab, (512,), generator=gp).tolist()
            mixed_context = min(2048, args.context)

            def mixed_step():
                ids = [f"m{i}" for i in range(args.batch)]
                fill_context(engine, ids, mixed_context - 1)
                def cleanup():
                    for sid in ids + ["mp"]:
                        if engine.has_request(sid):
                            engine.end_request(sid)
                return [Entry(sid, [1 + i], [0]) for i, sid in enumerate(ids)] + [Entry("mp", portion, [511])], cleanup

            def short_prompt(tokens):
                def setup():
                    return [Entry("hp", portion[:tokens], [tokens - 1])], lambda: engine.end_request("hp")
                return setup

            host = {}
            for name, setup in ((f"mixed_{args.batch}_decodes_and_512", mixed_step), ("prefill_128", short_prompt(128)),
                                ("prefill_512", short_prompt(512))):
                wall, kernels, calls = host_gap(engine, setup)
                host[name] = {"wall_ms": round(wall, 3), "graph_ms": round(kernels, 3), "kernel_calls": calls,
                              "host_frac": round(max(0.0, 1.0 - kernels / wall), 4)}
            record["eager_steps"] = host
            long_prompt = 4 * args.prefill_tokens
            note(f"prefill of {long_prompt} tokens")
            rec = prefill_record(long_prompt, 3)
            points[f"prefill_{long_prompt}"] = rec["value"]
            fractions[f"prefill_{long_prompt}_mfma"] = rec["frac"]
            note("per-kernel times of one decode step and one prefill")
            record["kernels"] = kernel_breakdown(engine, args.batch, args.context, args.prefill_tokens, vocab)
            # the true 32-bit path at the same layer sizes, four layers of them
            if args.dtype == "bfloat16":
                f32_layers = min(4, args.layers)
                note(f"the 32-bit path: {f32_layers} layers")
                del loop
                raw32 = dict(raw, num_hidden_layers=f32_layers)
                eng32 = Engine.from_random(Qwen3Config.from_dict(raw32), seed=0, dtype="float32", page_size=PAGE,
                                           num_pages=max(args.batch * (-(-args.context // PAGE) + 1),
                                                         -(-args.prefill_tokens // PAGE)) + 8, max_seqs=args.batch + 1)
                fill_storage(eng32)
                el, ctx_mean = time_decode(eng32, args.batch, args.context, 8, 3, args.decode_run)
                points[f"f32_decode_b{args.batch}_layers{f32_layers}"] = round(args.batch * 8 / el, 2)
                fractions[f"f32_decode_b{args.batch}_layers{f32_layers}"] = round(
                    decode_bytes(raw32, args.batch, ctx_mean, 4) / (el / 8) / 1e9 / PEAK_HBM_GBS, 4)
                times = time_prefill(eng32, args.prefill_tokens, 2, vocab)
                points[f"f32_prefill_{args.prefill_tokens}_layers{f32_layers}"] = round(args.prefill_tokens / min(times), 1)
                fractions[f"f32_prefill_{args.prefill_tokens}_layers{f32_layers}_fma"] = round(
                    prefill_flops(raw32, args.prefill_tokens) / min(times) / PEAK_FLOPS["fp32"], 4)
                del eng32
            # the smallest shape of the family, all its layers (the model that the reference's command line names as its
            # example, inferrs/src/run.rs:35): steps so short that the kernels' fixed costs and, in eager steps, the host set the pace; prompts of
            # a repeated length run from captured graphs there
            if args.dtype == "bfloat16" and args.shape != "0.6B":
                small = SHAPES["0.6B"]
                note("the 0.6B shape: decode at batch 1 and 8 at a context of 2,048, prompts of 128 and 512 tokens")
                eng_s = Engine.from_random(Qwen3Config.from_dict(small), seed=0, dtype="bfloat16", page_size=PAGE,
                                           num_pages=8 * (2048 // PAGE + 2) + 8, max_seqs=9)
                fill_storage(eng_s)
                for b in (1, 8):
                    el, ctx_mean = time_decode(eng_s, b, 2048, 16, 4, args.decode_run)
                    points[f"shape0.6B_decode_b{b}_ctx2048"] = round(b * 16 / el, 2)
                    fractions[f"shape0.6B_decode_b{b}_ctx2048"] = round(decode_bytes(small, b, ctx_mean, 2) / (el / 16) / 1e9 / PEAK_HBM_GBS, 4)
                for tokens in (128, 512):
                    times = time_prefill(eng_s, tokens, 3, small["vocab_size"])
                    points[f"shape0.6B_prefill_{tokens}"] = round(tokens / (sum(times) / len(times)), 1)
                    fractions[f"shape0.6B_prefill_{tokens}_mfma"] = round(
                        prefill_flops(small, tokens) / (sum(times) / len(times)) / PEAK_FLOPS["bf16"], 4)
                del eng_s
    print(json.dumps(record))
    return 0


if __name__ == "__main__":
    sys.exit(main())
