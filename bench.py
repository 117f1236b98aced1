#!/usr/bin/env python3
"""Decode and prefill throughput of the engine at the Qwen2.5-7B shape on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--context 4096]

A step is one decode step of the whole batch through the engine loop (schedule, one graph replay
of the model, sampling, accept).  Weights are random (generated on the GPU from a seed), prompts
are token ids uniform over the vocabulary.  One JSON line is printed: decoded tokens per second
at the default batch, the prefill of one 2,048-token prompt, the decode step's share of the HBM
roofline, and under ``points`` decode throughput at batch 1 and 64 at the same context
(``decode_b*``) and the decode phase of the workload the shape is quoted with, 2,048-token
prompts and 256 generated tokens each, at batch 1, 8 and 64 (``gen_b*``), each with its time per
step, its mean context and its share of the HBM roofline.  ``fp32`` holds the cost of the true
32-bit path at the same layer sizes with fewer layers (both numbers are named), ``sizes`` batch 8
decoding and the same prefill at the 14B and 32B shapes (all layers) and, for the default shape,
batch 8 decoding at a context of 32,768 and a prompt portion behind 30,720 cached tokens.  The fractions
are of the published peaks; ``machine`` holds what this GPU reaches on a plain copy and on a
large library product, and the ``frac_of_measured_*`` fields are the same figures relative to
those.  ``--profile`` adds the time of one eagerly run decode step by class of kernel.
"""
from __future__ import annotations

import argparse
import gc
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
if ROOT not in sys.path:
    sys.path.insert(0, ROOT)

# MI355X published peaks
HBM_GBPS = 8000.0
PEAK_FLOPS = {"bfloat16": 2.5e15, "float32": 157.3e12}

# layer sizes of the Qwen2.5 shapes; the default run is the 7B one
SHAPE_7B = dict(vocab_size=152064, hidden_size=3584, intermediate_size=18944, num_hidden_layers=28,
                num_attention_heads=28, num_key_value_heads=4, head_dim=128, rope_theta=1000000.0,
                rms_norm_eps=1e-6, tie_word_embeddings=False, max_position_embeddings=32768)
SHAPE_14B = dict(SHAPE_7B, hidden_size=5120, intermediate_size=13824, num_hidden_layers=48, num_attention_heads=40,
                 num_key_value_heads=8, rms_norm_eps=1e-5)
SHAPE_32B = dict(SHAPE_7B, hidden_size=5120, intermediate_size=27648, num_hidden_layers=64, num_attention_heads=40,
                 num_key_value_heads=8)
SHAPES = {"7b": SHAPE_7B, "14b": SHAPE_14B, "32b": SHAPE_32B}


def make_config(layers: int | None, shape: str = "7b", positions: int = 0):
    from tensorline_amd.config import Qwen2Config
    d = dict(SHAPES[shape], architectures=["Qwen2ForCausalLM"])
    if layers:
        d["num_hidden_layers"] = layers
    if positions:
        d["max_position_embeddings"] = positions
    return Qwen2Config.from_dict(d)


def layer_matrix_params(cfg) -> int:
    H, I = cfg.hidden_size, cfg.intermediate_size
    return (cfg.q_size + 2 * cfg.kv_size) * H + cfg.q_size * H + 3 * H * I


def decode_bytes(cfg, batch: int, context: int, elem: int = 2) -> float:
    """Bytes a decode step has to read: every weight it uses once, and the cache of the live requests."""
    L, H, V = cfg.num_hidden_layers, cfg.hidden_size, cfg.vocab_size
    weights = (L * layer_matrix_params(cfg) + V * H) * elem
    weights += L * (cfg.q_size + 2 * cfg.kv_size) * 4 + (2 * L + 1) * H * 4          # biases and norm weights
    weights += batch * H * elem                                                        # embedding rows
    kv = batch * context * 2 * cfg.kv_size * elem * L
    return float(weights + kv)


def prefill_flops(cfg, tokens: int, rows: int = 1) -> float:
    L, V, H = cfg.num_hidden_layers, cfg.vocab_size, cfg.hidden_size
    linear = 2.0 * tokens * L * layer_matrix_params(cfg)
    attn = 4.0 * cfg.num_attention_heads * cfg.head_dim * (tokens * (tokens + 1) / 2) * L
    head = 2.0 * rows * V * H
    return linear + attn + head


def random_prompts(n: int, length: int, vocab: int, seed: int):
    import numpy as np
    rng = np.random.default_rng(seed)
    return [rng.integers(0, vocab, size=length).tolist() for _ in range(n)]


def sync():
    import torch
    torch.cuda.synchronize()


def bench_decode(llm, batch: int, context: int, steps: int, warmup: int, seed: int) -> dict:
    """Fill ``batch`` sequences, then time ``steps`` decode steps in which every sequence decodes one
    token.  Prompts are prefilled in portions under the engine's token budget; sequences admitted
    early decode while the later ones are still being prefilled (continuous batching), so prompts
    are shortened by the number of prefill steps: no sequence passes ``context`` tokens before the
    last timed step, and none finishes before it."""
    from tensorline_amd import SamplingParams
    cfg = llm.model_config
    eng = llm.engine
    budget = eng.scheduler.max_batched_tokens
    prompt_len = context - (warmup + steps) - 1
    prefill_steps = -(-batch * prompt_len // budget) + 1
    prompt_len -= prefill_steps if batch > 1 else 0
    assert prompt_len >= 1
    reqs = [eng.add_request(p, SamplingParams(max_tokens=10 ** 9, stop_token_ids={-1}))
            for p in random_prompts(batch, prompt_len, cfg.vocab_size, seed)]
    t0 = time.perf_counter()
    while any(r.num_computed < r.prompt_len for r in reqs):          # prefill, in portions
        eng.step()
    sync()
    fill_s = time.perf_counter() - t0
    for _ in range(warmup):
        eng.step()
    eng.drain()                                                      # nothing in flight when the clock starts
    sync()
    assert all(not r.done for r in reqs) and len(eng.scheduler.running) == batch and not eng.scheduler.waiting
    import torch
    c0 = eng.counters()
    lens0 = [len(r.tokens) for r in reqs]
    e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    t0 = time.perf_counter()
    e0.record()
    for _ in range(steps):
        eng.step()
    eng.drain()                                                      # and nothing when it stops: K steps queued, K read
    e1.record()
    sync()
    dt = time.perf_counter() - t0
    c1 = eng.counters()
    lens1 = [len(r.tokens) for r in reqs]
    assert c1["tokens_generated"] - c0["tokens_generated"] == batch * steps, "a timed step did not decode every sequence"
    assert all(b - a == steps for a, b in zip(lens0, lens1)) and max(lens1) <= context + 1
    assert c1["preemptions"] == c0["preemptions"], "a sequence was preempted inside the timed steps"
    mean_ctx = (sum(lens0) + sum(lens1)) / (2.0 * batch)
    out = {"tok_s": batch * steps / dt, "ms_per_step": dt / steps * 1e3, "fill_s": fill_s, "mean_context": mean_ctx,
           "graph_replays": c1["graph_replays"] - c0["graph_replays"], "ms_per_step_events": e0.elapsed_time(e1) / steps}
    for r in reqs:
        eng.abort(r)
    assert llm.cache.all_free()
    return out


def bench_decode_at_context(llm, batch: int, context: int, steps: int, warmup: int, seed: int) -> dict:
    """Decode steps of ``batch`` sequences at a long context without the prefill that would put them
    there (a million tokens for 64 sequences at 16,384): every sequence is given pages for ``context``
    tokens of a cache filled with random values, and the step function (the graphs' runner, as in
    serving) decodes ``warmup + steps`` tokens for each, the engine's greedy pick read after every
    step.  What a step reads and computes is what it would after a real prompt; the scheduler and the
    overlap of its host work with the step before are not part of this measurement."""
    import torch

    from tensorline_amd.engine.batch import StepEntry
    from tensorline_amd.ops import kernels
    cfg, cache, runner = llm.model_config, llm.cache, llm.engine.runner
    g = torch.Generator(device="cuda:0").manual_seed(seed)
    for i in range(len(llm.model.schedule)):
        if cache.owns_storage(i):
            for plane in cache.storage(i).values():
                plane.normal_(0.0, 0.5, generator=g)
    first = context - (warmup + steps)
    rids = [("long", i) for i in range(batch)]
    for rid in rids:
        cache.add_request(rid)
        assert cache.grow(rid, context), "the pool is too small for this point"
    tokens = [p[0] for p in random_prompts(batch, 1, cfg.vocab_size, seed)]
    e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    t0 = 0.0
    for s in range(warmup + steps):
        if s == warmup:
            sync()
            t0 = time.perf_counter()
            e0.record()
        logits = runner.step([StepEntry(rid, [tok], first + s, [0]) for rid, tok in zip(rids, tokens)])
        tokens = kernels.argmax(logits).tolist()
    e1.record()
    sync()
    dt = time.perf_counter() - t0
    for rid in rids:
        cache.release(rid)
    assert cache.all_free()
    return {"tok_s": batch * steps / dt, "ms_per_step": dt / steps * 1e3, "ms_per_step_events": e0.elapsed_time(e1) / steps,
            "mean_context": first + warmup + (steps + 1) / 2.0, "fill_s": 0.0, "graph_replays": 0}


def bench_generate(llm, batch: int, prompt_len: int, new_tokens: int, seed: int) -> dict:
    """The decode phase of the workload the shape is quoted with: ``batch`` requests, each a prompt of
    ``prompt_len`` random tokens and ``new_tokens`` generated ones.  Prompts are prefilled under the
    engine's token budget (requests admitted early decode meanwhile); the timed steps are those
    from the moment every prompt is cached until the first request ends, so each of them decodes
    one token for every one of the ``batch`` requests."""
    import torch

    from tensorline_amd import SamplingParams
    cfg, eng = llm.model_config, llm.engine
    reqs = [eng.add_request(p, SamplingParams(max_tokens=new_tokens, stop_token_ids={-1}))
            for p in random_prompts(batch, prompt_len, cfg.vocab_size, seed)]
    while any(r.num_computed < r.prompt_len for r in reqs):
        eng.step()
    eng.drain()
    sync()                                                  # every request has its first token; all decode from here
    assert all(not r.done for r in reqs) and len(eng.scheduler.running) == batch
    steps = new_tokens - max(r.num_generated for r in reqs)
    lens0 = [len(r.tokens) for r in reqs]
    g0 = eng.tokens_generated
    e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    t0 = time.perf_counter()
    e0.record()
    for _ in range(steps):
        eng.step()
    eng.drain()
    e1.record()
    sync()
    dt = time.perf_counter() - t0
    lens1 = [len(r.tokens) for r in reqs]
    assert eng.tokens_generated - g0 == batch * steps and all(b - a == steps for a, b in zip(lens0, lens1))
    eng.run_until_done()
    assert all(r.done and r.num_generated == new_tokens for r in reqs) and llm.cache.all_free()
    return {"tok_s": batch * steps / dt, "ms_per_step": dt / steps * 1e3, "steps": steps,
            "mean_context": (sum(lens0) + sum(lens1)) / (2.0 * batch), "ms_per_step_events": e0.elapsed_time(e1) / steps}


def profile_decode_step(llm, batch: int, context: int, seed: int) -> dict:
    """One decode step of ``batch`` sequences at about ``context`` tokens run eagerly, timed by class
    of kernel with events around every launch (tensorline_amd/ops/profile.py)."""
    from tensorline_amd import SamplingParams
    from tensorline_amd.engine.runner import ModelRunner
    from tensorline_amd.ops.profile import KernelTimer
    cfg, eng = llm.model_config, llm.engine
    prompt_len = context - 16 - (-(-batch * context // eng.scheduler.max_batched_tokens) if batch > 1 else 0)
    reqs = [eng.add_request(p, SamplingParams(max_tokens=10 ** 9, stop_token_ids={-1}))
            for p in random_prompts(batch, prompt_len, cfg.vocab_size, seed)]
    while any(r.num_computed < r.prompt_len for r in reqs):
        eng.step()
    eng.drain()
    graph_runner, eager, overlap = eng.runner, ModelRunner(llm.model, llm.cache), eng.overlap
    eager.fit_context = graph_runner.fit_context
    eng.runner, eng.overlap = eager, False                   # one step at a time, read before the next
    try:
        for _ in range(3):
            eng.step()
        timer = KernelTimer()
        with timer.measuring():
            eng.step()
    finally:
        eng.runner, eng.overlap = graph_runner, overlap
    for r in reqs:
        eng.abort(r)
    return timer.summary()


def bench_prefill(llm, tokens: int, reps: int, seed: int) -> dict:
    """One prompt of ``tokens`` tokens in one step, logits for its last position."""
    from tensorline_amd.engine.batch import StepEntry
    from tensorline_amd.ops import kernels
    cfg = llm.model_config
    cache, runner = llm.cache, llm.engine.runner
    prompt = random_prompts(1, tokens, cfg.vocab_size, seed)[0]
    times = []
    for i in range(reps + 1):
        rid = ("prefill", i)
        cache.add_request(rid)
        assert cache.grow(rid, tokens)
        sync()
        t0 = time.perf_counter()
        logits = runner.step([StepEntry(rid, prompt, 0, [tokens - 1])])
        kernels.argmax(logits).tolist()                                # the engine's greedy pick, as in a decode step
        sync()
        times.append(time.perf_counter() - t0)
        cache.release(rid)
    best = min(times[1:])                                              # the first run warms up
    return {"s": best, "tok_s": tokens / best}


def prefill_portion_flops(cfg, tokens: int, context: int) -> float:
    """A portion of ``tokens`` tokens behind ``context`` cached ones, logits for its last position."""
    L, V, H = cfg.num_hidden_layers, cfg.vocab_size, cfg.hidden_size
    linear = 2.0 * tokens * L * layer_matrix_params(cfg)
    attn = 4.0 * cfg.num_attention_heads * cfg.head_dim * (tokens * context + tokens * (tokens + 1) / 2) * L
    return linear + attn + 2.0 * V * H


def bench_prefill_portion(llm, context: int, tokens: int, reps: int, seed: int) -> dict:
    """A prompt portion of ``tokens`` tokens in one step behind ``context`` tokens that earlier steps
    cached (in portions of the same size), logits for its last position."""
    from tensorline_amd.engine.batch import StepEntry
    from tensorline_amd.ops import kernels
    cfg, cache, runner = llm.model_config, llm.cache, llm.engine.runner
    prompt = random_prompts(1, context + tokens, cfg.vocab_size, seed)[0]
    rid = ("portion", 0)
    cache.add_request(rid)
    assert cache.grow(rid, context + tokens)
    for start in range(0, context, tokens):
        n = min(tokens, context - start)
        runner.step([StepEntry(rid, prompt[start:start + n], start, [])])
    times = []
    for _ in range(reps + 1):                                          # the same portion again: it overwrites its own keys
        sync()
        t0 = time.perf_counter()
        logits = runner.step([StepEntry(rid, prompt[context:], context, [tokens - 1])])
        kernels.argmax(logits).tolist()
        sync()
        times.append(time.perf_counter() - t0)
    cache.release(rid)
    best = min(times[1:])
    return {"s": best, "tok_s": tokens / best}


def measure_machine(dtype) -> dict:
    """What this GPU reaches on two plain jobs, beside the published peaks: a device-to-device
    copy of 2 GiB (bytes read plus bytes written per second) and a square library product of
    8,192 rows in the benchmark's dtype (float32: the library's true 32-bit kernels)."""
    import torch
    src = torch.empty(1 << 30, dtype=torch.int16, device="cuda:0").fill_(1)
    dst = torch.empty_like(src)
    n = 8192
    a = torch.randn(n, n, dtype=dtype, device="cuda:0")
    b = torch.randn(n, n, dtype=dtype, device="cuda:0")

    def best_ms(fn, reps):
        fn()
        best = float("inf")
        for _ in range(reps):
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            e0.record()
            fn()
            e1.record()
            e1.synchronize()
            best = min(best, e0.elapsed_time(e1))
        return best
    copy_ms = best_ms(lambda: dst.copy_(src), 5)
    mm_ms = best_ms(lambda: torch.mm(a, b.t()), 5)
    return {"copy_GBps": round(2 * src.numel() * 2 / copy_ms / 1e6, 1),
            "gemm_TFLOPs": round(2 * n ** 3 / mm_ms / 1e9, 1)}


def run_workload(llm, requests: int, prompt_min: int, prompt_max: int, output_tokens: int, temperature: float,
                 seed: int) -> dict:
    """``requests`` prompts of uniform random length in [prompt_min, prompt_max] given to the scheduler
    at once (continuous batching, prompts in portions), ``output_tokens`` generated for each, greedy or
    seeded temperature sampling; the clock runs from the call to the last token."""
    import numpy as np
    import torch

    from tensorline_amd import SamplingParams
    cfg = llm.model_config
    rng = np.random.default_rng(seed)
    lengths = rng.integers(prompt_min, prompt_max + 1, size=requests)
    prompts = [rng.integers(0, cfg.vocab_size, size=int(n)).tolist() for n in lengths]
    params = [SamplingParams(max_tokens=output_tokens, temperature=temperature, top_p=1.0,
                             stop_token_ids={-1}, seed=seed + i) for i in range(requests)]
    c0 = llm.counters()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    outs = llm.generate(prompts, params)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    c = llm.counters()
    gen = sum(len(o.token_ids) for o in outs)
    assert all(len(o.token_ids) == output_tokens for o in outs) and llm.cache.all_free()
    ttft = sorted(o.stats.ttft_s for o in outs)
    steps = c["steps"] - c0["steps"]
    # what the run cannot do without: every step reads the weights once, every prompt token and every
    # generated token is multiplied with them once (attention left out: a lower bound on both)
    weight_bytes = decode_bytes(cfg, 0, 0, 2 if llm.model.dtype == torch.bfloat16 else 4)
    flops = 2.0 * (int(lengths.sum()) + gen) * cfg.num_hidden_layers * layer_matrix_params(cfg)
    return {"tok_s": gen / dt, "total_s": dt, "steps": steps, "prompt_tokens": int(lengths.sum()), "generated": gen,
            "ttft_p50_s": ttft[len(ttft) // 2], "ttft_max_s": ttft[-1],
            "preemptions": c["preemptions"] - c0["preemptions"], "graph_replays": c["graph_replays"] - c0["graph_replays"],
            "weight_reads_GBps": steps * weight_bytes / dt / 1e9, "product_flops_per_s": flops / dt}


def bench_workload(args) -> int:
    """A serving-style run: many concurrent requests through the scheduler (continuous batching,
    chunked prefill), as in the 14B and 32B workloads: ``--requests`` prompts of uniform random
    length in [--prompt-min, --prompt-max], ``--output-tokens`` each, greedy or seeded temperature
    sampling.  Prints one JSON line: generated tokens per second over the whole run."""
    from tensorline_amd import LLM
    cfg = make_config(args.layers, args.shape)
    max_len = args.prompt_max + args.output_tokens + 16
    page = 16
    llm = LLM(config=cfg, seed=args.seed, dtype=args.dtype, device="cuda:0", block_size=page,
              num_blocks=args.num_blocks or None, kv_mem_fraction=0.8, max_num_seqs=args.requests,
              max_batched_tokens=2048, max_model_len=max_len, graphs=not args.no_graphs, prefix_caching=False,
              tune_library=not args.no_tune)
    w = run_workload(llm, args.requests, args.prompt_min, args.prompt_max, args.output_tokens, args.temperature, args.seed)
    print(json.dumps({
        "metric": f"generated tok/s, {args.requests} concurrent requests (Qwen2.5-{args.shape.upper()} shape)",
        "value": round(w["tok_s"], 1), "unit": "tok/s", "n_gpus": 1, "steps": w["steps"], "warmup": 0,
        "ms_per_step": round(w["total_s"] / max(w["steps"], 1) * 1e3, 3), "higher_is_better": True, "scaling": "weak",
        "vs_baseline": None, "dtype": "bf16" if args.dtype in ("bfloat16", "bf16") else "fp32",
        "data": "synthetic: random weights from a seed, token ids uniform over the vocabulary",
        "config": {"model": f"Qwen2.5-{args.shape.upper()} shape", "global_batch": args.requests, "seq_len": max_len,
                   "parallelism": "single GPU", "layers": cfg.num_hidden_layers,
                   "layers_of_shape": SHAPES[args.shape]["num_hidden_layers"], "prompt_min": args.prompt_min,
                   "prompt_max": args.prompt_max, "output_tokens": args.output_tokens, "prompt_tokens": w["prompt_tokens"],
                   "temperature": args.temperature, "chunk": 2048, "kv_pages": llm.cache.num_blocks, "page_size": page,
                   "preemptions": w["preemptions"], "graph_replays": w["graph_replays"],
                   "ttft_p50_s": round(w["ttft_p50_s"], 3), "ttft_max_s": round(w["ttft_max_s"], 3),
                   "total_s": round(w["total_s"], 2)}}))
    return 0



# ---- the hybrid design (Samovik) beside the dense decoder at equal size ------------------------------
# Layer sizes that resemble real models of the kind: width, heads of 128, a latent of 192 + 64 rotated
# dimensions (a cached row of 256), state mixers with heads of 128 and 64, experts of which 6 are used
# and a shared one.  ``dense`` is the closest existing model at equal size: the same width, layers and
# vocabulary, grouped-query attention with the same number of heads of 128, and a feed-forward as wide as
# the experts a token uses plus the shared one.
HYBRID_SIZES = {
    "w1024": dict(width=1024, heads=8, experts=32, top=6, ff=512, shared_ff=1024, side=128),
    "w2048": dict(width=2048, heads=16, experts=64, top=6, ff=1408, shared_ff=2816, side=256),
    "w4096": dict(width=4096, heads=32, experts=64, top=6, ff=2048, shared_ff=4096, side=256),
}
HYBRID_VOCAB = 32000


def make_hybrid_config(size: str):
    from tensorline_amd.config import SamovikConfig
    z = HYBRID_SIZES[size]
    H = z["heads"]
    mlp = {"kind": "moe", "router": {"experts": z["experts"], "top": z["top"]}, "expert": {"ff": z["ff"], "limit": 7.0},
           "shared": {"ff": z["shared_ff"], "limit": 7.0}}
    latent = {"heads": H, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 192, "scale": 192 ** -0.5,
              "rot": {"base": 10000.0, "dims": 64, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    lightning = {"heads": H, "dim": 128, "vdim": 128, "decay": [1.0 - 2.0 ** (-5 - 3 * h / H) for h in range(H)]}
    wkv = {"heads": 2 * H, "dim": 64, "decay_rank": 64}
    layers = [{"type": t, "mixer": m, "mlp": mlp} for t, m in
              (("latent_attention", latent), ("lightning", lightning), ("wkv", wkv), ("latent_attention", latent))]
    return SamovikConfig.from_dict({"architecture": "Samovik", "vocab": HYBRID_VOCAB, "width": z["width"], "norm": {"eps": 1e-6},
                                    "token_side": {"dim": z["side"]}, "layers": layers})


def make_dense_twin(size: str):
    from tensorline_amd.config import Qwen2Config
    z = HYBRID_SIZES[size]
    return Qwen2Config.from_dict(dict(
        architectures=["Qwen2ForCausalLM"], vocab_size=HYBRID_VOCAB, hidden_size=z["width"],
        intermediate_size=z["top"] * z["ff"] + z["shared_ff"], num_hidden_layers=4, num_attention_heads=z["heads"],
        num_key_value_heads=max(1, z["heads"] // 4), head_dim=128, rope_theta=10000.0, rms_norm_eps=1e-6,
        tie_word_embeddings=False, max_position_embeddings=32768))


# ---- the Tumitar design beside the dense decoder at equal size ----------------------------------------
# Layer sizes that resemble real models of its kinds: attention heads of 128 in groups of four, a state-space
# side as wide as the model with heads of 64 and a state of 128, a gated recurrent layer as wide as the model
# with blocks of 128, a dense feed-forward of four widths, experts of which 6 are used.  Four layers (parallel
# + dense, parallel + experts, rglru + dense, parallel + experts), each run once.  ``dense`` has the same width,
# layers, vocabulary and attention heads, and a SwiGLU with the mean of the feed-forward weights a token reads.
TUMITAR_SIZES = {
    "w1024": dict(width=1024, heads=8, experts=32, top=6, ff=512),
    "w2048": dict(width=2048, heads=16, experts=64, top=6, ff=1408),
    "w4096": dict(width=4096, heads=32, experts=64, top=6, ff=2048),
}


def make_tumitar_config(size: str):
    from tensorline_amd.config import TumitarConfig
    z = TUMITAR_SIZES[size]
    W, H = z["width"], z["heads"]
    par = {"left": {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                    "q_temp": {"coef": 0.1, "every": 1024}},
           "right": {"heads": W // 64, "vdim": 64, "state": 128, "groups": 2, "conv": 4, "norm_groups": 2},
           "left_scale": 0.7, "right_scale": 0.7}
    moe = {"kind": "moe", "router": {"experts": z["experts"], "top": z["top"], "scale": 1.0}, "expert": {"ff": z["ff"]}}
    dense = {"kind": "dense", "ff": 4 * W}
    layers = [{"type": "parallel", "mixer": par, "mlp": dense}, {"type": "parallel", "mixer": par, "mlp": moe},
              {"type": "rglru", "mixer": {"width": W, "blocks": W // 128, "conv": 4}, "mlp": dense},
              {"type": "parallel", "mixer": par, "mlp": moe}]
    return TumitarConfig.from_dict({"architecture": "Tumitar", "vocab": HYBRID_VOCAB, "width": W, "norm": {"eps": 1e-6},
                                    "embedding": {"scale": 1.0}, "layers": layers})


def make_tumitar_twin(size: str):
    from tensorline_amd.config import Qwen2Config
    z = TUMITAR_SIZES[size]
    inter = (2 * 2 * 4 * z["width"] + 2 * 3 * z["top"] * z["ff"]) // (4 * 3) // 128 * 128
    return Qwen2Config.from_dict(dict(
        architectures=["Qwen2ForCausalLM"], vocab_size=HYBRID_VOCAB, hidden_size=z["width"], intermediate_size=inter,
        num_hidden_layers=4, num_attention_heads=z["heads"], num_key_value_heads=max(1, z["heads"] // 4), head_dim=128,
        rope_theta=10000.0, rms_norm_eps=1e-6, tie_word_embeddings=False, max_position_embeddings=32768))


# ---- the Zeganex design beside the dense decoder at equal size ----------------------------------------
# Layer sizes that resemble real models of its kinds: rotary layers with heads of 128 in groups of four, half of a
# head rotated, an output gate; two-map layers with half as many heads, maps of 64 and values of 128; convolutions of
# four taps; windows of 4,096 tokens (beyond the contexts measured, so that attention does the dense model's work);
# a SwiGLU of three widths, experts without gate of which 6 are used.  Four layers (rotary + dense, two maps +
# experts, rotary + experts, two maps reading the second layer's cache + experts).  ``dense`` has the same width,
# layers, vocabulary and attention heads, and a SwiGLU with the mean of the feed-forward weights a token reads.
ZEGANEX_SIZES = {
    "w1024": dict(width=1024, heads=8, experts=32, top=6, ff=512),
    "w2048": dict(width=2048, heads=16, experts=64, top=6, ff=1408),
    "w4096": dict(width=4096, heads=32, experts=64, top=6, ff=2048),
}


def make_zeganex_config(size: str):
    from tensorline_amd.config import ZeganexConfig
    z = ZEGANEX_SIZES[size]
    W, H = z["width"], z["heads"]
    rotary = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "conv": 4, "mask": {"size": 4096},
              "rot": {"dims": 64, "base": 10000.0, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    maps = {"heads": H // 2, "kv_heads": max(1, H // 8), "dim": 64, "vdim": 128, "scale": 64 ** -0.5, "conv": 4, "diff": 0.5,
            "mask": {"size": 4096}}
    moe = {"kind": "moe", "router": {"experts": z["experts"], "top": z["top"]}, "expert": {"ff": z["ff"]}}
    dense = {"kind": "dense", "ff": 3 * W}
    layers = [{"type": "attention_2", "mixer": rotary, "mlp": dense}, {"type": "attention", "mixer": maps, "mlp": moe},
              {"type": "attention_2", "mixer": rotary, "mlp": moe}, {"type": "attention", "mixer": {**maps, "kv_from": 1}, "mlp": moe}]
    return ZeganexConfig.from_dict({"architecture": "Zeganex", "vocab": HYBRID_VOCAB, "width": W, "norm": {"eps": 1e-6},
                                    "residual_mult": 0.5, "embedding": {"bigram": {"buckets": 65521, "mul_prev": 8191, "mul_cur": 31}},
                                    "layers": layers})


def make_zeganex_twin(size: str):
    from tensorline_amd.config import Qwen2Config
    z = ZEGANEX_SIZES[size]
    inter = (3 * 3 * z["width"] + 3 * 2 * z["top"] * z["ff"]) // (4 * 3) // 128 * 128
    return Qwen2Config.from_dict(dict(
        architectures=["Qwen2ForCausalLM"], vocab_size=HYBRID_VOCAB, hidden_size=z["width"], intermediate_size=inter,
        num_hidden_layers=4, num_attention_heads=z["heads"], num_key_value_heads=max(1, z["heads"] // 4), head_dim=128,
        rope_theta=10000.0, rms_norm_eps=1e-6, tie_word_embeddings=False, max_position_embeddings=32768))


# ---- the Kabulix design beside the dense decoder at equal size ----------------------------------------
# Layer sizes that resemble real models of its kinds: windowed layers with heads of 128 in groups of four whose values
# are their keys, half of a head rotated, four first tokens kept in sight; a latent layer with a latent of 192 + 64
# rotated dimensions (a cached row of 256) and a gate per output column; a chunked layer with heads of 128 and a gate
# per head; windows and chunks of 4,096 tokens (beyond the contexts measured, so that attention does the dense model's
# work); a GELU feed-forward of three widths, experts of which 6 of 64 in 4 of 8 groups are used beside a gated shared
# one.  Four layers (windowed + dense, latent + experts, windowed + experts, chunked + experts).  ``dense`` has the
# same width, layers, vocabulary and attention heads, and a SwiGLU with the mean of the feed-forward weights a token reads.
KABULIX_SIZES = {
    "w1024": dict(width=1024, heads=8, experts=32, top=6, ff=512, shared_ff=512),
    "w2048": dict(width=2048, heads=16, experts=64, top=6, ff=1408, shared_ff=1408),
    "w4096": dict(width=4096, heads=32, experts=64, top=6, ff=2048, shared_ff=2048),
}


def make_kabulix_config(size: str, reach: int = 4096):
    from tensorline_amd.config import KabulixConfig
    z = KABULIX_SIZES[size]
    W, H = z["width"], z["heads"]
    windowed = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                "mask": {"size": reach, "keep_first": 4}, "rot": {"dims": 64, "base": 10000.0}}
    latent = {"heads": H, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 192, "scale": 192 ** -0.5, "mask": {"size": reach},
              "rot": {"base": 10000.0, "dims": 64, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    chunked = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": reach}}
    moe = {"kind": "moe", "router": {"experts": z["experts"], "top": z["top"], "groups": {"count": 8, "keep": 4}},
           "expert": {"ff": z["ff"]}, "shared": {"ff": z["shared_ff"]}}
    dense = {"kind": "dense", "ff": 3 * W}
    layers = [{"type": "attention", "mixer": windowed, "mlp": dense}, {"type": "latent_attention", "mixer": latent, "mlp": moe},
              {"type": "attention", "mixer": windowed, "mlp": moe}, {"type": "attention_2", "mixer": chunked, "mlp": moe}]
    return KabulixConfig.from_dict({"architecture": "Kabulix", "vocab": HYBRID_VOCAB, "width": W, "norm": {"eps": 1e-6}, "layers": layers})


def make_kabulix_twin(size: str):
    from tensorline_amd.config import Qwen2Config
    z = KABULIX_SIZES[size]
    inter = (3 * z["width"] + 3 * (z["top"] * z["ff"] + z["shared_ff"])) // 4 // 128 * 128
    return Qwen2Config.from_dict(dict(
        architectures=["Qwen2ForCausalLM"], vocab_size=HYBRID_VOCAB, hidden_size=z["width"], intermediate_size=inter,
        num_hidden_layers=4, num_attention_heads=z["heads"], num_key_value_heads=max(1, z["heads"] // 4), head_dim=128,
        rope_theta=10000.0, rms_norm_eps=1e-6, tie_word_embeddings=False, max_position_embeddings=32768))


# ---- the Taluvik design beside the dense decoder at equal size ----------------------------------------
# Layer sizes that resemble real models of its kinds: a delta-rule layer with key and value heads of 128, twice as many
# value heads as query/key heads; a selective scan with an inner width of two and 16 states; chunked attention with heads
# of 128 in groups of four, whole heads rotated, capped scores (chunks of ``--reach`` tokens, beyond the contexts measured
# unless asked for, so that attention does the dense model's work); a GELU feed-forward of three widths beside each.  Four
# layers (delta, scan, attention, delta), each with weights of its own.  ``dense`` has the same width, layers, vocabulary
# and attention heads, and a SwiGLU that makes the layers' weights as many as the design's.
TALUVIK_SIZES = {
    "w1024": dict(width=1024, heads=8),
    "w2048": dict(width=2048, heads=16),
    "w4096": dict(width=4096, heads=32),
}


def make_taluvik_config(size: str, reach: int = 4096):
    from tensorline_amd.config import TaluvikConfig
    z = TALUVIK_SIZES[size]
    W, H = z["width"], z["heads"]
    delta = {"heads": H, "kv_heads": H // 2, "dim": 128, "vdim": 128, "conv": 4}
    scan = {"inner": 2 * W, "state": 16, "dt_rank": W // 16, "conv": 4}
    attention = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 30.0,
                 "mask": {"size": reach},
                 "rot": {"dims": 128, "base": 500000.0, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    ff = {"kind": "dense", "ff": 3 * W}
    layers = [{"type": "delta", "mixer": delta, "mlp": ff}, {"type": "mamba1", "mixer": scan, "mlp": ff},
              {"type": "attention", "mixer": attention, "mlp": ff}, {"type": "delta", "mixer": delta, "mlp": ff}]
    return TaluvikConfig.from_dict({"architecture": "Taluvik", "vocab": HYBRID_VOCAB, "width": W, "norm": {"eps": 1e-5},
                                    "embedding": {"scale": 1.0}, "residual_mult": 0.5, "layers": layers})


def make_taluvik_twin(size: str):
    from tensorline_amd.config import Qwen2Config
    z = TALUVIK_SIZES[size]
    W = z["width"]
    # mixers, in squares of the width: delta 4, scan 6 + its small matrices, attention 2.5, delta 4; dense attention 2.5
    extra = (4.0 + 6.0 + 2 * (W // 16 + 32) / W + W / 16 * 2 / W + 2.5 + 4.0) / 4 - 2.5
    inter = int(W * (3 + extra / 3)) // 128 * 128
    return Qwen2Config.from_dict(dict(
        architectures=["Qwen2ForCausalLM"], vocab_size=HYBRID_VOCAB, hidden_size=W, intermediate_size=inter,
        num_hidden_layers=4, num_attention_heads=z["heads"], num_key_value_heads=max(1, z["heads"] // 4), head_dim=128,
        rope_theta=10000.0, rms_norm_eps=1e-6, tie_word_embeddings=False, max_position_embeddings=32768))


# ---- the Vubotar design beside the Kabulix decoder at equal size --------------------------------------
# Layer sizes that resemble real models of its kinds: matrix memories with heads of 128 keys and 256 values; latent attention
# with queries through 3/8 of the width, a latent of 192 + 64 rotated dimensions (a cached row of 256); grouped attention with
# heads of 128 in groups of four, capped, with a bias over 32 buckets of distances up to 128, a window of ``--reach`` tokens
# (beyond the contexts measured unless asked for) and four kept first tokens; experts of which 6 of 64 (32 at the smallest
# size) are used.  Four layers (matrix memory, latent, grouped, matrix memory), each beside experts.  The framework's closest
# other design is Kabulix: ``kabulix`` has the same width, vocabulary, heads, masks, latent and experts, with its own masked
# attention where this design has matrix memories.
VUBOTAR_SIZES = {
    "w1024": dict(width=1024, heads=8, experts=32, top=6, ff=512),
    "w2048": dict(width=2048, heads=16, experts=64, top=6, ff=1408),
    "w4096": dict(width=4096, heads=32, experts=64, top=6, ff=2048),
}


def make_vubotar_config(size: str, reach: int = 4096):
    from tensorline_amd.config import VubotarConfig
    z = VUBOTAR_SIZES[size]
    W, H = z["width"], z["heads"]
    memory = {"heads": H // 2, "dim": 128, "vdim": 256, "gate_cap": 15.0}
    latent = {"heads": H, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": 3 * W // 8, "kv_rank": 192, "scale": 192 ** -0.5,
              "rot": {"base": 10000.0, "dims": 64}}
    grouped = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 30.0, "bias_max": 128,
               "bias_rows": 32, "mask": {"size": reach, "keep_first": 4}, "v_mix": True}
    moe = {"kind": "moe", "router": {"experts": z["experts"], "top": z["top"]}, "expert": {"ff": z["ff"]}}
    layers = [{"type": kind, "mixer": mixer, "mlp": moe} for kind, mixer in
              (("mlstm", memory), ("latent_attention", latent), ("attention", grouped), ("mlstm", memory))]
    return VubotarConfig.from_dict({"architecture": "Vubotar", "vocab": HYBRID_VOCAB, "width": W, "norm": {"eps": 1e-6},
                                    "embedding": {"scale": 1.0}, "logit_scale": 0.5, "logit_softcap": 30.0, "layers": layers})


def make_vubotar_twin(size: str, reach: int = 4096):
    from tensorline_amd.config import KabulixConfig
    z = VUBOTAR_SIZES[size]
    W, H = z["width"], z["heads"]
    windowed = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                "mask": {"size": reach, "keep_first": 4}, "rot": {"dims": 64, "base": 10000.0}}
    latent = {"heads": H, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 192, "scale": 192 ** -0.5, "rot": {"base": 10000.0, "dims": 64}}
    chunked = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": reach}}
    moe = {"kind": "moe", "router": {"experts": z["experts"], "top": z["top"]}, "expert": {"ff": z["ff"]}}
    layers = [{"type": kind, "mixer": mixer, "mlp": moe} for kind, mixer in
              (("attention", windowed), ("latent_attention", latent), ("attention", windowed), ("attention_2", chunked))]
    return KabulixConfig.from_dict({"architecture": "Kabulix", "vocab": HYBRID_VOCAB, "width": W, "norm": {"eps": 1e-6}, "layers": layers})


def profile_step(llm, entries_of, seed: int) -> dict:
    """Event time of every kernel of one eager step, summed per entry point (milliseconds), after a
    warm-up step of the same shape."""
    from tensorline_amd.engine.runner import ModelRunner
    from tensorline_amd.ops.profile import KernelTimer
    cache = llm.cache
    runner = ModelRunner(llm.model, cache)
    runner.fit_context = llm.engine.runner.fit_context
    out = {}
    for rep in range(2):
        entries = entries_of(cache, rep)
        timer = KernelTimer()
        if rep:
            with timer.measuring():
                runner.step(entries)
        else:
            runner.step(entries)
        sync()
        for e in entries:
            cache.release(e.rid)
        if rep:
            by_name: dict = {}
            for _, name, e0, e1 in timer._spans:
                by_name[name] = by_name.get(name, 0.0) + e0.elapsed_time(e1)
            out = {n: round(v, 4) for n, v in sorted(by_name.items(), key=lambda kv: -kv[1])}
    return out


def bench_hybrid(args, design: str = "samovik") -> int:
    """Prefill and decode throughput of a design at real layer sizes (``samovik``: HYBRID_SIZES, ``tumitar``:
    TUMITAR_SIZES, ``zeganex``: ZEGANEX_SIZES, ``kabulix``: KABULIX_SIZES, ``taluvik``: TALUVIK_SIZES)
    beside the dense decoder at equal size (``vubotar``: VUBOTAR_SIZES, beside Kabulix), and each step's time by kernel.  One JSON line; the default benchmark is not run."""
    import torch
    table, make, make_twin, model_text = {
        "samovik": (HYBRID_SIZES, make_hybrid_config, make_dense_twin,
                    "Samovik layer sizes (4 layers: latent attention, lightning, wkv, latent attention) beside "
                    "Qwen2 layers of equal width (4 layers)"),
        "tumitar": (TUMITAR_SIZES, make_tumitar_config, make_tumitar_twin,
                    "Tumitar layer sizes (4 layers: parallel + dense, parallel + experts, rglru + dense, parallel + experts) "
                    "beside Qwen2 layers of equal width (4 layers)"),
        "zeganex": (ZEGANEX_SIZES, make_zeganex_config, make_zeganex_twin,
                    "Zeganex layer sizes (4 layers: rotary attention + dense, two-map attention + experts, rotary attention + "
                    "experts, two-map attention on the second layer's cache + experts) beside Qwen2 layers of equal width (4 layers)"),
        "kabulix": (KABULIX_SIZES, (lambda size: make_kabulix_config(size, args.reach)), make_kabulix_twin,
                    "Kabulix layer sizes (4 layers: windowed attention with kept first tokens + dense, latent attention + experts, "
                    "windowed attention + experts, chunked attention + experts; windows and chunks of %d tokens) beside Qwen2 "
                    "layers of equal width (4 layers)" % args.reach),
        "taluvik": (TALUVIK_SIZES, (lambda size: make_taluvik_config(size, args.reach)), make_taluvik_twin,
                    "Taluvik layer sizes (4 layers: delta rule, selective scan, chunked attention with capped scores and sinks, delta "
                    "rule, a dense feed-forward beside each; chunks of %d tokens) beside Qwen2 layers of equal width and weights "
                    "(4 layers)" % args.reach),
        "vubotar": (VUBOTAR_SIZES, (lambda size: make_vubotar_config(size, args.reach)), (lambda size: make_vubotar_twin(size, args.reach)),
                    "Vubotar layer sizes (4 layers: matrix memory, latent attention, capped attention with a bias by distance behind a "
                    "window of %d tokens, matrix memory, experts beside each) beside Kabulix layers of equal width and experts "
                    "(4 layers)" % args.reach)}[design]
    other = "kabulix" if design == "vubotar" else "dense"

    from tensorline_amd import LLM
    from tensorline_amd.engine.batch import StepEntry
    page, tokens, batch, context = 16, args.prefill_tokens, args.batch, min(args.context, 2048)
    sizes = [s for s in (args.hybrid_sizes.split(",") if args.hybrid_sizes else sorted(table))]
    results = {}
    for size in sizes:
        row = {}
        for which, cfg in (("hybrid", make(size)), (other, make_twin(size))):
            max_len = max(context, tokens) + 16
            llm = LLM(config=cfg, seed=args.seed, dtype=args.dtype, device="cuda:0", block_size=page,
                      num_blocks=(batch + 1) * (-(-max_len // page)) + 8, max_num_seqs=batch, max_batched_tokens=max(2048, tokens),
                      max_model_len=max_len, graphs=not args.no_graphs, graph_warmup_tokens=0, prefix_caching=False,
                      tune_library=False, overlap=not args.no_overlap)
            pre = bench_prefill(llm, tokens, 3, args.seed + 2)
            dec = bench_decode(llm, batch, context, args.steps, args.warmup, args.seed + 1)
            entry = {"prefill_tok_s": round(pre["tok_s"], 1), "prefill_ms": round(pre["s"] * 1e3, 3),
                     "decode_tok_s": round(dec["tok_s"], 1), "decode_ms_per_step": round(dec["ms_per_step"], 4),
                     "weight_GB": round(llm.model.weight_bytes() / 1e9, 3)}
            if args.profile:
                prompt = random_prompts(1, tokens, cfg.vocab_size, args.seed + 3)[0]

                def prefill_entries(cache, rep):
                    rid = ("pp", rep)
                    cache.add_request(rid)
                    assert cache.grow(rid, tokens)
                    return [StepEntry(rid, prompt, 0, [tokens - 1])]

                def decode_entries(cache, rep):
                    out = []
                    for b in range(batch):
                        rid = ("pd", rep, b)
                        cache.add_request(rid)
                        assert cache.grow(rid, context)
                        out.append(StepEntry(rid, [prompt[b]], context - 1, [0]))
                    return out
                entry["prefill_kernels_ms"] = profile_step(llm, prefill_entries, args.seed)
                entry["decode_kernels_ms"] = profile_step(llm, decode_entries, args.seed)
            row[which] = entry
            del llm
            gc.collect()
            torch.cuda.empty_cache()
        row["hybrid_over_" + other] = {"prefill": round(row["hybrid"]["prefill_tok_s"] / row[other]["prefill_tok_s"], 3),
                                       "decode": round(row["hybrid"]["decode_tok_s"] / row[other]["decode_tok_s"], 3)}
        results[size] = row
    print(json.dumps({"metric": "hybrid_design_tok_s" if design == "samovik" else design + "_design_tok_s", "unit": "tok/s",
                      "n_gpus": 1, "dtype": args.dtype, "data": "synthetic",
                      "config": {"model": model_text, "prefill_tokens": tokens, "decode_batch": batch,
                                 "decode_context": context, "sizes": {k: table[k] for k in sizes}},
                      "results": results}))
    return 0


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=4096)
    ap.add_argument("--layers", type=int, default=0, help="fewer layers than the shape has (0: all)")
    ap.add_argument("--dtype", default="bfloat16")
    ap.add_argument("--prefill-tokens", type=int, default=2048)
    ap.add_argument("--prefill-behind", type=int, default=0,
                    help="measure the prefill as a portion behind this many cached tokens (0: a fresh prompt)")
    ap.add_argument("--no-points", action="store_true", help="skip the batch 1 and 64 decode points")
    ap.add_argument("--no-graphs", action="store_true")
    ap.add_argument("--no-overlap", action="store_true", help="read every decode step's tokens before queueing the next")
    ap.add_argument("--no-fp32", action="store_true", help="skip the 32-bit point")
    ap.add_argument("--no-sizes", action="store_true", help="skip the 14B and 32B shapes and the 32k contexts")
    ap.add_argument("--fp32-layers", type=int, default=4, help="layers of the model the 32-bit point runs")
    ap.add_argument("--profile", action="store_true", help="add the time of one eager decode step by class of kernel")
    ap.add_argument("--no-tune", action="store_true", help="keep the library's heuristic choice of kernels for prompt portions")
    ap.add_argument("--seed", type=int, default=0)
    ap.add_argument("--shape", default="7b", choices=sorted(SHAPES), help="layer sizes (default: the 7B shape)")
    ap.add_argument("--workload", action="store_true", help="serving-style run instead of the step benchmark")
    ap.add_argument("--requests", type=int, default=32)
    ap.add_argument("--prompt-min", type=int, default=256)
    ap.add_argument("--prompt-max", type=int, default=4096)
    ap.add_argument("--output-tokens", type=int, default=512)
    ap.add_argument("--temperature", type=float, default=0.7)
    ap.add_argument("--num-blocks", type=int, default=0, help="KV pages for --workload (0: 80%% of free memory)")
    ap.add_argument("--hybrid", action="store_true",
                    help="instead of the default benchmark: the hybrid design (Samovik) at real layer sizes beside the dense "
                         "decoder at equal size, prefill and decode; with --profile each step's time by kernel")
    ap.add_argument("--tumitar", action="store_true",
                    help="the same for the Tumitar design (attention beside a state-space mixer, gated recurrent layers, dense "
                         "and routed feed-forwards)")
    ap.add_argument("--zeganex", action="store_true",
                    help="the same for the Zeganex design (attention with short convolutions in two kinds, norms on both sides "
                         "of every branch, experts without gate)")
    ap.add_argument("--kabulix", action="store_true",
                    help="the same for the Kabulix design (windowed attention with kept first tokens, latent attention, chunked "
                         "attention, experts chosen within groups beside a gated shared expert)")
    ap.add_argument("--taluvik", action="store_true",
                    help="the same for the Taluvik design (gated delta rule, selective scan, chunked attention with capped scores "
                         "and sinks, both branches of a layer side by side)")
    ap.add_argument("--vubotar", action="store_true",
                    help="the same for the Vubotar design (matrix memories, latent attention with a queries' latent, capped attention "
                         "with a bias by distance, experts beside every mixer), beside the Kabulix decoder")
    ap.add_argument("--reach", type=int, default=4096, help="with --kabulix, --taluvik and --vubotar: tokens of the windows and chunks")
    ap.add_argument("--hybrid-sizes", default="", help="which of w1024,w2048,w4096 (default: all)")
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported")
        return 2
    if args.workload:
        return bench_workload(args)
    if args.hybrid:
        return bench_hybrid(args)
    if args.tumitar:
        return bench_hybrid(args, "tumitar")
    if args.zeganex:
        return bench_hybrid(args, "zeganex")
    if args.kabulix:
        return bench_hybrid(args, "kabulix")
    if args.taluvik:
        return bench_hybrid(args, "taluvik")
    if args.vubotar:
        return bench_hybrid(args, "vubotar")

    import torch

    from tensorline_amd import LLM
    cfg = make_config(args.layers, args.shape)
    full_layers = SHAPES[args.shape]["num_hidden_layers"]
    max_batch = max(args.batch, 1 if args.no_points else 64)
    max_len = max(args.context, args.prefill_behind + args.prefill_tokens) + 16
    page = 16
    llm = LLM(config=cfg, seed=args.seed, dtype=args.dtype, device="cuda:0", block_size=page,
              num_blocks=max_batch * (-(-max_len // page)) + 8, max_num_seqs=max_batch, max_batched_tokens=2048,
              max_model_len=max_len, graphs=not args.no_graphs, graph_warmup_tokens=0, prefix_caching=False,
              tune_library=not args.no_tune, overlap=not args.no_overlap)
    elem = 2 if args.dtype in ("bfloat16", "bf16") else 4
    dtype_key = "bfloat16" if elem == 2 else "float32"

    def with_roofline(run: dict, batch: int, model_cfg=cfg, elem_size=elem) -> dict:
        """tok/s, ms per step (wall clock and events), mean context and the share of the HBM peak of a decode run."""
        gbps = decode_bytes(model_cfg, batch, int(run["mean_context"]), elem_size) / (run["ms_per_step"] / 1e3) / 1e9
        return {"tok_s": round(run["tok_s"], 1), "ms": round(run["ms_per_step"], 4), "ms_events": round(run["ms_per_step_events"], 4),
                "ctx": round(run["mean_context"], 1), "GBps": round(gbps, 1), "hbm_frac": round(gbps / HBM_GBPS, 4)}

    main_run = bench_decode(llm, args.batch, args.context, args.steps, args.warmup, args.seed + 1)
    if args.prefill_behind > 0:
        pre = bench_prefill_portion(llm, args.prefill_behind, args.prefill_tokens, 3, args.seed + 2)
    else:
        pre = bench_prefill(llm, args.prefill_tokens, 3, args.seed + 2)
    points = {}
    if not args.no_points:
        for b in (1, 64):
            k = max(8, args.steps // 2)
            r = with_roofline(bench_decode(llm, b, args.context, k, 4, args.seed + 3 + b), b)
            points[f"decode_b{b}"] = r["tok_s"]
            points.update({f"decode_b{b}_{key}": r[key] for key in ("ms", "ctx", "hbm_frac")})
        # the workload the shape is quoted with: 2,048-token prompts, 256 generated tokens each
        for b in (1, 8, 64):
            r = with_roofline(bench_generate(llm, b, 2048, 256, args.seed + 100 + b), b)
            points[f"gen_b{b}"] = r["tok_s"]
            points.update({f"gen_b{b}_{key}": r[key] for key in ("ms", "ms_events", "ctx", "hbm_frac")})
    profile = profile_decode_step(llm, args.batch, args.context, args.seed + 7) if args.profile else None

    machine = measure_machine(torch.bfloat16 if elem == 2 else torch.float32)
    fp32 = None
    if elem == 2 and not args.no_points and not args.no_fp32:
        # the true 32-bit path at the same layer sizes, fewer layers: what the equality checks cost
        llm = None
        gc.collect()
        torch.cuda.empty_cache()
        cfg32 = make_config(args.fp32_layers, args.shape)
        llm32 = LLM(config=cfg32, seed=args.seed, dtype="float32", device="cuda:0", block_size=page,
                    num_blocks=8 * (-(-max_len // page)) + 8, max_num_seqs=8, max_batched_tokens=2048,
                    max_model_len=max_len, graphs=not args.no_graphs, graph_warmup_tokens=0, prefix_caching=False)
        pre32 = bench_prefill(llm32, args.prefill_tokens, 2, args.seed + 2)
        dec32 = with_roofline(bench_decode(llm32, 8, 2304, 8, 2, args.seed + 9), 8, cfg32, 4)
        fp32 = {"layers": cfg32.num_hidden_layers, "layers_of_shape": full_layers,
                "prefill_tok_s": round(pre32["tok_s"], 1), "prefill_ms": round(pre32["s"] * 1e3, 3),
                "prefill_frac": round(prefill_flops(cfg32, args.prefill_tokens) / pre32["s"] / PEAK_FLOPS["float32"], 4),
                "decode_b8_tok_s": dec32["tok_s"], "decode_b8_ms": dec32["ms"], "decode_b8_ctx": dec32["ctx"],
                "decode_b8_hbm_frac": dec32["hbm_frac"]}
        del llm32
    sizes = None
    if elem == 2 and not args.no_points and not args.no_sizes and args.shape == "7b" and not args.layers:
        # further sizes and contexts, all layers of each shape: batch 8 decoding at the same context and the
        # same prefill for the 14B and 32B shapes; for the default shape batch 8 decoding at a context of
        # 32,768 and a prompt portion behind 30,720 cached tokens
        llm = None
        gc.collect()
        torch.cuda.empty_cache()
        sizes = {}

        def other(shape: str, context: int, batch: int, steps: int, seqs: int = 0, length: int = 0, positions: int = 0,
                  pages: int = 0):
            """A model of all the layers of ``shape`` with room for ``seqs`` sequences of ``length`` tokens (or
            ``pages`` pages), and its decode point at ``batch`` sequences of ``context`` tokens (none for batch 0)."""
            c = make_config(0, shape, positions)
            seqs, length = max(seqs, batch), max(length, context + 16)
            m = LLM(config=c, seed=args.seed, dtype=args.dtype, device="cuda:0", block_size=page,
                    num_blocks=pages or seqs * (-(-length // page)) + 8, max_num_seqs=seqs, max_batched_tokens=2048,
                    max_model_len=length, graphs=not args.no_graphs, graph_warmup_tokens=0, prefix_caching=False,
                    tune_library=not args.no_tune, overlap=not args.no_overlap)
            if batch == 0:
                return c, m, {"layers": c.num_hidden_layers}
            dec = with_roofline(bench_decode(m, batch, context, steps, 4, args.seed + 11), batch, c)
            return c, m, {"layers": c.num_hidden_layers, f"decode_b{batch}_tok_s": dec["tok_s"], f"decode_b{batch}_ms": dec["ms"],
                          f"decode_b{batch}_ctx": dec["ctx"], f"decode_b{batch}_hbm_frac": dec["hbm_frac"]}

        def portion(m, c, behind: int, tag: str) -> dict:
            p = bench_prefill_portion(m, behind, args.prefill_tokens, 2, args.seed + 2)
            return {f"{tag}_behind": behind, f"{tag}_tokens": args.prefill_tokens, f"{tag}_tok_s": round(p["tok_s"], 1),
                    f"{tag}_ms": round(p["s"] * 1e3, 3),
                    f"{tag}_frac": round(prefill_portion_flops(c, args.prefill_tokens, behind) / p["s"] / PEAK_FLOPS[dtype_key], 4)}

        # the workloads the two wider shapes are quoted with: 32 requests with prompts of 256 to 4,096 tokens and
        # 512 tokens each sampled at temperature 0.7; 64 requests of 1,024 + 256 tokens, greedy
        workloads = {"14b": dict(requests=32, prompt_min=256, prompt_max=4096, output_tokens=512, temperature=0.7),
                     "32b": dict(requests=64, prompt_min=1024, prompt_max=1024, output_tokens=256, temperature=0.0)}
        for shape, wl in workloads.items():
            c, m, out = other(shape, args.context, 8, 16, seqs=wl["requests"], length=wl["prompt_max"] + wl["output_tokens"] + 16)
            p2 = bench_prefill(m, args.prefill_tokens, 2, args.seed + 2)
            out.update({"prefill_tok_s": round(p2["tok_s"], 1), "prefill_ms": round(p2["s"] * 1e3, 3),
                        "prefill_frac": round(prefill_flops(c, args.prefill_tokens) / p2["s"] / PEAK_FLOPS[dtype_key], 4)})
            w = run_workload(m, seed=args.seed, **wl)
            out.update({"workload_tok_s": round(w["tok_s"], 1), "workload_requests": wl["requests"],
                        "workload_prompt_tokens": w["prompt_tokens"], "workload_generated": w["generated"],
                        "workload_temperature": wl["temperature"], "workload_s": round(w["total_s"], 2),
                        "workload_steps": w["steps"], "workload_ttft_p50_s": round(w["ttft_p50_s"], 3),
                        "workload_preemptions": w["preemptions"],
                        # lower bounds: the weights once per step, the products of every token; attention left out
                        "workload_hbm_frac_weights": round(w["weight_reads_GBps"] / HBM_GBPS, 4),
                        "workload_mfma_frac_products": round(w["product_flops_per_s"] / PEAK_FLOPS[dtype_key], 4)})
            sizes[shape] = out
            del m
            gc.collect()
            torch.cuda.empty_cache()
        c, m, out = other("7b", 32768, 8, 16)
        out.update(portion(m, c, 32768 - args.prefill_tokens, "portion"))
        out.update(portion(m, c, 8192, "portion_8k"))
        out.update(portion(m, c, 16384, "portion_16k"))
        sizes["7b_32k"] = out
        del m
        gc.collect()
        torch.cuda.empty_cache()
        # batch 64 at 16,384 tokens and batch 8 at 65,536 (positions beyond the shape's 32,768 allowed for this
        # point): the cache is filled with random values instead of by a million tokens of prefill
        points_long = ((64, 16384), (8, 65536))
        c, m, out = other("7b", 0, 0, 0, seqs=64, length=65536 + 16, positions=131072,
                          pages=max(b * (-(-(n + 16) // page)) for b, n in points_long) + 8)
        out.update({"max_position_embeddings": 131072, "cache": "random values, no prefill"})
        for batch, context in points_long:
            d = with_roofline(bench_decode_at_context(m, batch, context, 12, 4, args.seed + 13), batch, c)
            out.update({f"decode_b{batch}_ctx{context}_{key}": d[key] for key in ("tok_s", "ms", "ms_events", "hbm_frac")})
        sizes["7b_long"] = out
        del m
        gc.collect()
        torch.cuda.empty_cache()
    step_s = main_run["ms_per_step"] / 1e3
    achieved = decode_bytes(cfg, args.batch, int(main_run["mean_context"]), elem) / step_s / 1e9
    flops = (prefill_portion_flops(cfg, args.prefill_tokens, args.prefill_behind) if args.prefill_behind > 0
             else prefill_flops(cfg, args.prefill_tokens))
    line = {
        "metric": f"decode tok/s @ batch {args.batch}, context {args.context} (Qwen2.5-{args.shape.upper()} shape)",
        "value": round(main_run["tok_s"], 1),
        "unit": "tok/s",
        "n_gpus": 1,
        "steps": args.steps,
        "warmup": args.warmup,
        "ms_per_step": round(main_run["ms_per_step"], 4),
        "ms_per_step_gpu_events": round(main_run["ms_per_step_events"], 4),
        "higher_is_better": True,
        "scaling": "weak",
        "vs_baseline": None,
        "dtype": "bf16" if elem == 2 else "fp32",
        "data": "synthetic: random weights from a seed, token ids uniform over the vocabulary",
        "config": {
            "model": f"Qwen2.5-{args.shape.upper()} shape", "global_batch": args.batch, "seq_len": args.context,
            "parallelism": "single GPU", "layers": cfg.num_hidden_layers, "layers_of_shape": full_layers,
            "hidden_size": cfg.hidden_size, "intermediate_size": cfg.intermediate_size,
            "num_attention_heads": cfg.num_attention_heads, "num_key_value_heads": cfg.num_key_value_heads,
            "head_dim": cfg.head_dim, "vocab_size": cfg.vocab_size, "page_size": page,
            "prefill_tokens": args.prefill_tokens, "graphs": not args.no_graphs, "library_tuning": not args.no_tune, "sampling": "greedy",
            "overlap": not args.no_overlap,
            "decode_graph_replays": main_run["graph_replays"], "mean_context": round(main_run["mean_context"], 1),
        },
        "prefill": {"value": round(pre["tok_s"], 1), "tokens": args.prefill_tokens, "behind": args.prefill_behind,
                    "ms": round(pre["s"] * 1e3, 3),
                    "frac": round(flops / pre["s"] / PEAK_FLOPS[dtype_key], 4),
                    "frac_of_measured_gemm": round(flops / pre["s"] / (machine["gemm_TFLOPs"] * 1e12), 4)},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_GBPS, "unit": "GB/s",
                     "frac": round(achieved / HBM_GBPS, 4),
                     "frac_of_measured_copy": round(achieved / machine["copy_GBps"], 4)},
        "points": points,
        "machine": machine,
    }
    if fp32 is not None:
        line["fp32"] = fp32
    if sizes is not None:
        line["sizes"] = sizes
    if profile is not None:
        line["profile"] = profile
    print(json.dumps(line))
    torch.cuda.synchronize()
    return 0


if __name__ == "__main__":
    sys.exit(main())
