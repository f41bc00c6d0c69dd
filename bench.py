"""Decode and prefill throughput of the engine on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--prompt-len 512]
                    [--dtype bfloat16] [--layers L] [--no-points] [--phase all|decode|prefill]
                    [--preset llama-1b|llama-3b|llama-8b] [--context-len 8192]
    python bench.py --phase mixed --preset llama-3b --batch 32 --steps 256
    python bench.py --phase burst --preset small [--dtype float32]
    python bench.py --phase fogorax [--dtype float32] [--steps 64] [--batch 8]
    python bench.py --phase rudorax [--sizes w1024,w2048] [--steps 64] [--batch 8]
    python bench.py --phase ludelix [--sizes w1024,w2048] [--steps 64] [--batch 8]

Default run: the layer sizes of Llama 3.2 1B (16 layers, hidden 2048, 32 heads, 8 kv heads, head
size 64, SwiGLU 8192, vocabulary 128256, llama3 rope scaling, tied embeddings), random weights
N(0, 0.02), batch 8, 512-token uniform-random prompts, greedy, context cap 8192, pages of 16
tokens.  A step is one decode step of the whole engine (scheduler, batch building, forward,
sampling, bookkeeping).  One JSON line is printed; besides the decode figure it carries a
2,048-token prefill, the decode step's share of the HBM roofline, and decode at batch 1 and 64.
``points`` also holds (unless ``--no-points``) the same model over contexts of 4,096 and 8,192
tokens (decode at batch 8 and 64, one prompt of 8,192 tokens), the same model in true 32-bit (decode at batch 1
and 8, prefill of 2,048 tokens, with their shares of the fp32 bounds), the mixed workload at the
Llama 3.2 3B shape (32 requests, prompts of 128 to 4,096 tokens, chunked prefill under a
2,048-token budget beside decode steps, 256 new tokens each) and long-context decoding at the
Llama 3.1 8B shape, all 32 layers (batch 16 at 32,768-token prompts, 128 new tokens; before it
decode at batch 1 and 8 over 512-token prompts); the 32-bit, 3B and 8B models draw their random
weights on the device.
``--phase fogorax`` leaves the default workload alone and measures the Fogorax design instead:
decode (at ``--batch`` over ``--prompt-len``-token prompts) and a 2,048-token prefill at a few
layer sizes, each beside a Llama model of equal sizes whose layers all have the same sliding
window, the engine's closest existing model.
``--phase rudorax`` does the same for the Rudorax design (window attention and matrix-memory
layers in turn, routed experts), beside a Llama model whose dense feed-forward is as wide as
what a Rudorax token uses.
``--phase ludelix`` measures the Ludelix design (gated linear attention, attention whose values
are its keys, chunked attention beside a retention, experts chosen by a table) beside Rudorax,
the closest existing model, at equal sizes.
Peaks are the published MI355X ones: HBM 8 TB/s; dense MFMA 2.5 PFLOP/s for bf16, 157.3 TFLOP/s
for fp32.
"""

from __future__ import annotations

import argparse
import json
import os
import sys
import tempfile
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
if ROOT not in sys.path:
    sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0
MFMA_PEAK = {"bfloat16": 2.5e15, "float32": 157.3e12}
CONTEXT_CAP = 8192
BLOCK_SIZE = 16
PREFILL_TOKENS = 2048
MODEL_NAMES = {"llama-1b": "Llama 3.2 1B", "llama-3b": "Llama 3.2 3B", "llama-8b": "Llama 3.1 8B"}
# The model of the reference's own serving benchmark (benchmarks/BENCHMARK_REPORT.md:28-29,
# src/tokenvault/model_loader.py:24-27): 26.1M parameters.
SMALL = {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "vocab_size": 8192,
         "hidden_size": 512, "num_hidden_layers": 6, "num_attention_heads": 8, "num_key_value_heads": 4,
         "head_dim": 64, "intermediate_size": 1408, "max_position_embeddings": 2048,
         "rope_theta": 10000.0, "rope_scaling": None, "rms_norm_eps": 1e-6, "hidden_act": "silu",
         "tie_word_embeddings": False}


def build_engine(model, dtype, max_num_seqs, num_tokens_cached, use_graphs=True, run_steps=None,
                 context_cap=CONTEXT_CAP):
    """``model``: a model folder, or a config.json dictionary whose random weights are drawn on
    the device."""
    import kvforge_amd
    from kvforge_amd import CacheConfig, EngineConfig, InferenceEngine, SchedulerConfig

    num_blocks = -(-num_tokens_cached // BLOCK_SIZE) + max_num_seqs + 8
    cfg = EngineConfig(
        cache=CacheConfig(block_size=BLOCK_SIZE, num_blocks=num_blocks, watermark=0.0),
        scheduler=SchedulerConfig(max_num_seqs=max_num_seqs, max_num_batched_tokens=PREFILL_TOKENS,
                                  max_model_len=context_cap),
        dtype=dtype, use_graphs=use_graphs)
    if run_steps is not None:
        cfg.decode_run_steps = run_steps
    if isinstance(model, dict):
        return InferenceEngine.from_config(model, cfg, on_device=True)
    return InferenceEngine.from_folder(model, cfg)


def random_prompts(vocab, n, length, seed):
    import torch
    g = torch.Generator().manual_seed(seed)
    return [torch.randint(1, vocab, (length,), generator=g).tolist() for _ in range(n)]


def early_tokens(batch, prompt_len):
    """Most tokens a request decodes before the last prompt of the batch has been read."""
    return -(-batch * prompt_len // PREFILL_TOKENS) + 1


def decode_run(engine, vocab, batch, prompt_len, steps, warmup, seed=0):
    """Prefill ``batch`` prompts, run ``warmup`` decode steps untimed, then time ``steps``."""
    import torch
    from kvforge_amd import SamplingParams

    # requests admitted first decode while the later prompts are still being read: leave them
    # room for that, so that every request lives through the timed steps
    params = SamplingParams(max_tokens=steps + warmup + early_tokens(batch, prompt_len) + 8,
                            temperature=0.0, ignore_eos=True)
    for p in random_prompts(vocab, batch, prompt_len, seed):
        engine.add_request(p, params)
    while any(not r.decoding for r in engine.scheduler.requests.values()) or engine.scheduler.num_waiting:
        engine.step()
    sched = engine.scheduler
    run_limit, run_ahead = sched.run_limit, sched.run_ahead

    def decode_steps(n):
        """Exactly ``n`` decode steps of the whole batch (the engine may take several between two
        looks of the host; the last run is cut to fit, and no run is queued ahead that these
        ``n`` steps would not read); returns the tokens produced."""
        produced, start = 0, engine.runner.num_forward_passes
        while engine.runner.num_forward_passes - start < n:
            left = n - (engine.runner.num_forward_passes - start)
            sched.run_limit = min(run_limit, left)
            sched.run_ahead = run_ahead and left >= 2 * run_limit
            produced += sum(len(o.new_token_ids) for o in engine.step())
        sched.run_limit, sched.run_ahead = run_limit, run_ahead
        assert engine.runner.num_forward_passes - start == n
        return produced

    decode_steps(warmup)
    assert len(engine.scheduler.running) == batch
    ctx_start = [r.num_tokens for r in engine.scheduler.running]
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    produced = decode_steps(steps)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    ctx_end = [r.num_tokens for r in engine.scheduler.running]
    assert len(ctx_end) == batch and produced == batch * steps, (len(ctx_end), produced)
    for rid in list(engine.scheduler.requests):
        engine.abort_request(rid)
    mean_ctx = (sum(ctx_start) + sum(ctx_end)) / 2.0 / max(1, batch)
    return {"tokens": produced, "seconds": dt, "tok_s": produced / dt, "ms_per_step": dt / steps * 1e3,
            "mean_ctx": mean_ctx}


def prefill_run(engine, vocab, tokens, repeats=3, seed=1):
    import torch
    from kvforge_amd import SamplingParams

    best = None
    params = SamplingParams(max_tokens=1, temperature=0.0, ignore_eos=True)
    for i in range(repeats + 1):
        prompt = random_prompts(vocab, 1, tokens, seed + i)[0]
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        engine.generate([prompt], params)
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        if i > 0:                      # the first run warms buffers and kernels
            best = dt if best is None else min(best, dt)
    return best


def mixed_run(engine, vocab, requests, new_tokens, seed=0):
    """``requests`` prompts of 128 to 4,096 tokens (uniform), all there at once: chunked prefill
    under the token budget mixed with the decode steps of those already running, ``new_tokens``
    each.  Returns prompt tokens, generated tokens and seconds."""
    import random
    import torch
    from kvforge_amd import SamplingParams

    rng = random.Random(seed)
    g = torch.Generator().manual_seed(seed)
    lens = [rng.randint(128, 4096) for _ in range(requests)]
    prompts = [torch.randint(1, vocab, (n,), generator=g).tolist() for n in lens]
    params = SamplingParams(max_tokens=new_tokens, temperature=0.0, ignore_eos=True)
    engine.generate(prompts[:2], SamplingParams(max_tokens=24, temperature=0.0, ignore_eos=True))  # warm-up
    engine.metrics.reset()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    outs = engine.generate(prompts, params)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    mixed_run.last = {"lens": lens, "steps": engine.metrics.num_steps,
                      "step_tokens": list(engine.metrics.batched_tokens)}
    return sum(lens), sum(len(o.output_token_ids) for o in outs), dt


def burst_run(folder, vocab, dtype, use_graphs, seed=0):
    """The workload of the reference's serving benchmark (benchmarks/BENCHMARK_REPORT.md:30-36):
    48 requests, all there at once, prompts of 16 to 128 tokens and 8 to 128 new tokens (uniform),
    greedy, eos ignored; at most 16 sequences and 1,024 tokens in a step, 1,024 pages of 16
    tokens, chunked prefill, first come first served."""
    import random
    import torch
    from kvforge_amd import CacheConfig, EngineConfig, InferenceEngine, SamplingParams, SchedulerConfig

    rng = random.Random(seed)
    g = torch.Generator().manual_seed(seed)
    lens = [rng.randint(16, 128) for _ in range(48)]
    news = [rng.randint(8, 128) for _ in range(48)]
    prompts = [torch.randint(1, vocab, (n,), generator=g).tolist() for n in lens]
    params = [SamplingParams(max_tokens=n, temperature=0.0, ignore_eos=True) for n in news]
    cfg = EngineConfig(cache=CacheConfig(block_size=16, num_blocks=1024),
                       scheduler=SchedulerConfig(max_num_seqs=16, max_num_batched_tokens=1024),
                       dtype=dtype, use_graphs=use_graphs)
    best = None
    engine = InferenceEngine.from_folder(folder, cfg)
    for _ in range(3):                               # the first pass compiles, captures and warms
        engine.metrics.reset()
        passes = engine.runner.num_forward_passes
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        outs = engine.generate(prompts, params)
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        generated = sum(len(o.output_token_ids) for o in outs)
        assert generated == sum(news)
        summary = engine.metrics.summary()
        if best is None or dt < best[0]:
            best = (dt, generated, summary, engine.runner.num_forward_passes - passes)
    return sum(lens), best


def decode_bytes(engine, nums, elem, batch, mean_ctx):
    """What a decode step has to read: every weight it uses once, and the cache of the live
    requests."""
    return engine.model.weight_bytes + batch * mean_ctx * nums["kv_values_per_token"] * elem


def prefill_flops(nums, n):
    """Linear layers over ``n`` tokens, the head for one row, causal attention."""
    return (2.0 * n * nums["linear_params"] + 2.0 * nums["head_params"]
            + 2.0 * n * n * nums["attn_hd"] * nums["layers"])


def fp32_points(cfg, vocab, nums, steps=48, warmup=8):
    """The 1B shape in true 32-bit, weights drawn and held in 32-bit on the device: decode at
    batch 1 and 8, prefill of 2,048 tokens."""
    import torch
    out = {}
    for b in (8, 1):
        need = b * (512 + steps + warmup + early_tokens(b, 512) + 32)
        engine = build_engine(cfg, "float32", b, max(need, PREFILL_TOKENS + 64))
        r = decode_run(engine, vocab, b, 512, steps, warmup)
        out[f"fp32_decode_b{b}"] = round(r["tok_s"], 1)
        out[f"fp32_decode_b{b}_ms"] = round(r["ms_per_step"], 4)
        out[f"fp32_decode_b{b}_hbm_frac"] = round(
            decode_bytes(engine, nums, 4, b, r["mean_ctx"]) / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4)
        if b == 8:
            s = prefill_run(engine, vocab, PREFILL_TOKENS, repeats=2)
            out["fp32_prefill_tok_s"] = round(PREFILL_TOKENS / s, 1)
            out["fp32_prefill_ms"] = round(s * 1e3, 3)
            out["fp32_prefill_frac"] = round(prefill_flops(nums, PREFILL_TOKENS) / s / MFMA_PEAK["float32"], 4)
        del engine
        torch.cuda.empty_cache()
    return out


def longer_1b_points(folder, vocab, nums, steps=32, warmup=4):
    """The 1B shape in bf16 further out: decode at batch 8 and 64 over contexts of 4,096 and
    8,192 tokens (their share of the HBM roofline), and one prompt of 8,192 tokens read in
    portions of 2,048 (its share of the matrix-core peak)."""
    import torch
    out = {}
    for ctx in (4096, 8192):
        for b in (8, 64):
            prompt = ctx - steps - warmup - 8
            need = b * (prompt + steps + warmup + early_tokens(b, prompt) + 32)
            engine = build_engine(folder, "bfloat16", b, need, context_cap=ctx + 1024)
            r = decode_run(engine, vocab, b, prompt, steps, warmup)
            key = f"decode_b{b}_ctx{ctx}"
            out[key] = round(r["tok_s"], 1)
            out[key + "_ms"] = round(r["ms_per_step"], 4)
            out[key + "_hbm_frac"] = round(
                decode_bytes(engine, nums, 2, b, r["mean_ctx"]) / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4)
            if ctx == 8192 and b == 8:
                s = prefill_run(engine, vocab, 8192, repeats=2)
                out["prefill_8192_tok_s"] = round(8192 / s, 1)
                out["prefill_8192_ms"] = round(s * 1e3, 3)
                out["prefill_8192_frac"] = round(prefill_flops(nums, 8192) / s / MFMA_PEAK["bfloat16"], 4)
            del engine
            torch.cuda.empty_cache()
    return out


def mixed_3b_points(requests=32, new_tokens=256):
    """The mixed workload at the Llama 3.2 3B shape, bf16: 32 requests with prompts of 128 to 4,096
    tokens, chunked prefill under a 2,048-token budget, 256 decoded tokens each."""
    import torch
    import kvforge_amd
    cfg = kvforge_amd.preset_dict("llama-3b")
    nums = model_numbers(cfg, cfg["num_hidden_layers"])
    engine = build_engine(cfg, "bfloat16", requests, requests * (4096 + new_tokens + 64))
    prompt_tokens, generated, dt = mixed_run(engine, cfg["vocab_size"], requests, new_tokens)
    info = mixed_run.last
    flops = 2.0 * nums["linear_params"] * (prompt_tokens + generated)
    cache_read = 0.0
    per_token = nums["kv_values_per_token"] * 2
    for n in info["lens"]:
        flops += 2.0 * n * n * nums["attn_hd"] * nums["layers"]                      # the prompt, causal
        flops += 4.0 * new_tokens * (n + new_tokens / 2) * nums["attn_hd"] * nums["layers"]
        cache_read += new_tokens * (n + new_tokens / 2) * per_token                  # decode steps
    read = info["steps"] * engine.model.weight_bytes + cache_read
    out = {"mixed_3b_tok_s": round((prompt_tokens + generated) / dt, 1),
           "mixed_3b_gen_tok_s": round(generated / dt, 1), "mixed_3b_s": round(dt, 4),
           "mixed_3b_steps": info["steps"], "mixed_3b_ms_per_step": round(dt / info["steps"] * 1e3, 4),
           "mixed_3b_mfma_frac": round(flops / dt / MFMA_PEAK["bfloat16"], 4),
           "mixed_3b_hbm_frac": round(read / dt / 1e9 / HBM_PEAK_GBS, 4)}
    del engine
    torch.cuda.empty_cache()
    return out


def long_8b_points(batch=16, prompt_len=32768, new_tokens=128, warmup=8):
    """Long-context decode at the Llama 3.1 8B shape, all 32 layers, bf16: batch 16 at prompts of
    32,768 tokens, 128 new tokens each; before it decode at batch 1 and 8 over short prompts."""
    import torch
    import kvforge_amd
    cfg = kvforge_amd.preset_dict("llama-8b")
    nums = model_numbers(cfg, cfg["num_hidden_layers"])
    steps = new_tokens - 1
    need = batch * (prompt_len + steps + warmup + early_tokens(batch, prompt_len) + 32)
    engine = build_engine(cfg, "bfloat16", batch, need, context_cap=prompt_len + 1024)
    short = {}
    for b in (1, 8):        # the same model over short contexts: 512-token prompts, batch 1 and 8
        r = decode_run(engine, cfg["vocab_size"], b, 512, 48, 8)
        short[f"decode_8b_b{b}"] = round(r["tok_s"], 1)
        short[f"decode_8b_b{b}_ms"] = round(r["ms_per_step"], 4)
        short[f"decode_8b_b{b}_hbm_frac"] = round(
            decode_bytes(engine, nums, 2, b, r["mean_ctx"]) / (r["seconds"] / 48) / 1e9 / HBM_PEAK_GBS, 4)
    t0 = time.perf_counter()
    r = decode_run(engine, cfg["vocab_size"], batch, prompt_len, steps, warmup)
    total = time.perf_counter() - t0
    read = decode_bytes(engine, nums, 2, batch, r["mean_ctx"])
    out = {"long_8b_tok_s": round(r["tok_s"], 1), "long_8b_ms_per_step": round(r["ms_per_step"], 4),
           "long_8b_hbm_frac": round(read / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4),
           "long_8b_layers": cfg["num_hidden_layers"], "long_8b_batch": batch,
           "long_8b_context": int(r["mean_ctx"]), "long_8b_steps": steps,
           "long_8b_prefill_tok_s": round(batch * prompt_len / max(total - r["seconds"], 1e-9), 1),
           **short}
    del engine
    torch.cuda.empty_cache()
    return out


def products_run(cfg, rows, repeats=6):
    """The four matrix products of one layer alone, ``rows`` rows of bf16 activations each over
    ``repeats`` copies of its weight in turn (so that no copy is found in a cache), through the
    same entry points the parts use: microseconds per product.  For profiles and counters of a
    single kernel."""
    import torch
    from kvforge_amd.kernels import ops
    h, H, KV, d, I = (cfg["hidden_size"], cfg["num_attention_heads"], cfg["num_key_value_heads"],
                      cfg["head_dim"], cfg["intermediate_size"])
    dev, bf = "cuda", torch.bfloat16
    ops.library_ready(dev)
    out = {}
    for name, (n, k) in {"qkv": ((H + 2 * KV) * d, h), "o": (h, H * d), "gate_up": (2 * I, h), "down": (h, I)}.items():
        ws = [ops.streamed((torch.randn(n, k, device=dev) * 0.02).to(bf)) for _ in range(repeats)]
        a = (torch.randn(rows, k, device=dev)).to(bf)
        stream = torch.zeros(rows, n, device=dev)
        plain = torch.empty(rows, n, device=dev, dtype=bf)
        gated = torch.empty(rows, n // 2, device=dev, dtype=bf)

        def launch(w):
            if name in ("o", "down"):
                ops.gemm(a, w, stream, accumulate=True)
            elif name == "gate_up" and ops.bf16_kernel_takes(a, w, False, True):
                ops.gemm_fused(a, w, gated, silu_pairs=True)
            else:
                ops.gemm(a, w, plain)
        for w in ws:
            launch(w)
        torch.cuda.synchronize()
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        e0.record()
        for w in ws:
            launch(w)
        e1.record()
        torch.cuda.synchronize()
        out[f"{name}_us"] = round(e0.elapsed_time(e1) * 1e3 / repeats, 2)
        del ws
    return out


# (name, width, heads, kv heads, head size, feed-forward, layers, vocabulary, per-layer token input)
FOGORAX_SIZES = [("w1024", 1024, 16, 4, 64, 4096, 8, 32000, 32),
                 ("w2048", 2048, 32, 8, 64, 8192, 8, 128256, 64),
                 ("w4096", 4096, 32, 8, 128, 14336, 4, 128256, 128)]
FOGORAX_WINDOW, FOGORAX_KEEP = 1024, 4


def fogorax_points(dtype, batch, prompt_len, steps, warmup, use_graphs=True):
    """Fogorax at a few sizes that resemble a real model's layers, beside a Llama model of the
    same sizes with the same sliding window in every layer; random weights drawn on the device.
    Per size and model: ms per decode step, its share of the HBM roofline, tokens a second of a
    2,048-token prefill and its share of the matrix-core peak."""
    import torch
    from kvforge_amd.config.presets import fogorax as fogorax_config

    elem = 2 if dtype == "bfloat16" else 4
    out = {}
    for name, w, H, KV, d, ff, layers, vocab, side in FOGORAX_SIZES:
        llama = {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "vocab_size": vocab,
                 "hidden_size": w, "num_hidden_layers": layers, "num_attention_heads": H,
                 "num_key_value_heads": KV, "head_dim": d, "intermediate_size": ff,
                 "max_position_embeddings": CONTEXT_CAP, "rope_theta": 500000.0, "rope_scaling": None,
                 "rms_norm_eps": 1e-5, "hidden_act": "silu", "tie_word_embeddings": False,
                 "sliding_window": FOGORAX_WINDOW, "layer_types": ["sliding_attention"] * layers}
        fog = fogorax_config(vocab=vocab, width=w, layers=layers, heads=H, kv_heads=KV, dim=d, ff=ff,
                             window=FOGORAX_WINDOW, keep_first=FOGORAX_KEEP, side_dim=side,
                             max_positions=CONTEXT_CAP, share_every=2)
        nums = {"llama": model_numbers(llama, layers)}
        # Fogorax: q, gate and output projections in every layer, keys and values in every other
        # one, three feed-forward matrices, the two small ones of the per-layer input
        per_layer = w * d * 3 * H + w * d * KV + 3 * w * ff + 2 * w * side
        nums["fogorax"] = {"linear_params": layers * per_layer, "head_params": vocab * w,
                           "kv_values_per_token": layers * KV * d, "attn_hd": H * d, "layers": layers}
        for model, cfg in (("llama", llama), ("fogorax", fog)):
            need = batch * (prompt_len + steps + warmup + early_tokens(batch, prompt_len) + 32)
            engine = build_engine(cfg, dtype, batch, max(need, PREFILL_TOKENS + 64), use_graphs=use_graphs)
            r = decode_run(engine, vocab, batch, prompt_len, steps, warmup)
            ctx = min(r["mean_ctx"], FOGORAX_WINDOW + FOGORAX_KEEP)
            s = prefill_run(engine, vocab, PREFILL_TOKENS, repeats=2)
            out[f"{name}_{model}"] = {
                "decode_ms": round(r["ms_per_step"], 4), "decode_tok_s": round(r["tok_s"], 1),
                "decode_hbm_frac": round(decode_bytes(engine, nums[model], elem, batch, ctx)
                                         / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4),
                "prefill_tok_s": round(PREFILL_TOKENS / s, 1), "prefill_ms": round(s * 1e3, 3),
                "prefill_frac": round(prefill_flops(nums[model], PREFILL_TOKENS) / s / MFMA_PEAK[dtype], 4)}
            del engine
            torch.cuda.empty_cache()
    return out


# (name, width, q heads, kv heads, head size, recurrent heads, their key size, their value size,
#  expert width, experts, chosen, identity outputs, shared width, layers, vocabulary)
RUDORAX_SIZES = [("w1024", 1024, 16, 4, 64, 4, 128, 256, 512, 16, 2, 2, 1024, 8, 32000),
                 ("w2048", 2048, 32, 8, 64, 8, 128, 256, 1024, 32, 4, 2, 2048, 8, 128256),
                 ("w4096", 4096, 32, 8, 128, 8, 256, 512, 2048, 32, 4, 2, 4096, 4, 128256)]
RUDORAX_WINDOW = 1024


def rudorax_points(dtype, batch, prompt_len, steps, warmup, use_graphs=True, only=None):
    """Rudorax at a few sizes that resemble a real model's layers (attention and matrix-memory
    layers in turn, routed experts in all), beside a Llama model of the same width, heads and
    window whose dense feed-forward is as wide as what a Rudorax token uses (its chosen experts
    plus the shared one); random weights drawn on the device.  Per size and model: ms per decode
    step, its share of the HBM roofline, tokens a second of a 2,048-token prefill and its share
    of the matrix-core peak.  A Rudorax decode step has to read: the mixers, routers and shared
    experts once, the experts that the batch's tokens are expected to choose (a share
    ``1 - (1 - top/experts)^batch`` of them), the window's keys and values, and every sequence's
    recurrent state (read and written)."""
    import torch
    from kvforge_amd.config.presets import rudorax_stack

    elem = 2 if dtype == "bfloat16" else 4
    out = {}
    for name, w, H, KV, d, Hm, dk, dv, ff, E, top, ident, shared, layers, vocab in RUDORAX_SIZES:
        if only and name not in only:
            continue
        dense = top * ff + shared
        llama = {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "vocab_size": vocab,
                 "hidden_size": w, "num_hidden_layers": layers, "num_attention_heads": H,
                 "num_key_value_heads": KV, "head_dim": d, "intermediate_size": dense,
                 "max_position_embeddings": CONTEXT_CAP, "rope_theta": 500000.0, "rope_scaling": None,
                 "rms_norm_eps": 1e-5, "hidden_act": "silu", "tie_word_embeddings": False,
                 "sliding_window": RUDORAX_WINDOW, "layer_types": ["sliding_attention"] * layers}
        rud = rudorax_stack(vocab=vocab, width=w, pairs=layers // 2, heads=H, kv_heads=KV, dim=d,
                            window=RUDORAX_WINDOW, lstm_heads=Hm, lstm_dim=dk, lstm_vdim=dv, ff=ff,
                            experts=E, top=top, identity=ident, shared_ff=shared, max_positions=CONTEXT_CAP)
        attn = w * d * (2 * H + 2 * KV)
        lstm = w * (2 * Hm * dk + 3 * Hm * dv + 2 * Hm)
        routed = 3 * w * ff
        fixed = (layers // 2) * (attn + lstm) + layers * (3 * w * shared + w * (E + ident))
        nums = {"llama": model_numbers(llama, layers),
                "rudorax": {"linear_params": fixed + layers * top * routed, "head_params": vocab * w,
                            "kv_values_per_token": 2 * (layers // 2) * KV * d, "attn_hd": H * d,
                            "layers": layers // 2}}
        touched = E * (1.0 - (1.0 - top / E) ** batch)
        state_bytes = (layers // 2) * Hm * (dk * dv + dk + 1) * 4 * 2
        for model, cfg in (("llama", llama), ("rudorax", rud)):
            need = batch * (prompt_len + steps + warmup + early_tokens(batch, prompt_len) + 32)
            engine = build_engine(cfg, dtype, batch, max(need, PREFILL_TOKENS + 64), use_graphs=use_graphs)
            r = decode_run(engine, vocab, batch, prompt_len, steps, warmup)
            ctx = min(r["mean_ctx"], RUDORAX_WINDOW)
            s = prefill_run(engine, vocab, PREFILL_TOKENS, repeats=2)
            if model == "llama":
                read = decode_bytes(engine, nums[model], elem, batch, ctx)
            else:
                read = ((fixed + layers * touched * routed + vocab * w) * elem
                        + batch * (ctx * nums[model]["kv_values_per_token"] * elem + state_bytes))
            out[f"{name}_{model}"] = {
                "decode_ms": round(r["ms_per_step"], 4), "decode_tok_s": round(r["tok_s"], 1),
                "decode_hbm_frac": round(read / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4),
                "prefill_tok_s": round(PREFILL_TOKENS / s, 1), "prefill_ms": round(s * 1e3, 3),
                "prefill_frac": round(prefill_flops(nums[model], PREFILL_TOKENS) / s / MFMA_PEAK[dtype], 4)}
            del engine
            torch.cuda.empty_cache()
    return out


# (name, width, q heads, kv heads, head size, latent heads' plain / rotated / value size, latent rank,
#  memory heads, their size, feed-forward, groups of four layers, vocabulary)
BUZINEX_SIZES = [("w1024", 1024, 16, 4, 64, 64, 32, 64, 192, 16, 64, 4096, 2, 32000),
                 ("w2048", 2048, 32, 8, 64, 64, 32, 64, 192, 32, 64, 8192, 2, 128256),
                 ("w4096", 4096, 32, 8, 128, 128, 64, 128, 192, 64, 64, 14336, 1, 128256)]
BUZINEX_WINDOW, BUZINEX_DECAY_RANK = 1024, 64


def buzinex_points(dtype, batch, prompt_len, steps, warmup, use_graphs=True, only=None):
    """Buzinex at a few sizes that resemble a real model's layers (groups of capped attention,
    latent attention, a decaying matrix memory without a feed-forward, latent attention), beside
    a Llama model of the same width, heads, feed-forward and number of layers that keeps every
    key; random weights drawn on the device.  Per size and model: ms per decode step, its share
    of the HBM roofline, tokens a second of a 2,048-token prefill and its share of the
    matrix-core peak.  A Buzinex decode step has to read: every matrix once, the keys and values
    of the attention layers, one latent row (``rot_dim + kv_rank``) per token of the window in
    the latent layers, and every sequence's memories (read and written)."""
    import torch
    from kvforge_amd.config.presets import buzinex_stack

    elem = 2 if dtype == "bfloat16" else 4
    out = {}
    for name, w, H, KV, d, ld, lr, lv, rank, Hm, dm, ff, groups, vocab in BUZINEX_SIZES:
        if only and name not in only:
            continue
        layers = 4 * groups
        llama = {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "vocab_size": vocab,
                 "hidden_size": w, "num_hidden_layers": layers, "num_attention_heads": H,
                 "num_key_value_heads": KV, "head_dim": d, "intermediate_size": ff,
                 "max_position_embeddings": CONTEXT_CAP, "rope_theta": 500000.0, "rope_scaling": None,
                 "rms_norm_eps": 1e-5, "hidden_act": "silu", "tie_word_embeddings": True}
        buz = buzinex_stack(vocab=vocab, width=w, groups=groups, heads=H, kv_heads=KV, dim=d, latent_dim=ld,
                            rot_dim=lr, kv_rank=rank, window=BUZINEX_WINDOW, wkv_heads=Hm, wkv_dim=dm, ff=ff,
                            max_positions=CONTEXT_CAP)
        for layer in buz["layers"]:
            if layer["type"] == "latent_attention":
                layer["mixer"]["vdim"] = lv
        attn = w * d * (2 * H + 2 * KV)
        latent = w * (H * (ld + lr) + rank + lr) + H * (ld + lv) * rank + H * lv * w
        memory = 5 * w * Hm * dm + BUZINEX_DECAY_RANK * (w + Hm * dm)
        linear = groups * (attn + 2 * latent + memory + 3 * 3 * w * ff)
        nums = {"llama": model_numbers(llama, layers),
                "buzinex": {"linear_params": linear, "head_params": vocab * w,
                            "kv_values_per_token": groups * 2 * KV * d, "attn_hd": H * d, "layers": groups}}
        # what the latent layers add to a prompt's arithmetic: scores and sums over rot + rank and rank
        state_bytes = groups * (Hm * dm * dm + w) * 4 * 2
        for model, cfg in (("llama", llama), ("buzinex", buz)):
            need = batch * (prompt_len + steps + warmup + early_tokens(batch, prompt_len) + 32)
            engine = build_engine(cfg, dtype, batch, max(need, PREFILL_TOKENS + 64), use_graphs=use_graphs)
            r = decode_run(engine, vocab, batch, prompt_len, steps, warmup)
            s = prefill_run(engine, vocab, PREFILL_TOKENS, repeats=2)
            if model == "llama":
                read = decode_bytes(engine, nums[model], elem, batch, r["mean_ctx"])
                flops = prefill_flops(nums[model], PREFILL_TOKENS)
            else:
                seen = min(r["mean_ctx"], BUZINEX_WINDOW)
                read = ((linear + vocab * w) * elem
                        + batch * (r["mean_ctx"] * nums[model]["kv_values_per_token"] * elem
                                   + seen * 2 * groups * (lr + rank) * elem + state_bytes))
                n = PREFILL_TOKENS
                pairs = n * min(n, BUZINEX_WINDOW) - min(n, BUZINEX_WINDOW) ** 2 / 2.0     # (query, key) pairs under the window
                flops = (prefill_flops(nums[model], n)
                         + 2 * groups * 2.0 * pairs * H * (lr + 2 * rank)      # latent scores and sums
                         + groups * n * Hm * 4.0 * dm * dm)                      # the memories' updates and reads
            out[f"{name}_{model}"] = {
                "decode_ms": round(r["ms_per_step"], 4), "decode_tok_s": round(r["tok_s"], 1),
                "decode_hbm_frac": round(read / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4),
                "prefill_tok_s": round(PREFILL_TOKENS / s, 1), "prefill_ms": round(s * 1e3, 3),
                "prefill_frac": round(flops / s / MFMA_PEAK[dtype], 4)}
            del engine
            torch.cuda.empty_cache()
    return out


# (name, width, q heads, kv heads, head size, memory heads, their key size, their value size,
#  expert width, experts, chosen, shared width, groups of four layers, vocabulary)
LUDELIX_SIZES = [("w1024", 1024, 16, 4, 64, 4, 128, 256, 512, 16, 2, 1024, 2, 32000),
                 ("w2048", 2048, 32, 8, 64, 8, 128, 256, 1024, 32, 4, 2048, 2, 128256),
                 ("w4096", 4096, 32, 8, 128, 8, 256, 512, 2048, 32, 4, 4096, 1, 128256)]
LUDELIX_WINDOW, LUDELIX_GATE_RANK = 1024, 16


def ludelix_points(dtype, batch, prompt_len, steps, warmup, use_graphs=True, only=None):
    """Ludelix at a few sizes that resemble a real model's layers (groups of gated linear
    attention with a dense feed-forward, attention whose values are its keys, chunked attention
    beside a retention, attention again, the last three with experts chosen by a table), beside
    the engine's closest existing model, Rudorax, of the same width, heads, window, memory heads,
    experts and number of layers (window attention and matrix-memory layers in turn, routed
    experts in all); random weights drawn on the device.  Per size and model: ms per decode step,
    its share of the HBM roofline, tokens a second of a 2,048-token prefill and its share of the
    matrix-core peak.  A decode step has to read: the mixers, shared experts and dense
    feed-forwards once, the experts that the batch's tokens are expected to choose (a share
    ``1 - (1 - top/experts)^batch`` of them), the keys and values under window and chunk, and
    every sequence's memories (read and written)."""
    import torch
    from kvforge_amd.config.presets import ludelix_stack, rudorax_stack

    elem = 2 if dtype == "bfloat16" else 4
    out = {}
    for name, w, H, KV, d, Hm, dk, dv, ff, E, top, shared, groups, vocab in LUDELIX_SIZES:
        if only and name not in only:
            continue
        layers = 4 * groups
        lud = ludelix_stack(vocab=vocab, width=w, groups=groups, heads=H, kv_heads=KV, dim=d, window=LUDELIX_WINDOW,
                            mem_heads=Hm, mem_dim=dk, mem_vdim=dv, ff=ff, experts=E, top=top, shared_ff=shared,
                            max_positions=CONTEXT_CAP)
        rud = rudorax_stack(vocab=vocab, width=w, pairs=layers // 2, heads=H, kv_heads=KV, dim=d,
                            window=LUDELIX_WINDOW, lstm_heads=Hm, lstm_dim=dk, lstm_vdim=dv, ff=ff,
                            experts=E, top=top, identity=0, shared_ff=shared, max_positions=CONTEXT_CAP)
        routed = 3 * w * ff
        touched = E * (1.0 - (1.0 - top / E) ** batch)
        memory = w * Hm * (2 * dk + 3 * dv)                               # q, k, v, gate, output
        # Ludelix, a group: gla (+ its gates' two matrices) with a dense feed-forward; attention
        # (q, k, output) twice; chunked attention (q, k, v, output, a gate row per head) beside a retention
        l_fixed = groups * (memory + LUDELIX_GATE_RANK * (w + Hm * dk) + 2 * w * (top * ff + shared)
                            + 2 * w * d * (2 * H + KV) + w * d * (2 * H + 2 * KV) + w * H + memory
                            + 3 * (3 * w * shared + w))
        l_routed_layers = 3 * groups
        l_kv = 3 * groups * 2 * KV * d                                     # key and value pages of three layers a group
        l_state = groups * 2 * Hm * dk * dv * 4 * 2
        r_fixed = (layers // 2) * (w * d * (2 * H + 2 * KV) + w * (2 * Hm * dk + 3 * Hm * dv + 2 * Hm)) \
            + layers * (3 * w * shared + w * E)
        r_kv = (layers // 2) * 2 * KV * d
        r_state = (layers // 2) * Hm * (dk * dv + dk + 1) * 4 * 2
        n = PREFILL_TOKENS
        seen = min(n, LUDELIX_WINDOW)
        pairs = n * seen - seen * seen / 2.0                               # (query, key) pairs under a window
        per_model = {
            "ludelix": (lud, l_fixed, l_routed_layers, l_kv, l_state,
                        3 * groups * 4.0 * pairs * H * d + 2 * groups * n * Hm * 4.0 * dk * dv),
            "rudorax": (rud, r_fixed, layers, r_kv, r_state,
                        (layers // 2) * 4.0 * pairs * H * d + (layers // 2) * n * Hm * 4.0 * dk * dv)}
        for model, (cfg, fixed, routed_layers, kv, state_bytes, mixing) in per_model.items():
            need = batch * (prompt_len + steps + warmup + early_tokens(batch, prompt_len) + 32)
            engine = build_engine(cfg, dtype, batch, max(need, PREFILL_TOKENS + 64), use_graphs=use_graphs)
            r = decode_run(engine, vocab, batch, prompt_len, steps, warmup)
            ctx = min(r["mean_ctx"], LUDELIX_WINDOW)
            s = prefill_run(engine, vocab, PREFILL_TOKENS, repeats=2)
            read = ((fixed + routed_layers * touched * routed + vocab * w) * elem
                    + batch * (ctx * kv * elem + state_bytes))
            flops = 2.0 * n * (fixed + routed_layers * top * routed) + 2.0 * vocab * w + mixing
            out[f"{name}_{model}"] = {
                "decode_ms": round(r["ms_per_step"], 4), "decode_tok_s": round(r["tok_s"], 1),
                "decode_hbm_frac": round(read / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4),
                "prefill_tok_s": round(PREFILL_TOKENS / s, 1), "prefill_ms": round(s * 1e3, 3),
                "prefill_frac": round(flops / s / MFMA_PEAK[dtype], 4)}
            del engine
            torch.cuda.empty_cache()
    return out


# (name, width, heads of the attention layers, kv heads of Buzinex's, their head size, latent heads' plain /
#  rotated / value size, latent rank, delta memories, q/k heads they share, their key and value size, mamba2
#  memories, their value size, state size, groups, Buzinex's memories, their size, feed-forward, expert width,
#  experts, chosen, groups of four layers, vocabulary)
BALALORN_SIZES = [("w1024", 1024, 16, 4, 64, 64, 32, 64, 192, 8, 4, 128, 128, 32, 64, 128, 4, 16, 64, 4096, 1024, 16, 4, 2, 32000),
                  ("w2048", 2048, 32, 8, 64, 64, 32, 64, 192, 16, 8, 128, 128, 64, 64, 128, 8, 32, 64, 8192, 2048, 32, 4, 2, 128256),
                  ("w4096", 4096, 32, 8, 128, 128, 64, 128, 192, 32, 16, 128, 128, 128, 64, 128, 8, 64, 64, 14336, 3584, 32, 4, 1, 128256)]
BALALORN_FIELDS = ("width", "heads", "kv_heads", "head_dim", "latent_dim", "latent_rot_dim", "latent_vdim", "kv_rank",
                   "delta_heads", "delta_kv_heads", "delta_dim", "delta_vdim", "ssm_heads", "ssm_vdim", "ssm_state",
                   "ssm_groups", "wkv_heads", "wkv_dim", "ff", "expert_ff", "experts", "top", "groups", "vocab")


def balalorn_points(dtype, batch, prompt_len, steps, warmup, use_graphs=True, only=None, models=None):
    """Balalorn at a few sizes that resemble a real model's layers (groups of a gated delta rule
    with a dense feed-forward, latent attention with experts, Mamba-2 with experts, latent
    attention over the same latents with a dense feed-forward), beside the engine's closest
    existing model, Buzinex, of the same width, heads, latents, feed-forward (as wide as the chosen
    experts together) and number of layers; random weights drawn on the device.  Per size and
    model: ms per decode step, its share of the HBM roofline, tokens a second of a 2,048-token
    prefill and its share of the matrix-core peak.  A Balalorn decode step has to read: the
    mixers and dense feed-forwards once, the experts that the batch's tokens are expected to
    choose (a share ``1 - (1 - top/experts)^batch`` of them), one latent row (``rot_dim + kv_rank``) per
    token in each latent layer, and every sequence's memories (read and written)."""
    import torch
    from kvforge_amd.config.presets import balalorn_stack, buzinex_stack

    elem = 2 if dtype == "bfloat16" else 4
    out = {}
    for (name, w, H, KV, d, ld, lr, lv, rank, Hd, Gd, dk, dv, Hs, sv, N, Gs, Hm, dm, ff, eff, E, top, groups,
         vocab) in BALALORN_SIZES:
        if only and name not in only:
            continue
        bal = balalorn_stack(vocab=vocab, width=w, groups=groups, heads=H, latent_dim=ld, rot_dim=lr, kv_rank=rank,
                             mem_heads=Hd, mem_kv_heads=Gd, mem_dim=dk, mem_vdim=dv, ssm_heads=Hs, ssm_vdim=sv,
                             state=N, ssm_groups=Gs, ff=ff, moe_ff=eff, experts=E, top=top, max_positions=CONTEXT_CAP)
        buz = buzinex_stack(vocab=vocab, width=w, groups=groups, heads=H, kv_heads=KV, dim=d, latent_dim=ld,
                            rot_dim=lr, kv_rank=rank, window=BUZINEX_WINDOW, wkv_heads=Hm, wkv_dim=dm, ff=ff,
                            max_positions=CONTEXT_CAP)
        for layer in bal["layers"] + buz["layers"]:
            if layer["type"] == "latent_attention":
                layer["mixer"]["vdim"] = lv
        latent_q = w * H * (ld + lr) + H * (ld + lv) * rank + H * lv * w
        latent_kv = w * (rank + lr)
        delta = w * (2 * Gd * dk + 3 * Hd * dv + 2 * Hd)
        ssm = w * (3 * Hs * sv + 2 * Gs * N + Hs)
        routed = 3 * w * eff
        touched = E * (1.0 - (1.0 - top / E) ** batch)
        bal_fixed = groups * (delta + ssm + 2 * (latent_q + w * H) + latent_kv + 2 * 3 * w * ff + 2 * w * E)
        bal_state = groups * (Hd * dk * dv + 3 * (2 * Gd * dk + Hd * dv) + Hs * sv * N + 3 * (Hs * sv + 2 * Gs * N)) * 4 * 2
        attn = w * d * (2 * H + 2 * KV)
        memory = 5 * w * Hm * dm + BUZINEX_DECAY_RANK * (w + Hm * dm)
        buz_fixed = groups * (attn + 2 * (latent_q + latent_kv) + memory + 3 * 3 * w * ff)
        buz_state = groups * (Hm * dm * dm + w) * 4 * 2
        n = PREFILL_TOKENS
        full = n * n / 2.0                                                   # (query, key) pairs, causal
        seen = min(n, BUZINEX_WINDOW)
        windowed = n * seen - seen * seen / 2.0
        per_pair = 2.0 * H * (lr + 2 * rank)                                 # latent scores and sums
        rows = {"balalorn": (bal, bal_fixed, 2 * groups, 2 * groups * (lr + rank), None, bal_state,
                             2 * groups * full * per_pair + groups * n * (6.0 * Hd * dk * dv + 4.0 * Hs * sv * N)),
                "buzinex": (buz, buz_fixed, 0, 2 * groups * (lr + rank), BUZINEX_WINDOW, buz_state,
                            2 * groups * windowed * per_pair + groups * (full * 4.0 * H * d + n * 4.0 * Hm * dm * dm))}
        for model, (cfg, fixed, routed_layers, latent_row, window, state_bytes, mixing) in rows.items():
            if models and model not in models:
                continue
            need = batch * (prompt_len + steps + warmup + early_tokens(batch, prompt_len) + 32)
            engine = build_engine(cfg, dtype, batch, max(need, PREFILL_TOKENS + 64), use_graphs=use_graphs)
            r = decode_run(engine, vocab, batch, prompt_len, steps, warmup)
            s = prefill_run(engine, vocab, PREFILL_TOKENS, repeats=2)
            ctx = min(r["mean_ctx"], window) if window else r["mean_ctx"]
            keys = r["mean_ctx"] * groups * 2 * KV * d if model == "buzinex" else 0.0
            read = ((fixed + routed_layers * touched * routed + vocab * w) * elem
                    + batch * ((ctx * latent_row + keys) * elem + state_bytes))
            flops = 2.0 * n * (fixed + routed_layers * top * routed) + 2.0 * vocab * w + mixing
            out[f"{name}_{model}"] = {
                "decode_ms": round(r["ms_per_step"], 4), "decode_tok_s": round(r["tok_s"], 1),
                "decode_hbm_frac": round(read / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4),
                "prefill_tok_s": round(PREFILL_TOKENS / s, 1), "prefill_ms": round(s * 1e3, 3),
                "prefill_frac": round(flops / s / MFMA_PEAK[dtype], 4)}
            del engine
            torch.cuda.empty_cache()
    return out


# (name, width, latent heads, their plain / rotated / value size, query latent, key latent, attention heads beside the
#  memories, their kv heads and size, delta memories, q/k heads they share, their key and value size, rank of their
#  gates, feed-forward, expert width, experts, chosen, groups of four layers, vocabulary): every size that Balalorn has
#  as in BALALORN_SIZES
DEPOLIX_SIZES = [("w1024", 1024, 16, 64, 32, 64, 384, 192, 16, 4, 64, 8, 4, 128, 128, 128, 4096, 1024, 16, 4, 2, 32000),
                 ("w2048", 2048, 32, 64, 32, 64, 768, 192, 32, 8, 64, 16, 8, 128, 128, 128, 8192, 2048, 32, 4, 2, 128256),
                 ("w4096", 4096, 32, 128, 64, 128, 1536, 192, 32, 8, 128, 32, 16, 128, 128, 128, 14336, 3584, 32, 4, 1, 128256)]
DEPOLIX_FIELDS = ("width", "latent_heads", "latent_dim", "latent_rot_dim", "latent_vdim", "q_rank", "kv_rank", "heads",
                  "kv_heads", "head_dim", "delta_heads", "delta_kv_heads", "delta_dim", "delta_vdim", "gate_rank", "ff",
                  "expert_ff", "experts", "top", "groups", "vocab")
DEPOLIX_WINDOW, DEPOLIX_KEEP = 1024, 16


def depolix_points(dtype, batch, prompt_len, steps, warmup, use_graphs=True, only=None, models=None):
    """Depolix at a few sizes that resemble a real model's layers (groups of latent attention with a dense
    feed-forward, attention with a bias by distance beside a delta-rule memory with experts, latent attention with
    experts, the two side by side with a dense feed-forward), beside the engine's closest existing model, Balalorn, of
    the same width, latents, memories, feed-forwards and number of layers (``balalorn_points``); random weights drawn
    on the device.  Per size and model: ms per decode step, its share of the HBM roofline, tokens a second of a
    2,048-token prefill and its share of the matrix-core peak, with the bytes and products of the work itself, as
    for Balalorn."""
    import torch
    from kvforge_amd.config.presets import depolix_stack

    elem = 2 if dtype == "bfloat16" else 4
    out = {}
    for (name, w, H, ld, lr, lv, qr, rank, Ha, KV, d, Hd, Gd, dk, dv, gr, ff, eff, E, top, groups, vocab) in DEPOLIX_SIZES:
        if only and name not in only:
            continue
        if not models or "depolix" in models:
            cfg = depolix_stack(vocab=vocab, width=w, groups=groups, heads=H, latent_dim=ld, rot_dim=lr, q_rank=qr,
                                kv_rank=rank, att_heads=Ha, att_kv_heads=KV, att_dim=d, window=DEPOLIX_WINDOW, mem_heads=Hd,
                                mem_kv_heads=Gd, mem_dim=dk, mem_vdim=dv, gate_rank=gr, ff=ff, moe_ff=eff, experts=E, top=top,
                                max_positions=CONTEXT_CAP)
            for layer in cfg["layers"]:
                if layer["type"] == "latent_attention":
                    layer["mixer"]["vdim"] = lv
            latent = w * (qr + rank + lr + 2 * H * lv) + qr * H * (ld + lr) + H * (ld + lv) * rank
            left = w * (2 * Ha * d + 2 * KV * d + Ha)
            right = w * (2 * Gd * dk + 2 * Hd * dv + 2 * gr + Hd) + gr * Hd * (dk + dv)
            routed = 3 * w * eff
            touched = E * (1.0 - (1.0 - top / E) ** batch)
            fixed = groups * (2 * (latent + left + right) + 2 * 3 * w * ff + 2 * w * E)
            state_bytes = 2 * groups * (Hd * dk * dv + 3 * (2 * Gd * dk + Hd * dv) + 3 * (Ha + 2 * KV) * d) * 4 * 2
            n = PREFILL_TOKENS
            full, seen = n * n / 2.0, min(n, DEPOLIX_WINDOW)
            windowed = n * seen - seen * seen / 2.0
            mixing = 2 * groups * (full * 2.0 * H * (lr + 2 * rank) + windowed * 4.0 * Ha * d + n * 6.0 * Hd * dk * dv)
            need = batch * (prompt_len + steps + warmup + early_tokens(batch, prompt_len) + 32)
            engine = build_engine(cfg, dtype, batch, max(need, PREFILL_TOKENS + 64), use_graphs=use_graphs)
            r = decode_run(engine, vocab, batch, prompt_len, steps, warmup)
            s = prefill_run(engine, vocab, PREFILL_TOKENS, repeats=2)
            ctx = r["mean_ctx"]
            kept = min(ctx, DEPOLIX_WINDOW + DEPOLIX_KEEP) * 2 * KV * d
            read = ((fixed + 2 * groups * touched * routed + vocab * w) * elem
                    + batch * (2 * groups * (ctx * (lr + rank) + kept) * elem + state_bytes))
            flops = 2.0 * n * (fixed + 2 * groups * top * routed) + 2.0 * vocab * w + mixing
            out[f"{name}_depolix"] = {
                "decode_ms": round(r["ms_per_step"], 4), "decode_tok_s": round(r["tok_s"], 1),
                "decode_hbm_frac": round(read / (r["seconds"] / steps) / 1e9 / HBM_PEAK_GBS, 4),
                "prefill_tok_s": round(PREFILL_TOKENS / s, 1), "prefill_ms": round(s * 1e3, 3),
                "prefill_frac": round(flops / s / MFMA_PEAK[dtype], 4)}
            del engine
            torch.cuda.empty_cache()
        if not models or "balalorn" in models:
            out.update(balalorn_points(dtype, batch, prompt_len, steps, warmup, use_graphs, [name], ["balalorn"]))
    return out


def model_numbers(cfg, layers_run):
    h, H, KV, d, I, V = (cfg["hidden_size"], cfg["num_attention_heads"], cfg["num_key_value_heads"],
                         cfg["head_dim"], cfg["intermediate_size"], cfg["vocab_size"])
    per_layer = h * d * (2 * H + 2 * KV) + 3 * h * I
    return {"linear_params": layers_run * per_layer, "head_params": V * h,
            "kv_values_per_token": 2 * layers_run * KV * d, "attn_hd": H * d, "layers": layers_run}


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=255)
    ap.add_argument("--warmup", type=int, default=16)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--prompt-len", type=int, default=512)
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--preset", choices=["llama-1b", "llama-3b", "llama-8b", "small"], default="llama-1b",
                    help="layer sizes of the model (random weights); the default is the headline run")
    ap.add_argument("--context-len", type=int, default=CONTEXT_CAP,
                    help="longest request the engine admits (prompt and new tokens)")
    ap.add_argument("--layers", type=int, default=None, help="run fewer layers than the model has")
    ap.add_argument("--no-points", action="store_true",
                    help="skip decode at batch 1 and 64, the 32-bit run and the 3B and 8B workloads")
    ap.add_argument("--only-points", default=None,
                    help="comma-separated subset of longer_1b,fp32,mixed_3b,long_8b to run besides the main line")
    ap.add_argument("--no-graphs", action="store_true")
    ap.add_argument("--decode-run-steps", type=int, default=None,
                    help="decode steps the device takes between two looks of the host (engine default: 8)")
    ap.add_argument("--phase", choices=["all", "decode", "prefill", "mixed", "burst", "products", "fogorax", "rudorax", "buzinex", "ludelix", "balalorn", "depolix"],
                    default="all",
                    help="for profiles: only the decode steps at --batch, or only the prefill; "
                         "mixed: --batch requests with prompts of 128 to 4,096 tokens, chunked "
                         "prefill beside decode steps, --steps new tokens each; burst: the "
                         "workload of the reference's own serving benchmark (48 short requests "
                         "at once, 16 sequences a step), for --preset small or any other; "
                         "products: the four matrix products of a layer alone at --batch rows "
                         "(launch to launch, so short ones show the host's time); fogorax: the "
                         "Fogorax design at a few layer sizes beside a Llama model of equal sizes; "
                         "rudorax: the Rudorax design likewise (--sizes names some of them); "
                         "buzinex: the Buzinex design likewise; ludelix: the Ludelix design beside Rudorax; "
                         "balalorn: the Balalorn design beside Buzinex; depolix: the Depolix design beside Balalorn")
    ap.add_argument("--sizes", default="", help="with --phase rudorax, buzinex, ludelix, balalorn or depolix: the sizes to run, with commas")
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py measures one GPU; --gpus {args.gpus} is not supported by this engine")
        return 2

    import torch
    import kvforge_amd

    if args.phase == "fogorax":
        steps = min(args.steps, 64)
        print(json.dumps({"phase": "fogorax", "dtype": args.dtype, "batch": args.batch,
                          "prompt_len": args.prompt_len, "steps": steps, "window": FOGORAX_WINDOW,
                          "keep_first": FOGORAX_KEEP, "prefill_tokens": PREFILL_TOKENS,
                          "sizes": {n: {"width": w, "heads": H, "kv_heads": KV, "head_dim": d, "ff": ff,
                                        "layers": L, "vocab": V, "side_dim": sd}
                                    for n, w, H, KV, d, ff, L, V, sd in FOGORAX_SIZES},
                          **fogorax_points(args.dtype, args.batch, args.prompt_len, steps,
                                           min(args.warmup, 8), not args.no_graphs)}))
        return 0
    if args.phase == "rudorax":
        steps = min(args.steps, 64)
        print(json.dumps({"phase": "rudorax", "dtype": args.dtype, "batch": args.batch,
                          "prompt_len": args.prompt_len, "steps": steps, "window": RUDORAX_WINDOW,
                          "prefill_tokens": PREFILL_TOKENS,
                          "sizes": {r[0]: dict(zip(("width", "heads", "kv_heads", "head_dim", "lstm_heads",
                                                    "lstm_dim", "lstm_vdim", "expert_ff", "experts", "top",
                                                    "identity", "shared_ff", "layers", "vocab"), r[1:]))
                                    for r in RUDORAX_SIZES},
                          **rudorax_points(args.dtype, args.batch, args.prompt_len, steps,
                                           min(args.warmup, 8), not args.no_graphs,
                                           [x for x in args.sizes.split(",") if x] or None)}))
        return 0
    if args.phase == "buzinex":
        steps = min(args.steps, 64)
        print(json.dumps({"phase": "buzinex", "dtype": args.dtype, "batch": args.batch,
                          "prompt_len": args.prompt_len, "steps": steps, "window": BUZINEX_WINDOW,
                          "prefill_tokens": PREFILL_TOKENS,
                          "sizes": {r[0]: dict(zip(("width", "heads", "kv_heads", "head_dim", "latent_dim",
                                                    "latent_rot_dim", "latent_vdim", "kv_rank", "memory_heads",
                                                    "memory_dim", "ff", "groups", "vocab"), r[1:]))
                                    for r in BUZINEX_SIZES},
                          **buzinex_points(args.dtype, args.batch, args.prompt_len, steps,
                                           min(args.warmup, 8), not args.no_graphs,
                                           [x for x in args.sizes.split(",") if x] or None)}))
        return 0
    if args.phase == "ludelix":
        steps = min(args.steps, 64)
        print(json.dumps({"phase": "ludelix", "dtype": args.dtype, "batch": args.batch,
                          "prompt_len": args.prompt_len, "steps": steps, "window": LUDELIX_WINDOW,
                          "prefill_tokens": PREFILL_TOKENS,
                          "sizes": {r[0]: dict(zip(("width", "heads", "kv_heads", "head_dim", "memory_heads",
                                                    "memory_dim", "memory_vdim", "expert_ff", "experts", "top",
                                                    "shared_ff", "groups", "vocab"), r[1:]))
                                    for r in LUDELIX_SIZES},
                          **ludelix_points(args.dtype, args.batch, args.prompt_len, steps,
                                           min(args.warmup, 8), not args.no_graphs,
                                           [x for x in args.sizes.split(",") if x] or None)}))
        return 0
    if args.phase == "balalorn":
        steps = min(args.steps, 64)
        print(json.dumps({"phase": "balalorn", "dtype": args.dtype, "batch": args.batch,
                          "prompt_len": args.prompt_len, "steps": steps, "buzinex_window": BUZINEX_WINDOW,
                          "prefill_tokens": PREFILL_TOKENS,
                          "sizes": {r[0]: dict(zip(BALALORN_FIELDS, r[1:])) for r in BALALORN_SIZES},
                          **balalorn_points(args.dtype, args.batch, args.prompt_len, steps,
                                            min(args.warmup, 8), not args.no_graphs,
                                            [x for x in args.sizes.split(",") if x] or None)}))
        return 0
    if args.phase == "depolix":
        steps = min(args.steps, 64)
        print(json.dumps({"phase": "depolix", "dtype": args.dtype, "batch": args.batch,
                          "prompt_len": args.prompt_len, "steps": steps, "window": DEPOLIX_WINDOW,
                          "keep_first": DEPOLIX_KEEP, "prefill_tokens": PREFILL_TOKENS,
                          "sizes": {r[0]: dict(zip(DEPOLIX_FIELDS, r[1:])) for r in DEPOLIX_SIZES},
                          **depolix_points(args.dtype, args.batch, args.prompt_len, steps,
                                           min(args.warmup, 8), not args.no_graphs,
                                           [x for x in args.sizes.split(",") if x] or None)}))
        return 0
    if args.preset == "small" and args.phase != "burst":
        print("--preset small goes with --phase burst")
        return 2
    cfg = dict(SMALL) if args.preset == "small" else kvforge_amd.preset_dict(args.preset)
    full_layers = cfg["num_hidden_layers"]
    layers_run = args.layers or full_layers
    cfg["num_hidden_layers"] = layers_run
    elem = 2 if args.dtype == "bfloat16" else 4
    nums = model_numbers(cfg, layers_run)
    vocab = cfg["vocab_size"]

    if args.phase == "products":
        print(json.dumps({"phase": "products", "model": args.preset, "rows": args.batch, "dtype": "bfloat16",
                          **products_run(cfg, args.batch)}))
        return 0
    with tempfile.TemporaryDirectory(prefix="kvforge_bench_") as folder:
        kvforge_amd.write_random_model(folder, cfg, seed=0, dtype=args.dtype)
        if args.phase == "burst":
            prompt_tokens, (dt, generated, summary, passes) = burst_run(folder, vocab, args.dtype,
                                                                        not args.no_graphs)
            print(json.dumps({
                "phase": "burst", "model": args.preset, "dtype": args.dtype, "requests": 48,
                "prompt_tokens": prompt_tokens, "generated_tokens": generated, "seconds": round(dt, 4),
                "output_tok_s": round(generated / dt, 1), "forward_passes": passes,
                "ttft_p50_ms": round(summary["ttft_p50_ms"], 2), "ttft_p99_ms": round(summary["ttft_p99_ms"], 2),
                "tpot_p50_ms": round(summary["tpot_p50_ms"], 3),
                "reference_published": "84.6 output tok/s, TTFT p50 9,340 ms, TPOT p50 157.6 ms: "
                                       "small preset, fp32, one laptop CPU thread "
                                       "(benchmarks/BENCHMARK_REPORT.md:80)"}))
            return 0
        if args.phase == "mixed":
            engine = build_engine(folder, args.dtype, args.batch, args.batch * (4096 + args.steps + 64),
                                  use_graphs=not args.no_graphs, run_steps=args.decode_run_steps,
                                  context_cap=args.context_len)
            prompt_tokens, generated, dt = mixed_run(engine, vocab, args.batch, args.steps)
            print(json.dumps({"phase": "mixed", "model": args.preset, "requests": args.batch,
                              "dtype": args.dtype, "prompt_tokens": prompt_tokens,
                              "generated_tokens": generated, "seconds": round(dt, 4),
                              "total_tok_s": round((prompt_tokens + generated) / dt, 1),
                              "generated_tok_s": round(generated / dt, 1)}))
            return 0
        results = {}
        points = args.phase == "all" and not args.no_points
        batches = [args.batch] + ([b for b in (1, 64) if b != args.batch] if points else [])
        prefill_s = None
        for b in batches:
            need = b * (args.prompt_len + args.steps + args.warmup + early_tokens(b, args.prompt_len) + 32)
            engine = build_engine(folder, args.dtype, max(b, 1), max(need, PREFILL_TOKENS + 64),
                                  use_graphs=not args.no_graphs, run_steps=args.decode_run_steps,
                                  context_cap=args.context_len)
            if args.phase != "prefill":
                results[b] = decode_run(engine, vocab, b, args.prompt_len, args.steps, args.warmup)
            if b == args.batch:
                if args.phase != "decode":
                    prefill_s = prefill_run(engine, vocab, PREFILL_TOKENS)
                weight_bytes = engine.model.weight_bytes
            del engine
            torch.cuda.empty_cache()
        more = {}
        if points and args.preset == "llama-1b" and layers_run == full_layers:
            chosen = set((args.only_points or "longer_1b,fp32,mixed_3b,long_8b").split(","))
            for name, fn in (("longer_1b", lambda: longer_1b_points(folder, vocab, nums)),
                             ("fp32", lambda: fp32_points(cfg, vocab, nums)),
                             ("mixed_3b", mixed_3b_points), ("long_8b", long_8b_points)):
                if name not in chosen:
                    continue
                try:
                    more.update(fn())
                except Exception as e:   # the main line is printed whatever happens to an extra
                    print(f"bench: {name} failed: {type(e).__name__}: {e}", file=sys.stderr)
                    more[f"{name}_failed"] = 1
                    torch.cuda.empty_cache()

    if args.phase != "all":  # a partial run for a profile: say what was timed and stop
        part = ({"prefill_ms": round(prefill_s * 1e3, 3)} if args.phase == "prefill" else
                {"ms_per_step": round(results[args.batch]["ms_per_step"], 4)})
        print(json.dumps({"phase": args.phase, "batch": args.batch, "dtype": args.dtype, **part}))
        return 0
    main_run = results[args.batch]
    run_steps_used = args.decode_run_steps or kvforge_amd.EngineConfig().decode_run_steps
    step_s = main_run["seconds"] / args.steps
    kv_bytes = args.batch * main_run["mean_ctx"] * nums["kv_values_per_token"] * elem
    achieved = (weight_bytes + kv_bytes) / step_s / 1e9
    n = PREFILL_TOKENS
    line = {
        "metric": "decode tok/s (%s shape, batch %d)" % (MODEL_NAMES[args.preset], args.batch),
        "value": round(main_run["tok_s"], 1), "unit": "tokens/s", "n_gpus": 1,
        "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(main_run["ms_per_step"], 4), "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
        "data": "synthetic: random weights N(0, 0.02), uniform-random token ids",
        "config": {
            "model": MODEL_NAMES[args.preset].lower().replace(" ", "-") + "-shape", "layers": full_layers, "layers_run": layers_run,
            "hidden": cfg["hidden_size"], "heads": cfg["num_attention_heads"],
            "kv_heads": cfg["num_key_value_heads"], "head_dim": cfg["head_dim"],
            "intermediate": cfg["intermediate_size"], "vocab": vocab,
            "tied_embeddings": cfg["tie_word_embeddings"],
            "rope": "theta %.0e, llama3 factor %g" % (cfg["rope_theta"], cfg["rope_scaling"]["factor"]), "rms_norm_eps": cfg["rms_norm_eps"],
            "global_batch": args.batch, "seq_len": args.prompt_len, "new_tokens": args.steps + 1,
            "context_len": args.context_len, "block_size": BLOCK_SIZE, "parallelism": "single-gpu",
            "sampling": "greedy", "decode_run_steps": run_steps_used,
        },
        "prefill": {"value": round(n / prefill_s, 1), "tokens": n, "ms": round(prefill_s * 1e3, 3),
                    "frac": round(prefill_flops(nums, n) / prefill_s / MFMA_PEAK[args.dtype], 4)},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBS,
                     "unit": "GB/s", "frac": round(achieved / HBM_PEAK_GBS, 4)},
        "points": {**{f"decode_b{b}": round(r["tok_s"], 1) for b, r in results.items() if b != args.batch},
                   **more},
    }
    print(json.dumps(line))
    return 0


if __name__ == "__main__":
    sys.exit(main())
