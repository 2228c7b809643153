#!/usr/bin/env python3
"""Benchmark: decode tokens per second of the GPT-2 7B shape on one MI355X, through the engine's own
scheduler, step function, cache and kernels.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--layers L] [--dtype bfloat16]

A step is one decode step of the whole batch. Prints ONE JSON line: the decode rate at the
default batch, the prefill rate of a 2,048-token prompt with its fraction of the MFMA peak, the
decode step's fraction of the HBM roofline, and the decode rates at batch 1 and 64.
Weights are random (N(0, 0.02), drawn on the GPU), token ids are seeded uniform-random: synthetic data.
"""
import argparse
import json
import os
import sys
import time

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

# MI355X published peaks
HBM_BYTES_PER_S = 8.0e12
PEAK_FLOPS = {"bfloat16": 2.5e15, "float32": 157.3e12}


GENERATED = 256  # the benchmark's requests generate this many tokens after their prompt


def load_baseline_config():
    """Layer sizes of the reference's gpt2_7b configuration (config/gpt2_7b.yaml) with GPT-2's vocabulary."""
    return {"model_type": "gpt2", "n_layer": 32, "n_embd": 4096, "n_head": 32, "n_inner": 16384, "vocab_size": 50257,
            "n_positions": 2048, "layer_norm_epsilon": 1e-5, "activation_function": "gelu_new"}


# the other sizes of the reference's configurations (config/gpt2_xl.yaml, config/gpt2_20b.yaml), for --shape
OTHER_SHAPES = {
    "xl": {"model_type": "gpt2", "n_layer": 48, "n_embd": 1600, "n_head": 25, "n_inner": 6400, "vocab_size": 50257,
           "n_positions": 1024, "layer_norm_epsilon": 1e-5, "activation_function": "gelu_new"},
    "20b": {"model_type": "gpt2", "n_layer": 44, "n_embd": 6144, "n_head": 64, "n_inner": 24576, "vocab_size": 50257,
            "n_positions": 2048, "layer_norm_epsilon": 1e-5, "activation_function": "gelu_new"},
}


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=256)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--prompt-len", type=int, default=512)
    ap.add_argument("--layers", type=int, default=None, help="fewer layers than the configuration has (both numbers are reported)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--no-points", action="store_true", help="skip the batch 1 / 64 points and the prefill")
    ap.add_argument("--prefill-only", action="store_true", help="time the 2,048-token prefill alone (for profiling); prints its own line")
    ap.add_argument("--prefill-len", type=int, default=2048, help="with --prefill-only: tokens of the prompt (the headline point is 2,048)")
    ap.add_argument("--shape", default="7b", choices=["7b", "xl", "20b"],
                    help="layer sizes of the decode workload: 7b is the headline's; xl and 20b measure the same step at the other "
                         "sizes of the reference's configurations (use --no-points: the prefill point is 2,048 tokens)")
    ap.add_argument("--workload", default="decode", choices=["decode", "xl_mix", "20b", "zederax", "nakurax", "tativik", "kegetar", "lelatar", "kelasun"],
                    help="decode: the workload described above. xl_mix / 20b: continuous-batching workloads at the gpt2_xl and gpt2_20b sizes "
                         "through InferenceEngine.generate; they print their own line. zederax: prefill and decode rates of Zederax "
                         "layers at a few sizes beside GPT-2 layers of the same width, heads and inner width; its own line. nakurax: the same for "
                         "Nakurax layers (latent attention and attention beside a recurrence, in turn) beside Zederax and GPT-2 layers. tativik: Tativik "
                         "layers (windowed latent attention with a rotated key part and a generalized delta rule, in turn, routed experts) beside Nakurax layers. "
                         "kegetar: Kegetar layers (windowed attention that keeps the first positions beside gated linear attention, and attention whose "
                         "keys are its values, in turn; dense and routed feed-forwards in turn) beside Tativik layers. lelatar: Lelatar layers (attention with sinks "
                         "beside a gated delta rule with a dense feed-forward, and state-space duality, in turn, two layers looped, a token input a layer) beside "
                         "Kegetar layers. kelasun: Kelasun layers (attention with a distance term and sinks, and latent attention with a rotated key "
                         "part, in turn, routed experts without gates beside a shared one, a norm behind every sum) beside Tativik and Kegetar layers")
    ap.add_argument("--sizes", default="1k,2k,4k", help="with --workload zederax / nakurax: which of the sizes 1k, 2k, 4k to run")
    ap.add_argument("--batches", default="1,8,64", help="with --workload zederax: decode batch sizes to time ('' for none)")
    ap.add_argument("--no-prefill", action="store_true", help="with --workload zederax: skip the 2,048-token prompt")
    ap.add_argument("--arch", default="both", choices=["both", "zederax", "gpt2", "nakurax", "tativik", "kegetar", "lelatar", "kelasun"],
                    help="with --workload zederax / nakurax: one architecture only (for profiling)")
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported")
        return 2

    import torch

    from levanter_amd.config import InferenceEngineConfig, LmConfig
    from levanter_amd.engine import InferenceEngine, Request

    if args.workload in ("zederax", "nakurax", "tativik", "kegetar", "lelatar", "kelasun"):
        return zederax_workload(args)
    if args.workload != "decode":
        return serving_workload(args)

    raw = load_baseline_config() if args.shape == "7b" else dict(OTHER_SHAPES[args.shape])
    shape_name = {"7b": "GPT-2 7B", "xl": "GPT-2 XL", "20b": "GPT-2 20B"}[args.shape]
    full_layers = raw["n_layer"]
    if args.layers is not None:
        raw["n_layer"] = args.layers
    cfg = LmConfig.from_dict(raw)
    ps = 16
    max_batch = max(args.batch, 1 if args.no_points else 64)
    # Requests whose prompts are done first decode beside the prompt portions of the others: `early` tokens at most
    # before the timed steps begin. Nobody may end, and no page may be missing, before the last timed step.
    early = (max_batch * args.prompt_len + 2047) // 2048 + 8
    # The timed steps lie in the middle of the GENERATED tokens that follow the prompt, however few they are: their mean
    # context is prompt_len + GENERATED / 2 (untimed steps lead up to them).
    span = max(args.steps, GENERATED)
    ctx_end = args.prompt_len + early + args.warmup + span + 1
    if ctx_end > cfg.n_positions:
        print(f"bench.py: prompt {args.prompt_len} + {early + args.warmup + span + 1} steps exceed n_positions {cfg.n_positions}")
        return 2
    pages_per_seq = (max(ctx_end, 2048) + ps - 1) // ps
    ecfg = InferenceEngineConfig(max_pages=max_batch * ((ctx_end + ps - 1) // ps) + pages_per_seq, max_seqs=max_batch, page_size=ps,
                                 max_pages_per_seq=pages_per_seq, compute_dtype=args.dtype, max_prefill_size=2048,
                                 max_seqs_in_prefill=max_batch)
    t0 = time.time()
    engine = InferenceEngine.from_config(cfg, seed=0, config=ecfg)
    torch.cuda.synchronize()
    print(f"[bench] model ready in {time.time() - t0:.1f}s: {engine.model.weight_bytes() / 1e9:.2f} GB of weights", file=sys.stderr, flush=True)

    itemsize = 2 if args.dtype == "bfloat16" else 4
    L, D, F, V = cfg.n_layer, cfg.n_embd, cfg.inner_dim, cfg.vocab_size
    matrix_params = L * (3 * D * D + D * D + 2 * D * F)
    weight_bytes = (matrix_params + V * D) * itemsize + L * (3 * D + D + F + D + 4 * D) * 4 + 2 * D * 4
    kv_bytes_per_token = 2 * L * D * itemsize

    def prompts(batch, n, seed):
        g = torch.Generator().manual_seed(seed)
        return [torch.randint(0, V, (n,), generator=g).tolist() for _ in range(batch)]

    def decode_run(batch, steps, warmup, seed):
        """Prefill ``batch`` prompts, then time ``steps`` decode steps. Returns (seconds, mean context)."""
        engine.reset()
        reqs = [Request(prompt_tokens=p, request_id=i, max_new_tokens=early + warmup + max(steps, GENERATED) + 8, temperature=0.0)
                for i, p in enumerate(prompts(batch, args.prompt_len, seed))]
        seqs = engine.enqueue_requests(reqs)
        while any(s.n_cached < s.prompt_len for s in seqs) or any(not s.generated for s in seqs):
            engine.step()
        for _ in range(warmup):
            engine.step()
        ctx_now = sum(s.n_cached for s in seqs) / len(seqs)
        for _ in range(max(0, int(args.prompt_len + GENERATED / 2.0 - (steps + 1) / 2.0 - ctx_now))):
            engine.step()
        torch.cuda.synchronize()
        ctx0 = sum(s.n_cached for s in seqs) / len(seqs)
        before = dict(engine.stats)
        ev0, ev1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        t = time.perf_counter()
        ev0.record()
        for _ in range(steps):
            engine.step()
        ev1.record()
        torch.cuda.synchronize()
        dt = time.perf_counter() - t
        assert all(len(s.generated) >= warmup + steps and not s.done for s in seqs), "the timed steps did not all decode the whole batch"
        ctx_mean = ctx0 + (steps + 1) / 2.0
        # the device's own clock around the same steps, and the host's share of a step: what step() takes less the time it waits
        # for the device (src/levanter/inference/engine.py:1146-1159 logs the same split per iteration)
        timing = {"device_ms_per_step": round(ev0.elapsed_time(ev1) / steps, 4),
                  "host_ms_per_step": round(((engine.stats["step_s"] - before["step_s"]) - (engine.stats["wait_s"] - before["wait_s"])) / steps * 1e3, 4)}
        engine.reset()
        return dt, ctx_mean, timing

    def prefill_run(T, reps):
        """One prompt of T tokens in one step, ``reps`` times after one untimed run: the median, with the fastest and slowest."""
        times = []
        for rep in range(reps + 1):
            engine.reset()
            engine.enqueue_requests([Request(prompt_tokens=prompts(1, T, 50 + rep)[0], request_id=rep, max_new_tokens=1)])
            torch.cuda.synchronize()
            t = time.perf_counter()
            engine.step()
            torch.cuda.synchronize()
            if rep > 0:
                times.append(time.perf_counter() - t)
        times.sort()
        mid = times[len(times) // 2]
        flops = 2.0 * T * matrix_params + 2.0 * T * T * D * L + 2.0 * D * V
        return {"value": round(T / mid, 1), "tokens": T, "ms": round(mid * 1e3, 3), "frac": round(flops / mid / PEAK_FLOPS[args.dtype], 4),
                "ms_min": round(times[0] * 1e3, 3), "ms_max": round(times[-1] * 1e3, 3), "reps": reps}

    if args.prefill_only:
        if not 1 <= args.prefill_len < cfg.n_positions + 1:
            print(f"bench.py: --prefill-len {args.prefill_len} does not fit n_positions {cfg.n_positions}")
            return 2
        print(json.dumps({"prefill": prefill_run(args.prefill_len, 4), "model": f"gpt2_{args.shape} shape"}), flush=True)
        return 0

    dt, ctx_mean, timing = decode_run(args.batch, args.steps, args.warmup, seed=1)
    ms_per_step = dt / args.steps * 1e3
    value = args.batch * args.steps / dt
    step_bytes = weight_bytes + args.batch * ctx_mean * kv_bytes_per_token
    achieved = step_bytes / (dt / args.steps) / 1e9
    out = {
        "metric": (f"decode tok/s @ batch 8, {shape_name} shape, bf16" if args.batch == 8 and args.dtype == "bfloat16"
                   else f"decode tok/s @ batch {args.batch}, {shape_name} shape"),
        "value": round(value, 2), "unit": "tok/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(ms_per_step, 4), **timing, "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "data": "synthetic (random weights N(0,0.02), uniform-random token ids)",
        "config": {"model": f"gpt2_{args.shape} shape", "n_layer": L, "n_layer_full": full_layers, "n_embd": D, "n_head": cfg.n_head,
                   "head_dim": cfg.head_dim, "n_inner": F, "vocab_size": V, "n_positions": cfg.n_positions,
                   "global_batch": args.batch, "seq_len": args.prompt_len + GENERATED, "prompt_len": args.prompt_len,
                   "generated": GENERATED, "ctx_mean": round(ctx_mean, 1), "page_size": ps, "parallelism": "single GPU"},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_BYTES_PER_S / 1e9, "unit": "GB/s",
                     "frac": round(achieved / (HBM_BYTES_PER_S / 1e9), 4)},
    }
    if not args.no_points:
        # prefill of one 2,048-token prompt in one step (the logits of its last token)
        out["prefill"] = prefill_run(2048, 5)
        points = {}
        for b, steps in ((1, min(args.steps, 128)), (64, min(args.steps, 64))):
            d, _, _ = decode_run(b, steps, min(args.warmup, 4), seed=2 + b)
            points[f"decode_b{b}"] = round(b * steps / d, 2)
        # the same prefill with every matrix product on this repository's own kernels (none left to the vendor library)
        kernels = engine.env.kernels
        was, kernels.gemm_library = kernels.gemm_library, False
        try:
            points["prefill_own_kernels"] = prefill_run(2048, 3)["value"]
        finally:
            kernels.gemm_library = was
        out["points"] = points
    print(json.dumps(out), flush=True)
    return 0


def serving_workload(args) -> int:
    """End-to-end generation through the scheduler: requests are admitted, their prompts cut into portions under the
    token budget beside the decoding requests, until every request has its tokens. One JSON line."""
    import torch

    from levanter_amd.config import InferenceEngineConfig, LmConfig
    from levanter_amd.engine import InferenceEngine, Request

    ps = 16
    if args.workload == "xl_mix":  # gpt2_xl sizes (config/gpt2_xl.yaml), 64 requests, prompts U[16, 768], 128 new tokens, portions of 256
        raw = {"model_type": "gpt2", "n_layer": 48, "n_embd": 1600, "n_head": 25, "n_inner": 6400, "vocab_size": 50257,
               "n_positions": 1024, "layer_norm_epsilon": 1e-5, "activation_function": "gelu_new"}
        n_req, new_tokens, temperature, chunk = 64, 128, 0.0, 256
        g = torch.Generator().manual_seed(3)
        lens = torch.randint(16, 769, (n_req,), generator=g).tolist()
        name = "gpt2_xl shape, 64 requests, prompts U[16,768], 128 new tokens, portions of 256"
    else:  # gpt2_20b sizes (config/gpt2_20b.yaml), 32 requests x 1024-token prompts, 512 tokens each at temperature 1.0
        raw = {"model_type": "gpt2", "n_layer": 44, "n_embd": 6144, "n_head": 64, "n_inner": 24576, "vocab_size": 50257,
               "n_positions": 2048, "layer_norm_epsilon": 1e-5, "activation_function": "gelu_new"}
        n_req, new_tokens, temperature, chunk = 32, 512, 1.0, 2048
        lens = [1024] * n_req
        name = "gpt2_20b shape, 32 requests x 1024-token prompts, 512 new tokens at temperature 1.0"
    full_layers = raw["n_layer"]
    if args.layers is not None:
        raw["n_layer"] = args.layers
    cfg = LmConfig.from_dict(raw)
    V = cfg.vocab_size
    pages_per_seq = (max(lens) + new_tokens + ps) // ps
    itemsize = 2 if args.dtype == "bfloat16" else 4
    # 20b: the engine sizes the cache itself from what the weights leave of the memory (at most every request at full length)
    ecfg = InferenceEngineConfig(max_pages="auto" if args.workload == "20b" else n_req * pages_per_seq, cache_memory_reserve_gib=24.0,
                                 max_seqs=n_req, page_size=ps, max_pages_per_seq=pages_per_seq,
                                 compute_dtype=args.dtype, max_prefill_size=chunk, max_seqs_in_prefill=n_req, seed=0)
    t0 = time.time()
    engine = InferenceEngine.from_config(cfg, seed=0, config=ecfg)
    torch.cuda.synchronize()
    max_pages = max((g.pool.n_pages for g in engine.cache.groups), default=0)
    print(f"[bench] model ready in {time.time() - t0:.1f}s: {engine.model.weight_bytes() / 1e9:.2f} GB of weights, "
          f"{max_pages} pages of {ps} tokens", file=sys.stderr, flush=True)

    def requests(seed):
        g = torch.Generator().manual_seed(seed)
        return [Request(prompt_tokens=torch.randint(0, V, (n,), generator=g).tolist(), request_id=i, max_new_tokens=new_tokens,
                        temperature=temperature) for i, n in enumerate(lens)]

    # a short run first: kernels and the GEMM library are loaded (prompt portions of the workload's size among them) and
    # the decode shapes have been seen once
    warm = [Request(prompt_tokens=r.prompt_tokens[:chunk if i < 2 else 32], request_id=r.request_id, max_new_tokens=4, temperature=temperature)
            for i, r in enumerate(requests(1)[:4])]
    engine.generate(warm)
    engine.reset()
    engine.warm_up()
    step_ms = []
    print("[bench] warm-up done, the timed run starts", file=sys.stderr, flush=True)
    seqs = engine.enqueue_requests(requests(2))
    torch.cuda.synchronize()
    before = dict(engine.stats)
    t = time.perf_counter()
    while not all(s.done for s in seqs):
        t1 = time.perf_counter()
        engine.step()
        step_ms.append((time.perf_counter() - t1) * 1e3)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t
    generated = sum(len(s.generated) for s in seqs)
    prompt_tokens = sum(lens)
    slowest = max(range(len(step_ms)), key=step_ms.__getitem__)
    print(f"[bench] {len(step_ms)} steps; the slowest was step {slowest} ({step_ms[slowest]:.1f} ms)", file=sys.stderr, flush=True)
    step_ms.sort()
    pick = lambda q: round(step_ms[min(len(step_ms) - 1, int(q * len(step_ms)))], 3)
    out = {
        "metric": f"end-to-end generated tok/s, {name}", "value": round(generated / dt, 2), "unit": "tok/s", "n_gpus": 1,
        "steps": len(step_ms), "warmup": 0, "ms_per_step": round(dt / len(step_ms) * 1e3, 4),
        "host_ms_per_step": round(((engine.stats["step_s"] - before["step_s"]) - (engine.stats["wait_s"] - before["wait_s"])) / len(step_ms) * 1e3, 4),
        "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
        "data": "synthetic (random weights N(0,0.02), uniform-random token ids)",
        "config": {"model": args.workload, "n_layer": cfg.n_layer, "n_layer_full": full_layers, "n_embd": cfg.n_embd, "n_head": cfg.n_head,
                   "head_dim": cfg.head_dim, "n_inner": cfg.inner_dim, "vocab_size": V, "n_positions": cfg.n_positions,
                   "global_batch": n_req, "prompt_tokens": prompt_tokens, "new_tokens": new_tokens, "prefill_chunk": chunk,
                   "page_size": ps, "max_pages": max_pages, "temperature": temperature, "parallelism": "single GPU"},
        "seconds": round(dt, 3), "generated": generated, "all_tokens_per_s": round((generated + prompt_tokens) / dt, 1),
        "step_ms": {"p10": pick(0.1), "p50": pick(0.5), "p90": pick(0.9), "p99": pick(0.99), "max": round(step_ms[-1], 3)},
        "preemptions": engine.scheduler.n_preemptions,
    }
    print(json.dumps(out), flush=True)
    return 0


# Zederax layers at sizes that resemble real models' (width, query heads, key/value heads, key and value head size, inner
# width, layers, window), and GPT-2 layers of the same width, heads and inner width beside them
ZEDERAX_SIZES = {
    "1k": dict(width=1024, heads=16, kv_heads=4, dim=64, vdim=64, ff=4096, layers=8, window=1024),
    "2k": dict(width=2048, heads=16, kv_heads=4, dim=128, vdim=64, ff=8192, layers=8, window=1024),
    "4k": dict(width=4096, heads=32, kv_heads=8, dim=128, vdim=128, ff=16384, layers=4, window=2048),
}
ZEDERAX_VOCAB = 32000


def zederax_config(z):
    import math

    mixer = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["vdim"], "scale": 1.0 / math.sqrt(z["dim"]) * 4.0,
             "softcap": 30.0, "mask": {"size": z["window"]}, "v_mix": True}
    return {"architecture": "Zederax", "vocab": ZEDERAX_VOCAB, "width": z["width"], "norm": {"eps": 1e-6},
            "layers": [{"type": "attention", "mixer": dict(mixer), "mlp": {"kind": "dense", "ff": z["ff"]}} for _ in range(z["layers"])]}


def gpt2_config_like(z):
    return {"model_type": "gpt2", "n_layer": z["layers"], "n_embd": z["width"], "n_head": z["heads"], "n_inner": z["ff"],
            "vocab_size": ZEDERAX_VOCAB, "n_positions": 4096, "layer_norm_epsilon": 1e-5, "activation_function": "gelu_new"}


def nakurax_config(z):
    """Latent-attention layers and layers of a chunked rotary attention beside a gated recurrence, in turn, on four residual
    streams: the heads, head sizes, inner width and layer count of the size, the chunk as long as its window, a latent of
    two key heads' size (at most 256), a recurrence as wide as the model with a block per head."""
    import math

    latent = {"heads": z["heads"], "dim": z["dim"], "vdim": z["vdim"], "kv_rank": min(256, 2 * z["dim"]), "scale": 1.0 / math.sqrt(z["dim"])}
    left = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["vdim"], "scale": 1.0 / math.sqrt(z["dim"]),
            "mask": {"size": z["window"]}, "rot": {"dims": z["dim"] // 2, "base": 500000.0,
                                                   "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    parallel = {"left": left, "right": {"width": z["width"], "blocks": z["heads"], "conv": 4}, "left_scale": 0.7, "right_scale": 0.7}
    mlp = {"kind": "dense", "ff": z["ff"]}
    layers = [{"type": "latent_attention", "mixer": dict(latent), "mlp": dict(mlp)} if i % 2 == 0 else
              {"type": "parallel", "mixer": json.loads(json.dumps(parallel)), "mlp": dict(mlp)} for i in range(z["layers"])]
    return {"architecture": "Nakurax", "vocab": ZEDERAX_VOCAB, "width": z["width"], "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "streams": 4, "layers": layers}


def tativik_config(z):
    """Latent-attention layers (queries through a latent, a rotated key part of 32, a window, sinks, gates) and layers of the
    generalized delta rule, in turn, every sublayer between two norms in two groups and behind a gate; the heads, head sizes and
    layer count of the size, a latent of three key heads' size (at most 224, so that latent and rotated part fill a key of 256).
    The feed-forward has 32 experts of a quarter of the size's inner width in 8 groups of which 4 are kept, 4 experts a token:
    a token's experts hold as much as the size's dense feed-forward."""
    import math

    rot = 32
    latent = {"heads": z["heads"], "dim": z["dim"], "rot_dim": rot, "vdim": z["vdim"], "kv_rank": min(224, 3 * z["dim"]), "q_rank": z["width"] // 2,
              "scale": 1.0 / math.sqrt(z["dim"] + rot), "rot": {"dims": rot, "base": 500000.0}, "mask": {"size": z["window"]}}
    delta = {"heads": z["width"] // z["dim"], "dim": z["dim"], "decay_rank": 64}
    mlp = {"kind": "moe", "expert": {"ff": z["ff"] // 4}, "router": {"experts": 32, "top": 4, "groups": {"count": 8, "keep": 4}}}
    layers = [{"type": "latent_attention" if i % 2 == 0 else "general_delta", "mixer": dict(latent if i % 2 == 0 else delta), "mlp": json.loads(json.dumps(mlp))}
              for i in range(z["layers"])]
    return {"architecture": "Tativik", "vocab": ZEDERAX_VOCAB, "width": z["width"], "norm": {"eps": 1e-6, "groups": 2}, "residual_mult": 0.7, "layers": layers}


def kegetar_config(z):
    """Layers of a windowed rotary attention (the first 64 positions stay in sight, stretched frequencies, a gate per element) beside a
    gated linear attention with heads of the size's key and value sizes, and layers of an attention whose keys are its values with a
    distance term, in turn; the heads, head sizes, window and layer count of the size. The feed-forwards are in turn a dense gated one
    of two thirds of the size's inner width (three matrices hold what the size's two hold) and 30 experts of a quarter of that width
    beside 2 router outputs that return their input, in 8 groups of which 4 are kept, 4 a token, and a shared expert of the same width."""
    import math

    left = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["vdim"], "scale": 1.0 / math.sqrt(z["dim"]),
            "mask": {"size": z["window"], "keep_first": 64},
            "rot": {"dims": z["dim"], "base": 500000.0, "scaling": {"factor": 8.0, "original": 4096, "fast": 16.0, "slow": 2.0}}}
    right = {"heads": z["heads"], "dim": z["dim"], "vdim": z["vdim"], "tau": 8.0, "decay_rank": 64}
    attention = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["dim"], "scale": 1.0 / math.sqrt(z["dim"]), "mask": {"size": z["window"]}}
    dense = {"kind": "dense", "ff": z["ff"] * 2 // 3 // 256 * 256}
    moe = {"kind": "moe", "expert": {"ff": z["ff"] // 4, "limit": 7.0}, "router": {"experts": 30, "identity": 2, "top": 4, "groups": {"count": 8, "keep": 4}},
           "shared": {"ff": z["ff"] // 4, "limit": 7.0}}
    layers = []
    for i in range(z["layers"]):
        mixer = {"type": "parallel", "mixer": {"left": left, "right": right}} if i % 4 < 2 else {"type": "attention", "mixer": attention}
        layers.append(json.loads(json.dumps({**mixer, "mlp": dense if i % 2 == 0 else moe})))
    return {"architecture": "Kegetar", "vocab": ZEDERAX_VOCAB, "width": z["width"], "norm": {"eps": 1e-6}, "residual_mult": 0.5,
            "embedding": {"bigram": {"buckets": 65521, "mul_prev": 1009, "mul_cur": 13}}, "layers": layers}


def lelatar_config(z):
    """Layers of a causal rotary attention with sinks beside a gated delta rule, with a dense gated feed-forward of two thirds of the size's
    inner width (three matrices hold what the size's two hold), and layers of state-space duality (twice the width inside, heads of 64
    over a state of 128, no feed-forward), in turn; the heads and head sizes of the size. Two layers in the middle run twice, so that the
    layer runs are the size's layer count; every layer ends with a token input of a 16th of the width."""
    import math

    left = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["vdim"], "scale": 1.0 / math.sqrt(z["dim"]),
            "rot": {"dims": z["dim"] // 2, "base": 500000.0}}
    right = {"heads": z["heads"], "kv_heads": z["heads"] // 2, "dim": z["dim"], "vdim": z["vdim"], "conv": 4}
    mamba = {"heads": z["width"] // 32, "vdim": 64, "state": 128, "groups": 4, "norm_groups": 4, "conv": 4}
    n = z["layers"] - 2
    layers = [{"type": "parallel", "mixer": json.loads(json.dumps({"left": left, "right": right})), "mlp": {"kind": "dense", "ff": z["ff"] * 2 // 3 // 256 * 256}}
              if i % 2 == 0 else {"type": "mamba2", "mixer": dict(mamba), "mlp": None} for i in range(n)]
    start = max(0, n // 2 - 1)
    return {"architecture": "Lelatar", "vocab": ZEDERAX_VOCAB, "width": z["width"], "norm": {"eps": 1e-6}, "layers": layers,
            "loop": {"start": start, "stop": start + 2, "times": 2}, "token_side": {"dim": z["width"] // 16}}


def kelasun_config(z):
    """Layers of attention with a distance term, sinks and a temperature and layers of latent attention (queries through a latent, a rotated
    key part of 32 with stretched frequencies, a gate per element), in turn; the heads, head sizes and layer count of the size, the latents
    of Tativik's layers above (three key heads' size, at most 224; half the width for the queries). The feed-forward has 32 experts of a
    quarter of the size's inner width, 4 a token, and a shared one of the same width."""
    import math

    rot = 32
    attention = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["vdim"], "scale": 1.0 / math.sqrt(z["dim"]), "q_temp": {"coef": 0.1, "every": 2048}}
    latent = {"heads": z["heads"], "dim": z["dim"], "rot_dim": rot, "vdim": z["vdim"], "kv_rank": min(224, 3 * z["dim"]), "q_rank": z["width"] // 2,
              "scale": 1.0 / math.sqrt(z["dim"] + rot),
              "rot": {"dims": rot, "base": 500000.0, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    mlp = {"kind": "moe", "expert": {"ff": z["ff"] // 4}, "router": {"experts": 32, "top": 4}, "shared": {"ff": z["ff"] // 4}}
    layers = [json.loads(json.dumps({"type": "attention" if i % 2 == 0 else "latent_attention", "mixer": attention if i % 2 == 0 else latent, "mlp": mlp}))
              for i in range(z["layers"])]
    return {"architecture": "Kelasun", "vocab": ZEDERAX_VOCAB, "width": z["width"], "norm": {"eps": 1e-6}, "postln_alpha": 2.0, "logit_scale": 0.5, "layers": layers}


def zederax_workload(args) -> int:
    """Prefill (one 2,048-token prompt) and decode (batch 1, 8, 64 after 512-token prompts) through the engine, for Zederax
    (or, with --workload nakurax, Nakurax and Zederax) and for GPT-2 at equal sizes. One JSON line."""
    import torch

    from levanter_amd.config import InferenceEngineConfig, LmConfig
    from levanter_amd.engine import InferenceEngine, Request

    ps, prompt_len, V = 16, 512, ZEDERAX_VOCAB
    steps, warmup = min(args.steps, 128), args.warmup
    batches = tuple(int(b) for b in args.batches.split(",") if b)
    ctx_end = prompt_len + 64 + warmup + steps + 16
    pages_per_seq = (max(ctx_end, 2048) + ps - 1) // ps

    def prompts(batch, n, seed):
        g = torch.Generator().manual_seed(seed)
        return [torch.randint(0, V, (n,), generator=g).tolist() for _ in range(batch)]

    def measure(raw):
        most = max(batches, default=1)
        ecfg = InferenceEngineConfig(max_pages=most * ((ctx_end + ps - 1) // ps) + pages_per_seq, max_seqs=most, page_size=ps,
                                     max_pages_per_seq=pages_per_seq, compute_dtype=args.dtype, max_prefill_size=2048,
                                     max_seqs_in_prefill=most)
        engine = InferenceEngine.from_config(LmConfig.from_dict(raw), seed=0, config=ecfg)
        out = {"weights_gb": round(engine.model.weight_bytes() / 1e9, 3)}
        times = []
        for rep in range(0 if args.no_prefill else 4):
            engine.reset()
            engine.enqueue_requests([Request(prompt_tokens=prompts(1, 2048, 50 + rep)[0], request_id=rep, max_new_tokens=1)])
            torch.cuda.synchronize()
            t = time.perf_counter()
            engine.step()
            torch.cuda.synchronize()
            if rep > 0:
                times.append(time.perf_counter() - t)
        if times:
            out["prefill_2048_tok_s"] = round(2048 / sorted(times)[len(times) // 2], 1)
            out["prefill_2048_ms"] = round(sorted(times)[len(times) // 2] * 1e3, 3)
        for b in batches:
            engine.reset()
            reqs = [Request(prompt_tokens=p, request_id=i, max_new_tokens=64 + warmup + steps + 8, temperature=0.0)
                    for i, p in enumerate(prompts(b, prompt_len, b))]
            seqs = engine.enqueue_requests(reqs)
            while any(s.n_cached < s.prompt_len for s in seqs) or any(not s.generated for s in seqs):
                engine.step()
            for _ in range(warmup):
                engine.step()
            torch.cuda.synchronize()
            t = time.perf_counter()
            for _ in range(steps):
                engine.step()
            torch.cuda.synchronize()
            dt = time.perf_counter() - t
            assert all(not s.done for s in seqs)
            out[f"decode_b{b}_tok_s"] = round(b * steps / dt, 1)
            out[f"decode_b{b}_ms_per_step"] = round(dt / steps * 1e3, 4)
        engine.reset()
        del engine
        torch.cuda.empty_cache()
        return out

    results = {}
    for name in args.sizes.split(","):
        if name not in ZEDERAX_SIZES:
            print(f"bench.py: unknown size {name!r}; known: {', '.join(ZEDERAX_SIZES)}")
            return 2
        z = ZEDERAX_SIZES[name]
        results[name] = {"sizes": z}
        archs = [("zederax", zederax_config(z)), ("gpt2", gpt2_config_like(z))]
        if args.workload == "nakurax":
            archs.insert(0, ("nakurax", nakurax_config(z)))
        if args.workload == "tativik":  # beside the closest model: Nakurax's latent attention and recurrence
            archs = [("tativik", tativik_config(z)), ("nakurax", nakurax_config(z))]
        if args.workload == "kegetar":  # beside the closest model: Tativik's windowed attention, matrix-state recurrence and experts
            archs = [("kegetar", kegetar_config(z)), ("tativik", tativik_config(z))]
        if args.workload == "lelatar":  # beside the closest model: Kegetar's attention beside a recurrence with a matrix state, gated feed-forwards
            archs = [("lelatar", lelatar_config(z)), ("kegetar", kegetar_config(z))]
        if args.workload == "kelasun":  # beside the closest models: Tativik's latent attention and experts, Kegetar's attention with a distance term
            archs = [("kelasun", kelasun_config(z)), ("tativik", tativik_config(z)), ("kegetar", kegetar_config(z))]
        for arch, raw in archs:
            if args.arch in ("both", arch):
                print(f"[bench] {arch} at size {name} ...", file=sys.stderr, flush=True)
                results[name][arch] = measure(raw)
    print(json.dumps({"metric": ("prefill and decode tok/s of Kelasun layers beside Tativik and Kegetar layers of equal width, heads and head sizes" if args.workload == "kelasun" else
                                 "prefill and decode tok/s of Lelatar layers beside Kegetar layers of equal width, heads and head sizes" if args.workload == "lelatar" else
                                 "prefill and decode tok/s of Kegetar layers beside Tativik layers of equal width, heads and head sizes" if args.workload == "kegetar" else
                                 f"prefill and decode tok/s of Tativik layers beside Nakurax layers of equal width, heads and (per token) inner width" if args.workload == "tativik" else
                                 f"prefill and decode tok/s of {args.workload.capitalize()} layers beside {'Zederax and ' if args.workload == 'nakurax' else ''}GPT-2 layers of equal width, heads and inner width"),
                      "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warmup, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                      "data": "synthetic (random weights, uniform-random token ids)", "results": results}), flush=True)  # noqa: E501
    return 0


if __name__ == "__main__":
    sys.exit(main())
