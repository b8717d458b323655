#!/usr/bin/env python3
"""Decode and prefill throughput of the engine on one MI355X, Llama-3.1-8B shape, bfloat16,
random weights, synthetic token ids.

    python bench.py --gpus 1 --steps K --warmup W

A "step" is one decode step of the whole batch (default 8 requests).  The timed steps are centred on a cache
length of 3,072 tokens, the middle of the named sweep from 2,048 to 4,096: the default 2,000 steps cover the
sweep itself (prompts of 2,048 tokens), a short run (`--steps 20`) starts from prompts of about 3,050 tokens and
times the steps around 3,072, so that a step reads what a step of the sweep reads on average; `metric` names
the range that was timed.  The headline runs through the engine's own entry point: `Engine.add_request` and
`Engine.step`, with its scheduler, step function and sampler (greedy), as `tempura run` does.  Prints ONE
JSON line: decoded tokens per second (`value`), the step's share of the HBM roofline, the 2,048-token
prefill, and under `points`: batch 1 and 64 through the engine, the same three batches through the bare
step function (`runner_b*`: no scheduler, no sampler object), longer prefills, decoding at a 32 k context,
and the mixed serving workload (64 requests, prompts of 128..2,048 tokens in portions of 512 beside running
decodes, 256 output tokens each, Llama-3.2-3B shape) whose details are under `mixed`.
The reference measures prefill and single-token forwards its own way, with percentiles and a fingerprint of
the logits for run-to-run determinism (/root/reference/tools/bench-gpu/src/bench_real_model.rs:160-278);
its serving loop is /root/reference/server/src/engine_task.rs:581-875.
"""
from __future__ import annotations

import argparse
import json
import random
import sys
import time

HBM_PEAK_GBS = 8000.0                                   # MI355X HBM3E, published
MFMA_PEAK = {"bf16": 2.5e15, "fp16": 2.5e15, "fp8": 5.0e15, "fp32": 157.3e12}   # dense, published


def parse_args():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=2000, help="timed decode steps")
    ap.add_argument("--warmup", type=int, default=16, help="untimed decode steps")
    ap.add_argument("--model-config", default="llama-3.1-8b")
    ap.add_argument("--layers", type=int, default=None, help="run fewer layers than the configuration has")
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--prompt-len", type=int, default=2048)
    ap.add_argument("--context", type=int, default=4096)
    ap.add_argument("--page-size", type=int, default=16)
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--no-graph", action="store_true")
    ap.add_argument("--no-chain", action="store_true", help="wait for each step's tokens on the host before queueing the next step")
    ap.add_argument("--no-points", action="store_true", help="only the headline: no other batches, no bare step function")
    ap.add_argument("--no-prefill", action="store_true")
    ap.add_argument("--no-long", action="store_true", help="skip the long prefills and the 32 k decode point")
    ap.add_argument("--no-large-batches", action="store_true", help="skip decoding at batch 128 and 256")
    ap.add_argument("--no-mixed", action="store_true", help="skip the mixed serving workload")
    ap.add_argument("--no-fingerprint", action="store_true", help="skip the run-to-run determinism check")
    ap.add_argument("--point-steps", type=int, default=500, help="timed steps of the other points")
    ap.add_argument("--mixed-config", default="llama-3.2-3b")
    ap.add_argument("--mixed-requests", type=int, default=64)
    ap.add_argument("--mixed-output", type=int, default=256)
    ap.add_argument("--mixed-chunk", type=int, default=512)
    ap.add_argument("--mixed-temperature", type=float, default=0.0, help="0: greedy; above: seeded sampling with top-k 50")
    ap.add_argument("--decode-target-blocks", type=int, default=None, help="tuning: blocks the split decode attention aims at")
    ap.add_argument("--design", default=None, choices=["mifutar", "bomotar", "golavik", "zemarax", "tokatar", "makisun"],
                    help="instead of the headline: prefill and decode throughput of this design at layer sizes of real models, "
                         "beside Llama layers of equal size, with the time of every kernel entry point")
    ap.add_argument("--design-sizes", default="2048,4096", help="model widths of --design (comma separated)")
    ap.add_argument("--design-layers", type=int, default=4, help="layers of each model of --design")
    ap.add_argument("--design-models", default="", help="which models of --design run (comma separated; empty: all)")
    return ap.parse_args()


#: layer sizes of --design by model width: feed-forward width, attention heads x head size, key/value heads
DESIGN_SIZES = {1024: (4096, 16, 64, 4), 2048: (8192, 32, 64, 8), 4096: (14336, 32, 128, 8), 8192: (28672, 64, 128, 8)}


def design_bench(args) -> int:
    """Prefill (one prompt, one step) and decode (a batch, captured steps) of a design and of Llama layers
    of the same width, feed-forward width and attention heads, random weights, bfloat16 unless --dtype says
    otherwise.  A Mifutar model here has three state-space layers to one attention layer (window 1,024, four
    streams); the Llama beside it has the same window.  A Bomotar model here has, in every layer, an attention of the
    Llama layer's heads (values as wide as keys, four taps, YaRN rotation) beside a delta rule of width / 128 heads
    of 128 x 128 (low-rank projections of rank 64), and feed-forwards that alternate between a dense one and eight
    experts of a quarter of its width, two a token out of two of four groups; it stands beside the Mifutar model and
    the Llama layers (no window there).  A Golavik model here has layers of a channel delta rule (width / 128 heads of
    128 x 128, ranks 64), a general delta rule (width / 64 heads of 64), a latent attention of the Llama layer's heads
    (three quarters of a head unrotated, a quarter rotated, values as wide as the whole key, a latent of 512, window
    1,024) and a channel delta rule again, each with eight experts of a quarter of the dense width, two a token out of
    two of four groups, a norm in eight parts and four taps on the inputs; it stands beside the Bomotar model and the
    Llama layers.  A Zemarax model here has layers of an mLSTM (width / 128 heads of 128 x 128), a latent attention of
    the Llama layer's heads (a latent of 128, a query latent of width / 4), a windowed attention of the Llama layer's
    heads with a norm per head (window 1,024 keeping the first 64 tokens) and a latent attention that reads the second
    layer's latents, every attention with a sink; feed-forwards alternate between a dense one and eight ungated experts
    of a quarter of its width, two a token, with a shared expert; it stands beside the Bomotar model (the closest: norms
    around every sublayer, a matrix recurrence, a bigram embedding, routed experts) and the Llama layers.  A Tokatar model
    here has layers of an attention of the Llama layer's heads (chunks of 1,024, scores capped at 30, llama3-scaled
    rotation, gated heads), the same with biases, a norm over the projections, turned values and one added to the
    denominator, a latent attention of the Llama layer's heads (a latent of four heads beside a rotated part of half a head) and
    the first kind again, each with a gate on both sublayers and an ungated feed-forward of the Llama layer's width; it
    stands beside the Zemarax model (the closest: norms around every sublayer, attention over cached latents) and the
    Llama layers.  A Makisun model here has, in turn, layers of a token-shifted recurrence (width / 64 heads of 64, a decay
    of rank 64) and of two mixers side by side: an attention of the Llama layer's heads (a norm per head, window 1,024,
    gated heads) and a gated linear attention of width / 128 heads of 64 x 128 (a decay of rank 64); feed-forwards
    alternate between an ungated dense one and eight ungated experts of a quarter of its width, two a token, with a shared
    expert; it stands beside the Bomotar model (the closest: an attention beside a recurrence, routed experts) and the
    Llama layers.
    Prints one JSON line."""
    import torch
    from tempura_amd.config import BomotarConfig, GolavikConfig, LlamaConfig, MakisunConfig, MifutarConfig, TokatarConfig, ZemaraxConfig
    from tempura_amd.engine import Engine
    from tempura_amd.engine.loading import random_model
    from tempura_amd.engine.runner import StepEntry
    from tempura_amd.kernels import ops

    rng = random.Random(0)
    window, vocab, T, batch = 1024, 32000, args.prompt_len, args.batch
    design = args.design
    points = {}

    def say(msg):
        print(f"[bench] {msg}", file=sys.stderr, flush=True)

    def mifutar_config(width, ff, heads, dim, kv, layers):
        mamba = {"heads": 2 * width // 64, "vdim": 64, "state": 128, "groups": 8, "conv": 4, "norm_groups": 8}
        attn = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "bias_max": 512,
                "bias_buckets": 32, "mask": {"size": window}}
        mlp = {"ff": ff, "kind": "dense", "limit": 7.0}
        ls = [{"type": "attention", "mixer": attn, "mlp": mlp} if i % 4 == 3 else {"type": "mamba2", "mixer": mamba, "mlp": mlp}
              for i in range(layers)]
        return MifutarConfig.from_dict({"architecture": "Mifutar", "vocab": vocab, "width": width, "streams": 4, "logit_scale": 1.0,
                                        "norm": {"eps": 1e-6}, "layers": ls, "max_positions": 8192})

    def bomotar_config(width, ff, heads, dim, kv, layers):
        left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "conv": 4, "scale": dim ** -0.5,
                "rot": {"dims": dim, "base": 1000000.0, "scaling": {"factor": 4.0, "original": 2048, "fast": 16.0, "slow": 2.0}}}
        right = {"heads": width // 128, "kv_heads": width // 128, "dim": 128, "vdim": 128, "conv": 4, "decay_rank": 64, "gate_rank": 64}
        mixer = {"left": left, "right": right, "left_scale": 0.75, "right_scale": 1.1}
        dense = {"kind": "dense", "ff": ff}
        moe = {"kind": "moe", "expert": {"ff": ff // 4}, "router": {"experts": 8, "top": 2, "groups": {"count": 4, "keep": 2}}}
        ls = [{"type": "parallel", "mixer": mixer, "mlp": moe if i % 2 else dense} for i in range(layers)]
        return BomotarConfig.from_dict({"architecture": "Bomotar", "vocab": vocab, "width": width, "residual_mult": 0.8,
                                        "norm": {"eps": 1e-6}, "embedding": {"bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}},
                                        "layers": ls, "max_positions": 8192})

    def golavik_config(width, ff, heads, dim, kv, layers):
        channel = {"heads": width // 128, "kv_heads": width // 128, "dim": 128, "vdim": 128, "conv": 4, "decay_rank": 64, "gate_rank": 64}
        general = {"heads": width // 64, "dim": 64, "decay_rank": 64}
        latent = {"heads": heads, "dim": 3 * dim // 4, "rot_dim": dim // 4, "vdim": dim, "kv_rank": 512, "scale": dim ** -0.5,
                  "mask": {"size": window},
                  "rot": {"dims": dim // 4, "base": 1000000.0, "scaling": {"factor": 4.0, "original": 2048, "fast": 16.0, "slow": 2.0}}}
        moe = {"kind": "moe", "expert": {"ff": ff // 4}, "router": {"experts": 8, "top": 2, "scale": 2.5, "groups": {"count": 4, "keep": 2}}}
        kinds = [("channel_delta", channel), ("general_delta", general), ("latent_attention", latent), ("channel_delta", channel)]
        ls = [{"type": kinds[i % 4][0], "mixer": kinds[i % 4][1], "mlp": moe} for i in range(layers)]
        return GolavikConfig.from_dict({"architecture": "Golavik", "vocab": vocab, "width": width, "norm": {"eps": 1e-6, "groups": 8},
                                        "canon": {"taps": 4}, "layers": ls, "max_positions": 8192})

    def zemarax_config(width, ff, heads, dim, kv, layers):
        mlstm = {"heads": width // 128, "dim": 128, "vdim": 128, "gate_cap": 15.0}
        latent = {"heads": heads, "dim": dim, "vdim": dim, "kv_rank": 128, "q_rank": width // 4, "scale": dim ** -0.5}
        attn = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": window, "keep_first": 64}}
        dense = {"kind": "dense", "ff": ff}
        moe = {"kind": "moe", "expert": {"ff": ff // 4}, "router": {"experts": 8, "top": 2}, "shared": {"ff": ff // 4}}
        ls = []
        for i in range(layers):
            kind = ("mlstm", "latent_attention", "attention", "latent_attention")[i % 4]
            mixer = {"mlstm": mlstm, "attention": attn}.get(kind) or (dict(latent, kv_from=i - 2) if i % 4 == 3 else latent)
            ls.append({"type": kind, "mixer": mixer, "mlp": moe if i % 2 else dense})
        return ZemaraxConfig.from_dict({"architecture": "Zemarax", "vocab": vocab, "width": width, "max_positions": 8192, "logit_scale": 1.0,
                                        "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0, "bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}},
                                        "layers": ls})

    def tokatar_config(width, ff, heads, dim, kv, layers):
        scaling = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}
        attn = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": window}, "softcap": 30.0,
                "rot": {"dims": dim, "base": 500000.0, "scaling": scaling}}
        attn_2 = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": window},
                  "rot": {"dims": dim, "base": 500000.0}}
        latent = {"heads": heads, "dim": dim, "rot_dim": dim // 2, "vdim": dim, "kv_rank": 4 * dim, "scale": (dim + dim // 2) ** -0.5,
                  "rot": {"dims": dim // 2, "base": 500000.0}}
        kinds = [("attention", attn), ("attention_2", attn_2), ("latent_attention", latent), ("attention", attn)]
        ls = [{"type": kinds[i % 4][0], "mixer": kinds[i % 4][1], "mlp": {"kind": "dense", "ff": ff}} for i in range(layers)]
        return TokatarConfig.from_dict({"architecture": "Tokatar", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
                                        "embedding": {"scale": 1.0}, "layers": ls, "max_positions": 8192})

    def makisun_config(width, ff, heads, dim, kv, layers):
        wkv = {"heads": width // 64, "dim": 64, "decay_rank": 64}
        left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": window},
                "rot": {"dims": dim, "base": 500000.0}}
        right = {"heads": width // 128, "dim": 64, "vdim": 128, "tau": 16.0, "decay_rank": 64}
        parallel = {"left": left, "right": right, "left_scale": 0.75, "right_scale": 1.1}
        dense = {"kind": "dense", "ff": ff}
        moe = {"kind": "moe", "expert": {"ff": ff // 4}, "router": {"experts": 8, "top": 2}, "shared": {"ff": ff // 4}}
        kinds = [("wkv", wkv, dense), ("parallel", parallel, moe), ("wkv", wkv, moe), ("parallel", parallel, dense)]
        ls = [{"type": kinds[i % 4][0], "mixer": kinds[i % 4][1], "mlp": kinds[i % 4][2]} for i in range(layers)]
        return MakisunConfig.from_dict({"architecture": "Makisun", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
                                        "embedding": {"scale": 1.0}, "layers": ls, "max_positions": 8192})

    def llama_config(width, ff, heads, dim, kv, layers):
        return LlamaConfig(width, ff, layers, heads, kv, dim, vocab, 8192, 1e-5, 500000.0, None, False,
                           sliding_window=window if design == "mifutar" else None)

    def measure(model):
        pages = (batch + 1) * ((T + 600 + args.page_size - 1) // args.page_size) + 8
        eng = Engine(model, dtype=args.dtype, page_size=args.page_size, kv_pages=pages, max_batch_size=batch + 1,
                     max_num_batched_tokens=max(2048, T), use_graph=not args.no_graph)
        runner = eng.runner
        prompt = lambda n: [rng.randrange(vocab) for _ in range(n)]
        times = []
        for i in range(6):                        # prefill: a fresh request each time, the last four timed
            rid = ("p", i)
            runner.add_request(rid)
            toks = prompt(T)
            torch.cuda.synchronize()
            t = time.perf_counter()
            runner.step([StepEntry(rid, toks, [T - 1])])
            torch.cuda.synchronize()
            if i >= 2:
                times.append(time.perf_counter() - t)
            runner.end_request(rid)
        prefill_ms = 1e3 * sum(times) / len(times)
        rids = [("d", i) for i in range(batch)]
        for rid in rids:
            runner.add_request(rid)
            runner.step([StepEntry(rid, prompt(T), [])])
        lg = runner.step([StepEntry(rid, [1], [0]) for rid in rids])
        n_warm, n_steps = args.warmup, min(args.steps, 400)
        for i in range(n_warm + n_steps):
            if i == n_warm:
                torch.cuda.synchronize()
                t = time.perf_counter()
            toks = ops.argmax(lg).tolist()
            lg = runner.step([StepEntry(rid, [tk], [0]) for rid, tk in zip(rids, toks)])
        torch.cuda.synchronize()
        decode_ms = 1e3 * (time.perf_counter() - t) / n_steps
        for rid in rids:
            runner.end_request(rid)
        rep = eng.profile(prompt_len=T, batch=1, decode_steps=0)
        rep_d = eng.profile(prompt_len=T, batch=batch, decode_steps=4)
        table = lambda rows, div: {name: [calls // div if div > 1 else calls, round(us / div, 1)] for name, calls, us, _ in rows}
        return {"prefill_tokens_per_s": round(T / (prefill_ms / 1e3), 1), "prefill_ms": round(prefill_ms, 3),
                "decode_tokens_per_s": round(batch / (decode_ms / 1e3), 1), "decode_ms_per_step": round(decode_ms, 4),
                "weight_bytes": model.weight_bytes(include_embedding=False),
                "prefill_kernels_us": table(rep["prefill"], 1), "decode_kernels_us_per_step": table(rep_d["decode"], 4)}

    for width in [int(w) for w in args.design_sizes.split(",") if w]:
        if width not in DESIGN_SIZES:
            print(f"--design-sizes: no layer sizes for width {width} (known: {sorted(DESIGN_SIZES)})", file=sys.stderr)
            return 2
        ff, heads, dim, kv = DESIGN_SIZES[width]
        models = [("mifutar", mifutar_config(width, ff, heads, dim, kv, args.design_layers)),
                  ("llama", llama_config(width, ff, heads, dim, kv, args.design_layers))]
        if design == "bomotar":
            models.insert(0, ("bomotar", bomotar_config(width, ff, heads, dim, kv, args.design_layers)))
        if design == "golavik":
            models = [("golavik", golavik_config(width, ff, heads, dim, kv, args.design_layers)),
                      ("bomotar", bomotar_config(width, ff, heads, dim, kv, args.design_layers)), models[1]]
        if design == "zemarax":
            models = [("zemarax", zemarax_config(width, ff, heads, dim, kv, args.design_layers)),
                      ("bomotar", bomotar_config(width, ff, heads, dim, kv, args.design_layers)), models[1]]
        if design == "tokatar":
            models = [("tokatar", tokatar_config(width, ff, heads, dim, kv, args.design_layers)),
                      ("zemarax", zemarax_config(width, ff, heads, dim, kv, args.design_layers)), models[1]]
        if design == "makisun":
            models = [("makisun", makisun_config(width, ff, heads, dim, kv, args.design_layers)),
                      ("bomotar", bomotar_config(width, ff, heads, dim, kv, args.design_layers)), models[1]]
        chosen = [m for m in args.design_models.split(",") if m]
        for name, cfg in [m for m in models if not chosen or m[0] in chosen]:
            say(f"{name} width {width}: building")
            model = random_model(cfg, seed=0, dtype=args.dtype, device="cuda:0")
            points[f"{name}_w{width}"] = measure(model)
            say(f"{name} width {width}: prefill {points[f'{name}_w{width}']['prefill_tokens_per_s']} tok/s, "
                f"decode {points[f'{name}_w{width}']['decode_tokens_per_s']} tok/s")
            del model
            torch.cuda.empty_cache()
    first = next(iter(points))
    print(json.dumps({"metric": f"{design}_prefill_tokens_per_s_T{T}", "value": points[first]["prefill_tokens_per_s"], "unit": "tokens/s",
                      "n_gpus": 1, "higher_is_better": True, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                      "data": "synthetic", "vs_baseline": None,
                      "config": {"design": {"mifutar": "Mifutar beside Llama layers of equal size",
                                            "bomotar": "Bomotar beside Mifutar and Llama layers of equal size",
                                            "golavik": "Golavik beside Bomotar and Llama layers of equal size",
                                            "zemarax": "Zemarax beside Bomotar and Llama layers of equal size",
                                            "tokatar": "Tokatar beside Zemarax and Llama layers of equal size",
                                            "makisun": "Makisun beside Bomotar and Llama layers of equal size"}[design],
                                 "layers": args.design_layers, "prompt": T, "decode_batch": batch,
                                 "window": window if design == "mifutar" else None}, "points": points}))
    return 0


def percentile(xs, p):
    ys = sorted(xs)
    if not ys:
        return 0.0
    k = (len(ys) - 1) * p / 100.0
    lo = int(k)
    hi = min(lo + 1, len(ys) - 1)
    return ys[lo] + (ys[hi] - ys[lo]) * (k - lo)


def main() -> int:
    args = parse_args()
    if args.gpus != 1:
        print(f"bench.py measures one GPU only (this engine has no multi-GPU path); --gpus {args.gpus} is not supported")
        return 2
    if args.design:
        import torch
        if not torch.cuda.is_available():
            print("bench.py needs a GPU", file=sys.stderr)
            return 3
        return design_bench(args)

    import torch
    from tempura_amd.config import PRESETS, LlamaConfig
    from tempura_amd.engine import Engine
    from tempura_amd.engine.loading import random_model
    from tempura_amd.engine.runner import StepEntry
    from tempura_amd.kernels import ops
    from tempura_amd.sampling import SamplingParams

    if not torch.cuda.is_available():
        print("bench.py needs a GPU", file=sys.stderr)
        return 3
    if args.decode_target_blocks:
        ops.decode_target_blocks = args.decode_target_blocks
    elem = 2 if args.dtype == "bfloat16" else 4
    dshort = "bf16" if args.dtype == "bfloat16" else "fp32"
    rng = random.Random(0)

    def say(msg):
        print(f"[bench] {msg}", file=sys.stderr, flush=True)

    def make_engine(name, layers, max_batch, tokens_per_request, chunk):
        """An engine with random weights made on the device and room for max_batch requests of that length."""
        full = PRESETS[name]
        cfg = LlamaConfig.from_dict(full.to_dict())
        if layers is not None:
            cfg.num_hidden_layers = layers
        cfg.validate()
        t0 = time.time()
        model = random_model(cfg, seed=0, dtype=args.dtype, device="cuda:0")
        torch.cuda.synchronize()
        say(f"{name} model built in {time.time() - t0:.1f} s")
        pages = max_batch * ((tokens_per_request + args.page_size - 1) // args.page_size) + 8
        eng = Engine(model, dtype=args.dtype, page_size=args.page_size, kv_pages=pages, max_batch_size=max_batch,
                     max_num_batched_tokens=2048, prefill_chunk_size=chunk, use_graph=not args.no_graph,
                     chain_steps=not args.no_chain)
        weight_bytes = model.weight_bytes(include_embedding=False)
        if model.lm_head.tied:
            weight_bytes += model.embedding.weight.numel() * model.embedding.weight.element_size()
        return eng, cfg, full, weight_bytes

    def prompt(vocab, n):
        return [rng.randrange(vocab) for _ in range(n)]

    greedy = dict(temperature=0.0, ignore_eos=True)

    # ---- through the engine: add_request / step with scheduler, step function and sampler ---------------------
    def engine_decode(eng, cfg, weight_bytes, batch, prompt_len, n_warm, n_steps):
        """`batch` requests with prompts of prompt_len tokens decode n_warm + n_steps tokens; the steps after the
        warm-up are timed between synchronisations.  Returns tokens a second, the mean, median and 95th
        percentile of the step time in ms (from the arrival of each step's tokens on the host), the bytes a
        step has to read, and the range of cache lengths that was timed."""
        # (early requests decode while late ones still bring their prompts, a portion a step)
        margin = batch * (-(-prompt_len // 2048) + 1) + 8
        params = SamplingParams(max_new_tokens=n_warm + n_steps + margin, **greedy)
        rids = [eng.add_request(prompt(cfg.vocab_size, prompt_len), params) for _ in range(batch)]
        reqs = [eng.request(r) for r in rids]
        while not all(r.output for r in reqs):               # prompts in portions, until every request decodes
            eng.step()
        for _ in range(n_warm):
            eng.step()
        torch.cuda.synchronize()
        kv0 = sum(r.num_computed for r in reqs) / batch
        stamps = [time.perf_counter()]
        for _ in range(n_steps):
            out = eng.step()
            assert len(out) == batch
            stamps.append(time.perf_counter())
        torch.cuda.synchronize()
        dt = time.perf_counter() - stamps[0]
        kv1 = sum(r.num_computed for r in reqs) / batch
        for r in rids:
            eng.abort(r)
        while eng.has_unfinished():
            eng.step()
        per = [1e3 * (b - a) for a, b in zip(stamps, stamps[1:])]
        mean_ctx = (kv0 + kv1 + 1) / 2.0
        bytes_step = weight_bytes + batch * mean_ctx * cfg.kv_bytes_per_token(elem)
        return {"tps": batch * n_steps / dt, "ms": 1e3 * dt / n_steps, "p50": percentile(per, 50), "p95": percentile(per, 95),
                "bytes": bytes_step, "kv": (int(round(kv0)), int(round(kv1)))}

    # ---- the bare step function: tokens stay on the device, no scheduler, no sampler object -------------------
    def runner_decode(eng, cfg, batch, prompt_len, n_warm, n_steps):
        runner = eng.runner
        rids = [("d", batch, i) for i in range(batch)]
        for rid in rids:
            runner.add_request(rid)
            runner.step([StepEntry(rid, prompt(cfg.vocab_size, prompt_len), [])])
        lg = runner.step([StepEntry(rid, [rng.randrange(cfg.vocab_size)], [0]) for rid in rids])
        chosen = ops.argmax(lg)
        coming = ops.HostCopy(chosen)

        def one():
            nonlocal chosen, coming
            if not runner.use_graph or args.no_chain:
                lg = runner.step([StepEntry(rid, [t], [0]) for rid, t in zip(rids, coming.result())])
                chosen = ops.argmax(lg)
                coming = ops.HostCopy(chosen)
                return
            lg = runner.step_chained(rids, chosen)
            nxt = ops.argmax(lg)
            nxt_coming = ops.HostCopy(nxt)
            runner.prepare_decode(rids)
            coming.result()
            chosen, coming = nxt, nxt_coming

        for _ in range(n_warm):
            one()
        torch.cuda.synchronize()
        t = time.perf_counter()
        for _ in range(n_steps):
            one()
        torch.cuda.synchronize()
        dt = time.perf_counter() - t
        for rid in rids:
            runner.end_request(rid)
        return batch * n_steps / dt, 1e3 * dt / n_steps

    def prefill_point(eng, cfg, T, runs, warm=3):
        """One prompt of T tokens from an empty cache as one step; mean of `runs` after `warm` warm-ups, a fresh
        request (no cached keys) each time (/root/reference/tools/bench-gpu/src/bench_real_model.rs:160-278: warm-ups,
        then timed forwards on fresh sessions, tokens a second from the mean time)."""
        runner = eng.runner
        times = []
        for i in range(warm + runs):
            rid = ("p", T, i)
            runner.add_request(rid)
            toks = prompt(cfg.vocab_size, T)
            torch.cuda.synchronize()
            t = time.perf_counter()
            runner.step([StepEntry(rid, toks, [T - 1])])
            torch.cuda.synchronize()
            dt = time.perf_counter() - t
            runner.end_request(rid)
            if i >= warm:
                times.append(dt)
        ms = 1e3 * sum(times) / len(times)
        L, H, I, V = cfg.num_hidden_layers, cfg.hidden_size, cfg.intermediate_size, cfg.vocab_size
        qd, kvd = cfg.num_attention_heads * cfg.head_dim, cfg.num_key_value_heads * cfg.head_dim
        linear = L * (H * (qd + 2 * kvd) + qd * H + 3 * H * I)
        flops = 2.0 * T * linear + 2.0 * V * H + L * 4.0 * cfg.num_attention_heads * cfg.head_dim * T * (T + 1) / 2
        peak = MFMA_PEAK[dshort]
        return {"value": round(T / (ms / 1e3), 1), "tokens": T, "ms": round(ms, 3), "frac": round(flops / (ms / 1e3) / peak, 4)}

    def fingerprint(eng, cfg, batch, prompt_len, n_steps):
        """Two fresh runs of the same requests (greedy): the sum of the bit patterns of the last step's logits and
        the tokens must agree (/root/reference/tools/bench-gpu/src/bench_real_model.rs:193-224)."""
        runner = eng.runner
        g = random.Random(1234)
        prompts = [[g.randrange(cfg.vocab_size) for _ in range(prompt_len)] for _ in range(batch)]
        sums, toks = [], []
        for run in range(2):
            rids = [("f", run, i) for i in range(batch)]
            for rid, p in zip(rids, prompts):
                runner.add_request(rid)
                lg = runner.step([StepEntry(rid, p, [prompt_len - 1])])
            cur = [0] * batch
            seen = []
            lg = runner.step([StepEntry(rid, [p[-1]], [0]) for rid, p in zip(rids, prompts)])
            for _ in range(n_steps):
                cur = ops.argmax(lg).tolist()
                seen.append(cur)
                lg = runner.step([StepEntry(rid, [t], [0]) for rid, t in zip(rids, cur)])
            bits = lg.contiguous().view(torch.int32).to(torch.int64) & 0xFFFFFFFF
            sums.append(int(bits.sum().item()))
            nan = int(torch.isnan(lg).sum().item())
            toks.append(seen)
            for rid in rids:
                runner.end_request(rid)
        return {"bits_sum": sums[0], "runs": 2, "nan": nan, "equal": sums[0] == sums[1] and toks[0] == toks[1] and nan == 0}

    # ---- the mixed serving workload ---------------------------------------------------------------------------
    def mixed_workload(eng, cfg, weight_bytes):
        g = random.Random(7)
        n_req = args.mixed_requests
        lens = [g.randint(128, 2048) for _ in range(n_req)]
        prompts = [[g.randrange(cfg.vocab_size) for _ in range(n)] for n in lens]
        if args.mixed_temperature > 0:
            mk = lambda i: SamplingParams(temperature=args.mixed_temperature, top_k=50, seed=100 + i,
                                          max_new_tokens=args.mixed_output, ignore_eos=True)
        else:
            mk = lambda i: SamplingParams(max_new_tokens=args.mixed_output, **greedy)
        # (warm the graphs and the allocator with a short run of the same shape, untimed)
        warm = [eng.add_request(p[:160], SamplingParams(max_new_tokens=4, **greedy)) for p in prompts[: min(n_req, 64)]]
        while eng.has_unfinished():
            eng.step()
        before = eng.stats()
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        rids = [eng.add_request(p, mk(i)) for i, p in enumerate(prompts)]
        first = {}
        kinds = {"decode_only": 0, "mixed": 0, "prefill_only": 0}
        tokens_by_kind = {"decode_only": 0, "mixed": 0, "prefill_only": 0}
        host_by_kind = {"decode_only": 0.0, "mixed": 0.0, "prefill_only": 0.0}
        step_ms = []
        n_out = 0
        while eng.has_unfinished():
            ts = time.perf_counter()
            out = eng.step()
            te = time.perf_counter()
            ls = eng.last_step
            kind = "decode_only" if ls["prompt_tokens"] == 0 else ("prefill_only" if ls["decode_tokens"] == 0 else "mixed")
            kinds[kind] += 1
            tokens_by_kind[kind] += ls["prompt_tokens"] + ls["decode_tokens"]
            step_ms.append(1e3 * (te - ts))
            for rid, tok, done in out:
                n_out += 1
                if rid not in first:
                    first[rid] = te - t0
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        after = eng.stats()
        ttft = [1e3 * first[r] for r in rids]
        steps = sum(kinds.values())
        eager = after["eager_steps"] - before["eager_steps"]
        pack_ms = (after["eager_step_pack_ms"] * after["eager_steps"] - before["eager_step_pack_ms"] * before["eager_steps"]) / max(1, eager)
        return {
            "model": args.mixed_config, "requests": n_req, "prompt_tokens": sum(lens), "output_tokens": n_out,
            "chunk": args.mixed_chunk, "sampling": "greedy" if args.mixed_temperature <= 0 else f"T={args.mixed_temperature} top_k=50",
            "seconds": round(dt, 3), "output_tok_s": round(n_out / dt, 1), "total_tok_s": round((n_out + sum(lens)) / dt, 1),
            "ttft_ms": {"mean": round(sum(ttft) / len(ttft), 1), "p50": round(percentile(ttft, 50), 1), "p95": round(percentile(ttft, 95), 1)},
            "steps": steps, "steps_by_kind": kinds,
            "tokens_per_step": {k: round(tokens_by_kind[k] / kinds[k], 1) if kinds[k] else 0 for k in kinds},
            "step_ms": {"mean": round(sum(step_ms) / len(step_ms), 3), "p50": round(percentile(step_ms, 50), 3), "p95": round(percentile(step_ms, 95), 3)},
            "preemptions": after["preemptions"] - before["preemptions"],
            "eager_steps": eager, "host_pack_ms_per_eager_step": round(pack_ms, 4),
        }

    # =============================================================================================================
    large = [] if (args.no_points or args.no_large_batches) else [128, 256]
    max_batch = args.batch if args.no_points else max([args.batch, 64] + large)
    long_tokens = 0 if (args.no_long or args.no_points) else 8 * 33536       # eight requests at a 32 k context
    per_request = max(args.context, -(-long_tokens // max_batch))
    eng, cfg, full, weight_bytes = make_engine(args.model_config, args.layers, max_batch, per_request, 2048)
    steps, warmup = args.steps, args.warmup
    if args.prompt_len + warmup + steps + 2 > args.context:
        steps = max(1, args.context - args.prompt_len - warmup - 2)
    points = {}

    def centred(n_warm, n_steps):
        """The prompt length from which n_warm untimed and n_steps timed steps are centred on the middle of the
        sweep from --prompt-len to --context (never below --prompt-len)."""
        mid = (args.prompt_len + args.context) // 2
        return max(args.prompt_len, mid - n_warm - n_steps // 2)

    prefill = None
    if not args.no_prefill:
        prefill = prefill_point(eng, cfg, args.prompt_len, 10)
        say(f"prefill {prefill}")

    head = engine_decode(eng, cfg, weight_bytes, args.batch, centred(warmup, steps), warmup, steps)
    say(f"engine decode b{args.batch}: {head['tps']:.1f} tok/s, {head['ms']:.3f} ms/step (p50 {head['p50']:.3f}, p95 {head['p95']:.3f}), KV {head['kv']}")
    achieved = head["bytes"] / (head["ms"] / 1e3) / 1e9

    determinism = None
    if not args.no_fingerprint:
        determinism = fingerprint(eng, cfg, min(args.batch, 8), 256, 16)
        say(f"determinism {determinism}")

    if not args.no_points:
        ps = max(1, min(args.point_steps, steps))
        for b in (1, 64):
            r = engine_decode(eng, cfg, weight_bytes, b, centred(8, ps), 8, ps)
            points[f"decode_b{b}"] = round(r["tps"], 1)
            points[f"decode_b{b}_hbm_frac"] = round(r["bytes"] / (r["ms"] / 1e3) / 1e9 / HBM_PEAK_GBS, 4)
            say(f"engine decode b{b}: {r['tps']:.1f} tok/s, {r['ms']:.3f} ms/step")
        for b in large:
            # (their prompts alone are b x 3,000 tokens of prefill: fewer timed steps, around the same cache length)
            r = engine_decode(eng, cfg, weight_bytes, b, centred(4, 100), 4, 100)
            points[f"decode_b{b}"] = round(r["tps"], 1)
            points[f"decode_b{b}_hbm_frac"] = round(r["bytes"] / (r["ms"] / 1e3) / 1e9 / HBM_PEAK_GBS, 4)
            say(f"engine decode b{b}: {r['tps']:.1f} tok/s, {r['ms']:.3f} ms/step, KV {r['kv']}")
        for b in sorted({1, args.batch, 64}):
            # (the same number of steps, so the same range of context lengths, as the engine's figure it stands beside)
            nw, ns = (warmup, steps) if b == args.batch else (8, ps)
            tps, ms = runner_decode(eng, cfg, b, centred(nw, ns), nw, ns)
            points[f"runner_b{b}"] = round(tps, 1)
            say(f"step function alone b{b}: {tps:.1f} tok/s, {ms:.3f} ms/step")
        if not args.no_long:
            for T in (8192, 32768):
                p = prefill_point(eng, cfg, T, 3 if T <= 8192 else 2, warm=2)
                points[f"prefill_{T}"] = p["value"]
                points[f"prefill_{T}_frac"] = p["frac"]
                say(f"prefill {p}")
            r = engine_decode(eng, cfg, weight_bytes, 8, 32768, 4, min(ps, 200))
            points["decode_b8_kv32k"] = round(r["tps"], 1)
            points["decode_b8_kv32k_hbm_frac"] = round(r["bytes"] / (r["ms"] / 1e3) / 1e9 / HBM_PEAK_GBS, 4)
            say(f"engine decode b8 at KV {r['kv']}: {r['tps']:.1f} tok/s, {r['ms']:.3f} ms/step")

    mixed = None
    if not args.no_mixed:
        del eng
        torch.cuda.empty_cache()
        eng3, cfg3, _, wb3 = make_engine(args.mixed_config, None, args.mixed_requests, 2048 + args.mixed_output + 64, args.mixed_chunk)
        # the named workload: portions of exactly the chunk; then the engine's default, which lengthens portions
        # with budget that no other request can use
        eng3.scheduler.config.fill_budget = False
        mixed = mixed_workload(eng3, cfg3, wb3)
        points["mixed_output_tok_s"] = mixed["output_tok_s"]
        points["mixed_ttft_p50_ms"] = mixed["ttft_ms"]["p50"]
        points["mixed_ttft_p95_ms"] = mixed["ttft_ms"]["p95"]
        say(f"mixed {mixed}")
        eng3.scheduler.config.fill_budget = True
        filled = mixed_workload(eng3, cfg3, wb3)
        points["mixed_fill_budget_output_tok_s"] = filled["output_tok_s"]
        points["mixed_fill_budget_ttft_p50_ms"] = filled["ttft_ms"]["p50"]
        say(f"mixed, portions lengthened into spare budget {filled}")

    out = {
        "metric": f"decode tok/s at batch {args.batch} through the engine, {args.model_config} shape {dshort}, "
                  f"KV {head['kv'][0]}->{head['kv'][1]}",
        "value": round(head["tps"], 1),
        "unit": "tok/s",
        "n_gpus": 1,
        "steps": steps,
        "warmup": warmup,
        "ms_per_step": round(head["ms"], 4),
        "ms_per_step_p50": round(head["p50"], 4),
        "ms_per_step_p95": round(head["p95"], 4),
        "higher_is_better": True,
        "scaling": "weak",
        "vs_baseline": None,
        "dtype": dshort,
        "data": "synthetic",
        "config": {
            "model": args.model_config, "layers": cfg.num_hidden_layers, "layers_full": full.num_hidden_layers,
            "hidden": cfg.hidden_size, "heads": cfg.num_attention_heads, "kv_heads": cfg.num_key_value_heads,
            "head_dim": cfg.head_dim, "intermediate": cfg.intermediate_size, "vocab": cfg.vocab_size,
            "global_batch": args.batch, "seq_len": args.context, "prompt_len": args.prompt_len,
            "decode_from_kv": head["kv"][0],
            "page_size": args.page_size, "weights": "random N(0,0.02)", "parallelism": "single GPU",
            "graph": not args.no_graph, "steps_queued_ahead": not args.no_chain, "sampling": "greedy",
            "path": "Engine.add_request/step",
        },
        "prefill": prefill,
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                     "frac": round(achieved / HBM_PEAK_GBS, 4)},
        "points": points,
        "determinism": determinism,
        "mixed": mixed,
    }
    print(json.dumps(out))
    return 0


if __name__ == "__main__":
    sys.exit(main())
