#!/usr/bin/env python3
"""Flagship decode benchmark (driver contract).

Measures the BASELINE.json metric: decode tokens/sec, batch 1, synthetic
prompt, random-init weights, bf16.  Default model is Llama-3.2-1B at
EVERY N (TP=N) so the driver's 1/2/4/8-GPU curve compares like with
like; the metric's second config (Gemma-2-9B TP=8, fp8) runs via
``--model gemma-2-9b --dtype fp8``.  A "step" is one decoded token; the
timed region is K hipGraph-replayed decode steps (full forward incl.
lm_head + sampling).

Usage: python bench.py [--gpus N] [--steps K] [--warmup W] [--model M]
Launched by the driver for N>1 via torch.distributed.run (one rank/GPU).
"""

import argparse
import json
import os
import sys
import time

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))


COMPARE = ("turudra-2k", "turudra-4k", "garupel-2k", "garupel-4k",
           "fidizen-2k", "fidizen-4k", "dogalorn-2k", "dogalorn-4k")


def compare(cases, steps, warmup, prompt=2048, batches=(1, 4, 16)):
    """One JSON line per model, size and batch: random weights, bf16,
    synthetic prompts.  Beside each design stands the closest other model
    of equal width, heads and layer runs.  Windowed latent attention stands
    beside unwindowed one, a dense feed-forward beside two experts, both
    chosen, and a shared one that hold as much; pairs of attention and
    recurrence beside the attention alone, state-space layers beside linear
    attention with as large a state; other designs stand beside a
    transformer.  An MoE one gets one more expert
    and one more choice, so its experts match the design's routed + shared
    ones in stored and in active parameters; a dense one gets two thirds of
    the hidden size, so its three matrices match the design's two."""
    import numpy as np
    import torch

    from csrc.build import ensure_built
    ensure_built()
    import llm_np_cp_amd as L
    from llm_np_cp_amd.io.loader import LazyRandomWeights
    from llm_np_cp_amd.models.registry import engine_class

    def latent_design(c):
        def layer(l):
            m, f = l.mixer, l.mlp
            if f.kind == "dense":     # 2 matrices -> 3 experts of 3
                n, top, ff = 2, 2, f.ff * 2 // 9
            else:
                n, top, ff = f.experts, f.top, f.expert.ff
            e = {"ff": ff, "limit": 7.0}
            keep = ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale",
                    "rot")
            d = m.to_dict()
            return {"type": "latent_attention",
                    "mixer": {k: d[k] for k in keep},
                    "mlp": {"kind": "moe", "expert": e, "shared": e,
                            "router": {"experts": n, "top": top}}}
        return "turudra", L.ModelConfig.from_hf_dict({
            "architecture": "Turudra", "vocab": c.vocab_size,
            "width": c.hidden_size, "norm": {"eps": 1e-6},
            "residual_mult": 0.5, "layers": [layer(l) for l in c.layers]})

    def grouped_design(c):
        heads = next(l.mixer.left.heads for l in c.layers
                     if l.mixer.kind == "parallel")

        def layer(l):
            m = l.mixer
            if m.kind == "parallel":
                d = m.left.to_dict()
                kind, mix = "attention", {
                    **{k: d[k] for k in ("heads", "kv_heads", "dim", "vdim",
                                         "scale")},
                    "q_temp": {"coef": 0.1, "every": 2048}}
            else:
                kind, mix = "lightning", dict(
                    heads=heads, dim=m.state, vdim=m.inner // heads,
                    decay=[1 - 2.0 ** (-3 - h % 6) for h in range(heads)])
            return {"type": kind, "mixer": mix,
                    "mlp": {"kind": "dense", "ff": l.mlp.ff}}
        return "garupel", L.ModelConfig.from_hf_dict({
            "architecture": "Garupel", "vocab": c.vocab_size,
            "width": c.hidden_size, "norm": {"eps": 1e-6},
            "layers": [layer(l) for l in c.layers]})

    def closest(c):
        if c.model_type == "fidizen":
            return latent_design(c)
        if c.model_type == "dogalorn":
            return grouped_design(c)
        att, ff = c.layers[0].mixer, c.layers[0].mlp
        kw = dict(vocab_size=c.vocab_size, hidden_size=c.hidden_size,
                  num_hidden_layers=len(c.runs), head_dim=128,
                  num_attention_heads=att.heads,
                  num_key_value_heads=max(1, att.heads // 4),
                  max_position_embeddings=32768, tie_word_embeddings=False)
        if ff.kind == "moe":
            return "mixtral", L.ModelConfig(
                model_type="mixtral", intermediate_size=ff.expert.ff,
                num_local_experts=ff.experts + 1,
                num_experts_per_tok=ff.top + 1, **kw)
        return "qwen2", L.ModelConfig(
            model_type="qwen2", attention_bias=True,
            intermediate_size=round(ff.ff * 2 / 3 / 64) * 64, **kw)

    def seconds(fn, n):
        torch.cuda.synchronize()
        t = time.perf_counter()
        for _ in range(n):
            fn()
        torch.cuda.synchronize()
        return (time.perf_counter() - t) / n

    for case in cases:
        preset, _, side = case.partition(":")
        if "-" not in preset:
            preset = "turudra-" + preset
        family, _, size = preset.partition("-")
        design = L.preset_config(preset)
        for name, cfg in ((family, design), closest(design)):
            if side and side != name:
                continue
            rng = np.random.default_rng(0)
            ids = rng.integers(0, cfg.vocab_size, size=(max(batches),
                                                        prompt))
            line = {"model": f"{name}-{size}", "dtype": "bf16",
                    "data": "synthetic",
                    "layers": len(getattr(cfg, "runs", ())) or
                    cfg.num_hidden_layers}

            def show(what, dt, tokens):
                print(json.dumps({**line, "what": what, "ms": dt * 1e3,
                                  "tokens/s": tokens / dt}), flush=True)

            # a single-sequence engine for batch 1 (its own fused path in
            # the transformer), then one with rows for the batches
            for rows in (1, max(batches)):
                model = engine_class(cfg)(
                    cfg, LazyRandomWeights(cfg, seed=0), max_seq=4096,
                    max_batch=rows, seed=0)
                if rows == 1:
                    model.prefill(ids[0])
                    show(f"prefill {prompt}",
                         seconds(lambda: model.prefill(ids[0]), 5), prompt)
                    model.decode(max(warmup, 3), greedy=True)
                    show(f"decode batch 1 at {prompt}+",
                         seconds(lambda: model._graph.replay(), steps), 1)
                for B in [b for b in batches if b > 1 and rows > 1]:
                    model.prefill_batch(ids[:B])
                    model.decode_batch(max(warmup, 3), greedy=True)
                    show(f"decode batch {B} at {prompt}+",
                         seconds(lambda: model._graph.replay(), steps), B)
                del model
                torch.cuda.empty_cache()


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=200)
    ap.add_argument("--warmup", type=int, default=20)
    ap.add_argument("--model", type=str, default="llama-3.2-1b",
                    help="model preset (default llama-3.2-1b at every N "
                         "so the driver's 1/2/4/8-GPU scaling curve "
                         "compares like with like; gemma-2-9b etc. via "
                         "this flag; synthetic random-init weights)")
    ap.add_argument("--prompt-len", type=int, default=64)
    ap.add_argument("--max-seq", type=int, default=None)
    ap.add_argument("--dtype", type=str, default="bf16",
                    choices=["bf16", "fp8", "fp4"],
                    help="weight dtype (constant across N for honest "
                         "scaling; fp8 = BASELINE config 4)")
    ap.add_argument("--kv-dtype", type=str, default="bf16",
                    choices=["bf16", "fp8"],
                    help="KV-pool dtype (fp8 = e4m3 with per-head-pos "
                         "scales; halves the attention read stream)")
    ap.add_argument("--batch", type=int, default=1,
                    help="lockstep batched decode (throughput mode; "
                         "value = aggregate tokens/s over the batch)")
    ap.add_argument("--no-graph", action="store_true")
    ap.add_argument("--compare", nargs="*", default=None, metavar="CASE",
                    help="instead of the default workload: prefill and "
                         "decode throughput of the layer-list designs "
                         "beside the closest other model of equal size; "
                         "cases turudra-2k (or 2k), turudra-4k, garupel-2k, "
                         "garupel-4k, fidizen-2k, fidizen-4k, dogalorn-2k, "
                         "dogalorn-4k (default all), each optionally with "
                         ":turudra, :mixtral, :garupel, :qwen2, :fidizen or "
                         ":dogalorn for one side only")
    args = ap.parse_args()
    if args.compare is not None:
        return compare(args.compare or COMPARE, args.steps, args.warmup)

    import numpy as np
    import torch

    world = int(os.environ.get("WORLD_SIZE", "1"))
    n_gpus = max(world, args.gpus)
    model_name = args.model

    from csrc.build import ensure_built
    ensure_built()

    import llm_np_cp_amd as L
    from llm_np_cp_amd.io.loader import LazyRandomWeights
    from llm_np_cp_amd.models.engine import GPUModel
    from llm_np_cp_amd.parallel.tp import init_distributed

    rank, world = init_distributed()
    dtype = args.dtype
    cfg = L.preset_config(model_name)
    max_seq = args.max_seq or min(
        cfg.max_position_embeddings,
        args.prompt_len + args.steps + args.warmup + 64)
    w = LazyRandomWeights(cfg, seed=0)
    model = GPUModel(cfg, w, max_seq=max_seq, seed=0, dtype=dtype,
                     kv_dtype=args.kv_dtype, max_batch=args.batch)

    if rank == 0 and world > 1:
        from llm_np_cp_amd.parallel import tp as _tp
        mode = ("one-shot xGMI" if _tp.xgmi_comm() is not None
                else "RCCL fallback")
        print(f"# decode collectives: {mode} (world={world})",
              file=sys.stderr)

    rng = np.random.default_rng(0)
    prompt = rng.integers(0, cfg.vocab_size, size=args.prompt_len)

    def barrier():
        if world > 1:
            torch.distributed.barrier()

    # prefill + warmup
    use_graph = not args.no_graph
    if args.batch > 1:
        prompts = rng.integers(0, cfg.vocab_size,
                               size=(args.batch, args.prompt_len))
        model.prefill_batch(prompts)
        model.decode_batch(max(args.warmup, 2), greedy=True,
                           use_graph=use_graph)
        if model._graph_mode is None:
            use_graph = False
    else:
        model.prefill(prompt)
        if args.warmup > 0:
            model.decode(args.warmup, greedy=True, use_graph=use_graph,
                         first_from_logits=True)

    if use_graph and args.batch == 1:
        # no-op if the warmup already captured; on failure the step it
        # executed is harmless here (untimed region)
        _, ok = model.capture_decode_graph(True, 0.1)
        if not ok:
            if rank == 0:
                err = getattr(model, "_graph_error", None)
                print(f"# graph capture unavailable "
                      f"({type(err).__name__ if err else '?'}: {err}); "
                      f"timing eager launches", file=sys.stderr)
            use_graph = False

    # timed region: exactly K decode steps
    barrier()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    if use_graph:
        for _ in range(args.steps):
            model._graph.replay()
    elif args.batch > 1:
        for _ in range(args.steps):
            model._decode_batch_step(args.batch, True, 0.1)
    else:
        for _ in range(args.steps):
            model._decode_step(True, 0.1)
    torch.cuda.synchronize()
    barrier()
    t1 = time.perf_counter()

    elapsed = t1 - t0
    if world > 1:
        t = torch.tensor([elapsed], device=model.device)
        torch.distributed.all_reduce(t, op=torch.distributed.ReduceOp.MAX)
        elapsed = float(t.item())

    toks_per_s = args.steps * args.batch / elapsed
    ms_per_step = elapsed / args.steps * 1e3

    if rank == 0:
        out = {
            "metric": "decode tokens/sec",
            "value": toks_per_s,
            "unit": "tokens/s",
            "n_gpus": world,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": ms_per_step,
            "higher_is_better": True,
            "scaling": "strong",
            "vs_baseline": None,
            "dtype": dtype,
            "data": "synthetic",
            "config": {
                "model": model_name,
                "kv_dtype": args.kv_dtype,
                "global_batch": args.batch,
                "seq_len": args.prompt_len + args.warmup + args.steps,
                "parallelism": f"tp{world}",
            },
        }
        print(json.dumps(out))


if __name__ == "__main__":
    main()
