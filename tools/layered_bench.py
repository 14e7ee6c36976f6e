"""Prompt and decode throughput of a layered design at sizes that resemble a real model's layers, random weights, beside the closest other
model of the same width and depth: Timerax beside the DeepSeek engine's model of the same expert sizes, Ranutar beside Timerax.

  python bench.py --layered lite [--layered-design ranutar]           (this module's measure(), one JSON line)
  python tools/layered_bench.py --size wide --prompt 2048 --batch 1,16 --no-compare

  lite   27 layers of width 2048, 64 experts top 6 of 1408, shared expert 2816     (DeepSeek-V2-Lite's shapes; FP16 weights there)
  wide    3 layers of width 7168, 256 experts top 8 of 2048, shared expert 2048    (DeepSeek-V3's shapes; Q2_K weights there)
Ranutar's dense feed-forwards have as many weights as Timerax reads per token.
"""
import argparse
import json
import os
import sys
import time

import numpy as np

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
for p in (ROOT, os.path.join(ROOT, "deepseek.cpp_amd")):
    if p not in sys.path:
        sys.path.insert(0, p)


def config(size: str) -> dict:
    wide = size == "wide"
    D = 7168 if wide else 2048
    heads = 64 if wide else 16
    moe = {"kind": "moe", "router": {"experts": 256 if wide else 64, "top": 8 if wide else 6},
           "expert": {"ff": 2048 if wide else 1408, "limit": 7.0}, "shared": {"ff": 2048 if wide else 2816, "limit": 7.0}}
    delta = {"type": "channel_delta", "mixer": {"conv": 4, "dim": 128, "heads": heads, "kv_heads": heads, "vdim": 128}, "mlp": moe}
    par = {"type": "parallel", "mlp": moe, "mixer": {
        "left": {"heads": heads, "kv_heads": heads // 4, "dim": 128, "vdim": 128, "mask": {"size": 4096}, "scale": 0.0883883,
                 "rot": {"base": 500000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}},
        "right": {"heads": heads, "dim": 64, "vdim": 128, "gate_cap": 15.0}}}
    return {"architecture": "Timerax", "width": D, "vocab": 129280 if wide else 102400, "norm": {"eps": 1e-6}, "logit_softcap": 30.0,
            "layers": [delta, delta, par] * (1 if wide else 9)}


def ranutar(size: str) -> dict:
    wide = size == "wide"
    D, heads = (7168, 64) if wide else (2048, 16)
    mlp = {"kind": "dense", "ff": 27648 if wide else 16896}
    wkv = {"type": "wkv", "mixer": {"heads": D // 64, "dim": 64}, "mlp": mlp}
    delta = {"type": "delta", "mixer": {"conv": 4, "dim": 128, "heads": heads, "kv_heads": heads, "vdim": 128}, "mlp": mlp}
    lat = {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": 1536, "kv_rank": 512, "mask": {"size": 4096}, "scale": 0.0721688,
        "rot": {"base": 500000.0, "dims": 64}}}
    return {"architecture": "Ranutar", "width": D, "vocab": 129280 if wide else 102400, "norm": {"eps": 1e-6}, "canon": {"taps": 4}, "logit_scale": 0.5,
            "layers": [wkv, delta, lat] * (1 if wide else 9)}


CONFIGS = {"timerax": config, "ranutar": ranutar}


def timed(fn, reps):
    best = 1e9
    for _ in range(reps):
        t0 = time.perf_counter()
        fn()
        best = min(best, time.perf_counter() - t0)
    return best


def layered(ctx, size, prompts, batches, steps=32, ctx_len=512, reps=2, graph=True, design="timerax"):
    import dsk
    c = CONFIGS[design](size)
    M = dsk.LM(ctx, dtype="bfloat16", config=c, seed=1, options=f"piece_tokens={max(2048, min(8192, max(prompts)))},decode_graph={int(graph)}")
    rng = np.random.default_rng(0)
    toks = rng.integers(0, c["vocab"], max(prompts + [ctx_len]) + 1)
    out = {"device_gb": round(M.device_bytes() / 1e9, 1), "sequence_mb": round(M.info("sequence_kb") / 1024, 2), "prefill": {}, "decode": {}}
    for P in prompts:
        def run():
            s = M.seq_open()
            M.step([(s, toks[:P], [P - 1])])
            M.seq_close(s)
        run()
        dt = timed(run, reps)
        out["prefill"][str(P)] = {"ms": round(dt * 1e3, 3), "tok_s": round(P / dt, 1)}
    for B in batches:
        seqs = [M.seq_open() for _ in range(B)]
        for i in range(0, B, 4):
            M.step([(s, np.roll(toks, 7 * s)[:ctx_len], []) for s in seqs[i:i + 4]])
        nxt = list(range(B))

        def run(n):
            nonlocal nxt
            for _ in range(n):
                M.step_sample([(s, [int(t)]) for s, t in zip(seqs, nxt)])
                nxt = rng.integers(0, c["vocab"], B)  # (a random model repeats itself: random tokens keep the routing spread)
        run(4)
        t0 = time.perf_counter()
        run(steps)
        dt = (time.perf_counter() - t0) / steps
        ab = M.active_bytes(ctx_len + 4 + steps // 2)
        out["decode"][str(B)] = {"ms_per_step": round(dt * 1e3, 4), "tok_s": round(B / dt, 1)}
        if B == 1:
            out["decode"]["1"].update(algo_bytes_per_token=round(ab), token_frac_of_8TBs=round(ab / dt / 8e12, 4))
        for s in seqs:
            M.seq_close(s)
    out["graph_steps"] = M.info("graph_steps")
    M.close()
    return out


def deepseek(ctx, size, prompts, steps=32, ctx_len=512, reps=2, graph=True):
    """the existing model of the same width, depth and expert sizes: decode at batch 1, prompts through dsk_hydrate"""
    import dsk
    from tools import synth
    wide = size == "wide"
    c = synth.preset("v3" if wide else "v2lite", "q2_k" if wide else "fp16", False)
    if wide:
        c.n_layers, c.first_k_dense_replace = 3, 0
    c.max_seq_len = max(prompts + [ctx_len + steps + 8]) + 8
    M = dsk.Model(ctx, c, None, synth_seed=0)
    M.set_graph(graph)
    toks = np.random.default_rng(0).integers(0, c.vocab_size, max(prompts + [ctx_len + steps + 8]))
    out = {"weights": c.quant, "layers": c.n_layers, "prefill": {}, "why_not_batched": M.hydrate_why_not()}
    for P in prompts:
        M.hydrate(toks[:min(P, 64)], 0)
        dt = timed(lambda: M.hydrate(toks[:P], 0, dsk.MODE_OUTPUT_LOGITS), reps if not M.hydrate_why_not() else 1)
        out["prefill"][str(P)] = {"ms": round(dt * 1e3, 3), "tok_s": round(P / dt, 1)}
    for i in range(4):
        M.forward_argmax(int(toks[i]), ctx_len + i)
    t0 = time.perf_counter()
    for i in range(steps):
        M.forward_argmax(int(toks[i]), ctx_len + 4 + i)
    dt = (time.perf_counter() - t0) / steps
    ab = M.active_bytes(ctx_len + 4 + steps // 2)
    out["decode"] = {"1": {"ms_per_step": round(dt * 1e3, 4), "tok_s": round(1 / dt, 1), "algo_bytes_per_token": round(ab),
                           "token_frac_of_8TBs": round(ab / dt / 8e12, 4)}}
    M.close()
    return out


def measure(size="lite", prompts=(512, 2048), batches=(1, 4, 16), compare=True, steps=32, graph=True, ours=True, design="timerax"):
    import dsk
    ctx = dsk.Ctx(0)
    out = {"metric": f"layered design ({design.capitalize()}) prefill and decode throughput, {size}", "unit": "tok/s", "data": "synthetic (random weights)",
           "dtype": "bf16"}
    if ours:
        out[design] = layered(ctx, size, list(prompts), list(batches), steps, graph=graph, design=design)
        out["value"] = out[design]["decode"][str(batches[0])]["tok_s"]
    if compare and design == "timerax":
        out["deepseek"] = deepseek(ctx, size, [p for p in prompts if p <= 2048], steps, graph=graph)
    elif compare:
        out["timerax"] = layered(ctx, size, list(prompts), list(batches), steps, graph=graph)
    ctx.close()
    return out


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--size", default="lite", choices=["lite", "wide"])
    ap.add_argument("--design", default="timerax", choices=sorted(CONFIGS))
    ap.add_argument("--prompt", default="512,2048")
    ap.add_argument("--batch", default="1,4,16")
    ap.add_argument("--steps", type=int, default=32)
    ap.add_argument("--no-compare", action="store_true")
    ap.add_argument("--only-compare", action="store_true", help="the model it is compared with alone")
    ap.add_argument("--no-graph", action="store_true", help="decode steps launched one by one (kernel traces)")
    a = ap.parse_args()
    print(json.dumps(measure(a.size, [int(v) for v in a.prompt.split(",")], [int(v) for v in a.batch.split(",")], not a.no_compare, a.steps,
                             not a.no_graph, not a.only_compare, a.design)))


if __name__ == "__main__":
    main()
