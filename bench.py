"""Decode and prefill throughput of the engine at MiniCPM4-8B size with random weights on one GPU.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--context 4096] [--layers L]

A "step" is one decode step of the engine's own step function followed by greedy sampling, with
`--batch` requests that each hold `--context` tokens in the paged cache when the last timed step
ends.  One JSON line is printed: `value` is decoded tokens a second at the default batch;
`prefill` is one 2,048-token prompt in one step (the median of seven passes timed with events);
`roofline` prices the decode step against HBM bandwidth (every weight it uses read once, plus the
cache of the live requests); `points` holds decode at batch 1, 32 and 64 and `points_frac` the same
pricing of each; `fp32` the batch-8 step and the prefill on the true 32-bit path.  Peaks are MI355X's
published ones (HBM 8 TB/s; dense MFMA bf16 2.5 PFLOP/s, fp32 157.3 TFLOP/s).  Weights are random (N(0, 0.02), norms 1 + N(0, 0.02)) and the
cache of the context is filled with random keys and values instead of being computed: the timed
steps do all of their work.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK = 8.0e12
FLOP_PEAK = {"bf16": 2.5e15, "fp32": 157.3e12}


def config_8b(layers: int) -> dict:
    """The layer sizes of the MiniCPM4-8B shape."""
    sys.path.insert(0, os.path.join(ROOT, "examples"))
    from shapes import shape_config
    return shape_config("8b", layers)


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=32)
    ap.add_argument("--warmup", type=int, default=4)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=4096)
    ap.add_argument("--prefill-tokens", type=int, default=2048)
    ap.add_argument("--layers", type=int, default=32, help="layers to run (the 8B configuration has 32)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--page-size", type=int, default=64)
    ap.add_argument("--no-graph", action="store_true", help="launch every kernel of a decode step eagerly")
    ap.add_argument("--prefill-only", action="store_true", help="only the prefill measurement (for profiling)")
    ap.add_argument("--no-points", action="store_true", help="skip the batch 1 / 32 / 64 points, the prefill and the 32-bit record")
    ap.add_argument("--no-fp32", action="store_true", help="skip the 32-bit record (bfloat16 runs only)")
    ap.add_argument("--designs", action="store_true",
                    help="instead of the default workload: prefill and decode throughput of another design (--design) beside MiniCPM4 "
                         "at equal layer sizes (random weights), with the time and the roofline share of every kernel")
    ap.add_argument("--design-shapes", default="1024,4096", help="widths to compare with --designs")
    ap.add_argument("--design", default="kekevik", choices=["kekevik", "pugavik", "patadra", "bebuzen", "moputar", "lizezen"],
                    help="the design that --designs puts beside MiniCPM4 (moputar: beside Kekevik too, whose recurrence is the closest to its; "
                         "lizezen: beside Moputar and Patadra too, for its recurrence and its experts)")
    args = ap.parse_args()
    if args.gpus != 1 or int(os.environ.get("WORLD_SIZE", "1")) != 1:
        print("bench.py measures one GPU: this engine has no multi-GPU path (N>1 is not run)")
        return 2

    import torch
    from infinilm_amd.csrc import lib
    from infinilm_amd.engine.loading import require_gpu

    require_gpu("cuda:0")
    lib.load()
    if args.designs:
        print(json.dumps(compare_designs(args)))
        return 0
    FULL_LAYERS = 32
    cfg = config_8b(args.layers)
    record = measure(args, cfg, args.dtype, FULL_LAYERS, full=True)
    if args.dtype == "bfloat16" and not args.no_points and not args.no_fp32 and not args.prefill_only:
        torch.cuda.empty_cache()
        f = measure(args, cfg, "float32", FULL_LAYERS, full=False)
        record["fp32"] = {"decode_b%d" % args.batch: f["value"], "ms_per_step": f["ms_per_step"], "hbm_frac": f["roofline"]["frac"],
                          "prefill_ms": f["prefill"]["ms"], "prefill_frac": f["prefill"]["frac"]}
    print(json.dumps(record))
    return 0


def compare_designs(args) -> dict:
    """`--design` (and with moputar Kekevik, with lizezen Moputar and Patadra too) beside MiniCPM4 at equal width, layers, heads, head size and feed-forward parameters: prefill of
    `--prefill-tokens` tokens in one step, decode at batch 8 and 64 over `--context` tokens (recorded steps), and for
    every kernel entry point its calls, its time a call in eager steps and, where one bound names it, the share of that
    bound it reaches: bytes it must move over the HBM peak, or floating-point work over the vector float32 peak."""
    import torch
    from infinilm_amd import kernels
    from infinilm_amd.engine.loading import build_model, make_runner
    from infinilm_amd.engine.step import StepEntry
    from infinilm_amd.sampling import Sampler, SamplingParams
    from infinilm_amd.weights import fill_random_
    sys.path.insert(0, os.path.join(ROOT, "examples"))
    from shapes import bebuzen_shape, kekevik_shape, lizezen_shape, moputar_shape, patadra_shape, pugavik_shape

    layers = 8 if args.layers == 32 else args.layers
    T, ctx, ps = args.prefill_tokens, min(args.context, 2048), args.page_size
    design = args.design
    out = {"metric": f"prefill and decode tokens/s, {design.capitalize()} beside MiniCPM4 at equal layer sizes", "dtype": "bf16", "layers": layers,
           "prefill_tokens": T, "context": ctx, "data": "synthetic: random weights and token ids, random-filled cache", "shapes": {}}
    sampler, greedy = Sampler(0), SamplingParams(top_k=1)
    gen = torch.Generator().manual_seed(7)
    for width in [int(w) for w in args.design_shapes.split(",")]:
        heads, d, kv, V = width // 128, 128, 2, 32768
        cfgs = {
            "minicpm4": {"architectures": ["MiniCPMForCausalLM"], "model_type": "minicpm", "torch_dtype": "bfloat16", "rope_theta": 10000.0,
                         "num_hidden_layers": layers, "hidden_size": width, "num_attention_heads": heads, "num_key_value_heads": kv,
                         "head_dim": d, "intermediate_size": 4 * width, "vocab_size": V, "max_position_embeddings": 32768,
                         "rms_norm_eps": 1e-6, "tie_word_embeddings": True},
            design: patadra_shape(width, heads, d, layers, V) if design == "patadra" else
            bebuzen_shape(width, heads, d, kv, layers, V) if design == "bebuzen" else
            moputar_shape(width, heads, d, kv, layers, V) if design == "moputar" else
            lizezen_shape(width, heads, d, kv, layers, V) if design == "lizezen" else
            (kekevik_shape if design == "kekevik" else pugavik_shape)(width, heads, d, kv, layers, V, 6 * width)}
        if design == "moputar":
            cfgs["kekevik"] = kekevik_shape(width, heads, d, kv, layers, V, 6 * width)
        if design == "lizezen":
            cfgs["moputar"] = moputar_shape(width, heads, d, kv, layers, V)
            cfgs["patadra"] = patadra_shape(width, heads, d, layers, V)
        rec = {}
        for name, cfg in cfgs.items():
            model = build_model(cfg, "bfloat16", "cuda:0")
            fill_random_(model, seed=0, std=0.02, norm_init="one_plus")
            for pname, p in model.named_parameters().items():
                if pname.endswith(".correction"):      # (random corrections would outweigh the scores: every token the same experts)
                    p.tensor.zero_()
            Hs = model.spec.hidden_size
            params = sum(p.tensor.numel() for p in model.named_parameters().values())
            r = {"parameters": params}
            for graph in (True, False):
                runner = make_runner(model, num_pages=64 * (-(-(ctx + 1) // ps)) + -(-T // ps) + 4, page_size=ps, max_requests=65,
                                     enable_graph=graph)
                cache = runner.cache
                for e in cache.k:
                    cache.k[e].normal_(0, 1.0)
                    cache.v[e].normal_(0, 1.0)

                def prefill(passes):
                    prompt = torch.randint(0, V, (T,), generator=gen).tolist()
                    times = []
                    for i in range(passes):
                        cache.admit("p")
                        torch.cuda.synchronize()
                        t0 = time.perf_counter()
                        sampler.sample(runner.step([StepEntry("p", prompt, [T - 1])]), [(greedy, 0, 0)])
                        torch.cuda.synchronize()
                        times.append(time.perf_counter() - t0)
                        cache.release("p")
                    return sorted(times[1:])[len(times[1:]) // 2]

                def decode(batch, steps, warmup):
                    ids = [f"d{i}" for i in range(batch)]
                    for rid in ids:
                        cache.admit(rid)
                        cache.reserve(rid, ctx - steps - warmup)
                        cache.commit(rid, ctx - steps - warmup)
                    toks = torch.randint(0, V, (batch,), generator=gen).tolist()
                    for i in range(steps + warmup):
                        if i == warmup:
                            torch.cuda.synchronize()
                            t0 = time.perf_counter()
                        toks = sampler.sample(runner.step([StepEntry(rid, [t], [0]) for rid, t in zip(ids, toks)]),
                                              [(greedy, j, 0) for j in range(batch)])
                    torch.cuda.synchronize()
                    dt = (time.perf_counter() - t0) / steps
                    for rid in ids:
                        cache.release(rid)
                    return dt

                if graph:
                    pt = prefill(5)
                    r["prefill_tok_s"] = round(T / pt, 1)
                    r["prefill_ms"] = round(pt * 1e3, 3)
                    for b in (8, 64):
                        dt = decode(b, max(8, args.steps // 2), args.warmup)
                        r[f"decode_b{b}_tok_s"] = round(b / dt, 1)
                        r[f"decode_b{b}_ms"] = round(dt * 1e3, 4)
                else:   # eager steps with a pair of events around every launch: the kernels' own times
                    kernels.enable_timing(True)
                    prefill(2)
                    kernels.timing_report()
                    prefill(2)
                    rep_p = kernels.timing_report()
                    decode(64, 4, 2)
                    kernels.timing_report()
                    decode(64, 4, 0)
                    rep_d = kernels.timing_report()
                    kernels.enable_timing(False)
                    r["kernels_prefill_us"] = {k: [v["calls"], v["mean_us"]] for k, v in sorted(rep_p.items())}
                    r["kernels_decode_b64_us"] = {k: [v["calls"], v["mean_us"]] for k, v in sorted(rep_d.items())}
                    # bounds of the kernels that the design adds, and of the attention kernels beside them
                    us = lambda rep, k: rep[k]["mean_us"] * 1e-6 if k in rep else None
                    share = {}
                    state = heads * d * d * 4          # a head's state x heads (key size = value size = state entries = d here)
                    kvb = 2 * kv * d * 2               # cached bytes a token
                    if name == "patadra":
                        m0 = cfg["layers"][0]
                        E, top, ff, win = m0["mlp"]["router"]["experts"], m0["mlp"]["router"]["top"], m0["mlp"]["expert"]["ff"], m0["mixer"]["mask"]["size"]
                        gu, dn = "ilm_moe_gemm (gate/up)", "ilm_moe_gemm (down)"
                        if us(rep_p, gu):
                            share["experts' gate/up product prefill (flops / bf16 matrix peak)"] = round(2.0 * T * top * 2 * ff * Hs / us(rep_p, gu) / FLOP_PEAK["bf16"], 4)
                            share["experts' down product prefill (flops / bf16 matrix peak)"] = round(2.0 * T * top * ff * Hs / us(rep_p, dn) / FLOP_PEAK["bf16"], 4)
                            hit = min(E, 64 * top)
                            share["experts' gate/up product decode (weights of the experts hit read / HBM peak)"] = round(hit * 2 * ff * Hs * 2 / us(rep_d, gu) / HBM_PEAK, 4)
                            share["experts' down product decode (weights of the experts hit read / HBM peak)"] = round(hit * ff * Hs * 2 / us(rep_d, dn) / HBM_PEAK, 4)
                        lat = "ilm_attn_headmix_mfma"   # (one cached row of d entries a token, read as key and as value)
                        if us(rep_d, lat):
                            share["latent attention decode (window's cache read / HBM peak)"] = round(64 * min(ctx, win) * 2 * d * 2 / us(rep_d, lat) / HBM_PEAK, 4)
                        if us(rep_p, lat):
                            pairs = sum(min(i + 1, win) for i in range(T))
                            share["latent attention prefill (4 d flops a visible key and head / bf16 matrix peak)"] = round(
                                4.0 * d * pairs * heads / us(rep_p, lat) / FLOP_PEAK["bf16"], 4)
                        if us(rep_p, "ilm_stream_update"):
                            share["stream_update prefill (stream read + written, branch and gate read, rows written / HBM peak)"] = round(
                                T * Hs * (4 + 4 + 2 + 2 + 2) / us(rep_p, "ilm_stream_update") / HBM_PEAK, 4)
                    if name == "bebuzen":
                        win, inner, N = 1024, 2 * Hs, 16
                        m1 = cfg["layers"][1]["mlp"]
                        E, top, ff = m1["router"]["experts"], m1["router"]["top"], m1["expert"]["ff"]
                        seen, pairs = min(ctx, win), sum(min(i + 1, win) for i in range(T))
                        for label, what in (("ilm_attn_headmix_mfma", "attention with kept first tokens"),
                                            ("ilm_attn_headmix_mfma (unmixed)", "differential attention (two maps as heads)"),
                                            ("ilm_attn_maps_mfma", "differential attention (two maps in one pass)")):
                            if us(rep_d, label):
                                share[f"{what} decode (window's cache read / HBM peak)"] = round(64 * seen * kvb / us(rep_d, label) / HBM_PEAK, 4)
                            if us(rep_p, label):
                                share[f"{what} prefill (4 d flops a visible key and head / bf16 matrix peak)"] = round(
                                    4.0 * d * pairs * heads / us(rep_p, label) / FLOP_PEAK["bf16"], 4)
                        if us(rep_d, "ilm_selective_scan"):
                            share["selective_scan decode (state read + written / HBM peak)"] = round(64 * 2 * inner * N * 4 / us(rep_d, "ilm_selective_scan") / HBM_PEAK, 4)
                            share["selective_scan prefill (7 flops a token, channel and state entry / float32 vector peak)"] = round(
                                7.0 * T * inner * N / us(rep_p, "ilm_selective_scan") / FLOP_PEAK["fp32"], 4)
                        up, dn = "ilm_moe_gemm (up)", "ilm_moe_gemm (down)"
                        if us(rep_p, up):
                            share["experts' up product prefill (flops / bf16 matrix peak)"] = round(2.0 * T * top * ff * Hs / us(rep_p, up) / FLOP_PEAK["bf16"], 4)
                            share["experts' down product prefill (flops / bf16 matrix peak)"] = round(2.0 * T * top * ff * Hs / us(rep_p, dn) / FLOP_PEAK["bf16"], 4)
                            hit = min(E, 64 * top)
                            share["experts' up product decode (weights of the experts hit read / HBM peak)"] = round(hit * ff * Hs * 2 / us(rep_d, up) / HBM_PEAK, 4)
                            share["experts' down product decode (weights of the experts hit read / HBM peak)"] = round(hit * ff * Hs * 2 / us(rep_d, dn) / HBM_PEAK, 4)
                        if us(rep_p, "ilm_stream_update"):
                            share["stream_update prefill (stream read + written, branch read, rows written / HBM peak)"] = round(
                                T * Hs * (4 + 4 + 2 + 2) / us(rep_p, "ilm_stream_update") / HBM_PEAK, 4)
                    if name == "moputar":
                        chunk, n = 1024, cfg["streams"]
                        seen, pairs = (ctx - 1) % chunk + 1, sum(i % chunk + 1 for i in range(T))
                        C = 2 * (max(heads // 2, 1)) * d + heads * d       # convolved channels of a delta layer
                        Ca = heads * d + 2 * kv * d                        # ... of an attention layer with keys and values of its own
                        share["attention decode (own chunk's cache read / HBM peak)"] = round(64 * seen * kvb / us(rep_d, "ilm_attn_mfma") / HBM_PEAK, 4)
                        share["attention prefill (4 d flops a visible key and head / bf16 matrix peak)"] = round(
                            4.0 * d * pairs * heads / us(rep_p, "ilm_attn_tile") / FLOP_PEAK["bf16"], 4)
                        share["delta_step decode (state read + written / HBM peak)"] = round(64 * 2 * state / us(rep_d, "ilm_delta_step") / HBM_PEAK, 4)
                        share["delta_chunks prefill (6 dk dv flops a token and head / float32 vector peak)"] = round(
                            6.0 * T * heads * d * d / us(rep_p, "ilm_delta_chunks") / FLOP_PEAK["fp32"], 4)
                        share["hyper_update prefill (streams read + written, branch read, rows written / HBM peak)"] = round(
                            T * Hs * (4 * n + 4 * n + 2 + 2) / us(rep_p, "ilm_hyper_update") / HBM_PEAK, 4)
                        share["conv_delta_inputs prefill (rows read, float rows written / HBM peak)"] = round(
                            T * C * (2 + 4) / us(rep_p, "ilm_conv_delta_inputs") / HBM_PEAK, 4)
                        share["conv_norm_rope_kvwrite prefill (rows read and written, mean of both layer kinds / HBM peak)"] = round(
                            T * (Ca + heads * d) / 2 * (2 + 2) / us(rep_p, "ilm_conv_norm_rope_kvwrite") / HBM_PEAK, 4)
                    if name == "lizezen":
                        f = cfg["layers"][1]["mlp"]
                        E, top, ff = f["router"]["experts"], f["router"]["top"], f["expert"]["ff"]
                        real = top * E / (E + f["router"]["identity"])      # pairs a token that have matrices, on average
                        share["attention decode, both kinds (cache read / HBM peak)"] = round(64 * ctx * kvb / us(rep_d, "ilm_attn_mfma") / HBM_PEAK, 4)
                        share["attention prefill, both kinds (4 d flops a visible key and head / bf16 matrix peak)"] = round(
                            4.0 * T * T / 2 * heads * d / us(rep_p, "ilm_attn_tile") / FLOP_PEAK["bf16"], 4)
                        share["mlstm_step decode (state read + written / HBM peak)"] = round(64 * 2 * state / us(rep_d, "ilm_mlstm_step") / HBM_PEAK, 4)
                        share["mlstm_chunks prefill (4 dk dv flops a token and head / float32 vector peak)"] = round(
                            4.0 * T * heads * d * d / us(rep_p, "ilm_mlstm_chunks") / FLOP_PEAK["fp32"], 4)
                        share["dynamic tanh prefill (stream read + written, two branches read, rows written / HBM peak)"] = round(
                            T * Hs * (4 + 4 + 2 + 2 + 2) / us(rep_p, "ilm_add_rows (dynamic tanh)") / HBM_PEAK, 4)
                        share["qkv_norm_rope_kvwrite prefill (query and key rows read and written / HBM peak)"] = round(
                            T * (heads + 2 * kv) * d * (2 + 2) / us(rep_p, "ilm_qkv_norm_rope_kvwrite") / HBM_PEAK, 4)
                        gu, dn = "ilm_moe_gemm (gate/up)", "ilm_moe_gemm (down)"
                        share["experts' gate/up product prefill (flops / bf16 matrix peak)"] = round(2.0 * T * real * 2 * ff * Hs / us(rep_p, gu) / FLOP_PEAK["bf16"], 4)
                        share["experts' down product prefill (flops / bf16 matrix peak)"] = round(2.0 * T * real * ff * Hs / us(rep_p, dn) / FLOP_PEAK["bf16"], 4)
                        share["experts' gate/up product decode (all experts' weights read / HBM peak)"] = round(E * 2 * ff * Hs * 2 / us(rep_d, gu) / HBM_PEAK, 4)
                        share["experts' down product decode (all experts' weights read / HBM peak)"] = round(E * ff * Hs * 2 / us(rep_d, dn) / HBM_PEAK, 4)
                    if name == "minicpm4" and us(rep_p, "library_gemm"):
                        flops = 2.0 * T * Hs * ((heads + 2 * kv) * d + heads * d + 3 * cfg["intermediate_size"]) * layers
                        share["library products prefill, all of a step (flops / bf16 matrix peak)"] = round(
                            flops / (rep_p["library_gemm"]["total_ms"] * 1e-3 / 2) / FLOP_PEAK["bf16"], 4)
                    if name not in ("pugavik", "patadra", "bebuzen", "moputar", "lizezen") and us(rep_d, "ilm_decay_scan"):
                        share["decay_scan decode (state read + written / HBM peak)"] = round(64 * 2 * state / us(rep_d, "ilm_decay_scan") / HBM_PEAK, 4)
                        share["decay_scan prefill (4 dk dv flops a token and head / float32 vector peak)"] = round(
                            4.0 * T * heads * d * d / us(rep_p, "ilm_decay_scan") / FLOP_PEAK["fp32"], 4)
                    if name not in ("pugavik", "patadra", "bebuzen", "moputar", "lizezen") and us(rep_d, "ilm_attn_mfma"):
                        share["attention decode (cache read / HBM peak)"] = round(64 * ctx * kvb / us(rep_d, "ilm_attn_mfma") / HBM_PEAK, 4)
                    if name not in ("pugavik", "patadra", "bebuzen", "moputar", "lizezen") and us(rep_p, "ilm_attn_tile"):
                        share["attention prefill (4 d flops a visible key and head / bf16 matrix peak)"] = round(
                            4.0 * T * T / 2 * heads * d / us(rep_p, "ilm_attn_tile") / FLOP_PEAK["bf16"], 4)
                    if name == "pugavik":
                        win = 1024
                        hm = "ilm_attn_headmix_mfma" if "ilm_attn_headmix_mfma" in rep_d else "ilm_attn_headmix"
                        if us(rep_d, hm):
                            seen = min(ctx, win)
                            share["mixed-heads attention decode (window's cache read / HBM peak)"] = round(64 * seen * kvb / us(rep_d, hm) / HBM_PEAK, 4)
                            pairs = sum(min(i + 1, win) for i in range(T))
                            share["mixed-heads attention prefill (4 d flops a visible key and head / bf16 matrix peak)"] = round(
                                4.0 * d * pairs * heads / us(rep_p, hm) / FLOP_PEAK["bf16"], 4)
                        gstate = heads * (d // 2) * d * 4
                        if us(rep_d, "ilm_decay_scan"):
                            share["decay_scan (decay per channel) decode (state read + written / HBM peak)"] = round(64 * 2 * gstate / us(rep_d, "ilm_decay_scan") / HBM_PEAK, 4)
                            share["decay_scan (decay per channel) prefill (4 dk dv flops a token and head / float32 vector peak)"] = round(
                                4.0 * T * heads * (d // 2) * d / us(rep_p, "ilm_decay_scan") / FLOP_PEAK["fp32"], 4)
                        lat = "ilm_attn_headmix_mfma (unmixed)"   # (the latent layers' attention: one cached row of d entries a token, read as key and as value)
                        if us(rep_d, lat):
                            share["latent attention decode (cache read / HBM peak)"] = round(64 * ctx * 2 * d * 2 / us(rep_d, lat) / HBM_PEAK, 4)
                        if us(rep_p, lat):
                            share["latent attention prefill (4 d flops a visible key and head / bf16 matrix peak)"] = round(
                                4.0 * T * T / 2 * heads * d / us(rep_p, lat) / FLOP_PEAK["bf16"], 4)
                        if us(rep_p, "ilm_add_layernorm"):
                            share["add_layernorm prefill (stream read + written, two branches read, rows written / HBM peak)"] = round(
                                T * Hs * (4 + 4 + 2 + 2 + 2) / us(rep_p, "ilm_add_layernorm") / HBM_PEAK, 4)
                    if name == "minicpm4" and us(rep_p, "ilm_add_rmsnorm"):
                        share["add_rmsnorm prefill (stream read + written, branch read, rows written / HBM peak)"] = round(
                            T * Hs * (4 + 4 + 2 + 2) / us(rep_p, "ilm_add_rmsnorm") / HBM_PEAK, 4)
                    r["roofline_share"] = share
                del runner, cache
                torch.cuda.empty_cache()
            rec[name] = r
            del model
            torch.cuda.empty_cache()
        out["shapes"][str(width)] = rec
    return out


def measure(args, cfg, dtype, FULL_LAYERS, full):
    """One dtype's record; `full`: with the batch 1 / 32 / 64 points."""
    import torch
    from infinilm_amd.engine.loading import build_model, make_runner
    from infinilm_amd.engine.step import StepEntry
    from infinilm_amd.sampling import Sampler, SamplingParams
    from infinilm_amd.weights import fill_random_

    model = build_model(cfg, dtype, "cuda:0")
    fill_random_(model, seed=0, std=0.02, norm_init="one_plus")
    torch.cuda.synchronize()
    spec = model.spec
    H, V, L = spec.hidden_size, spec.vocab_size, len(spec.order)
    esize = 2 if dtype == "bfloat16" else 4
    dkey = "bf16" if dtype == "bfloat16" else "fp32"

    max_b = max(args.batch, 1 if (args.no_points or not full) else 64)
    ps = args.page_size
    pages_per_req = -(-(args.context + 1) // ps)
    num_pages = max(max_b * pages_per_req, -(-args.prefill_tokens // ps)) + 4
    runner = make_runner(model, num_pages=num_pages, page_size=ps, max_requests=max_b + 1,
                         enable_graph=not args.no_graph)
    cache = runner.cache
    for e in cache.k:
        cache.k[e].normal_(0, 1.0)
        cache.v[e].normal_(0, 1.0)
    sampler = Sampler(0)
    greedy = SamplingParams(top_k=1)
    gen = torch.Generator().manual_seed(7)

    # every tensor but the embedding table and the head: what the layers and the final norm read once a step
    outer = {model.embed.data_ptr(), model.head.data_ptr()}
    inner = [p.tensor for p in model.named_parameters().values() if p.tensor.data_ptr() not in outer]
    layer_weight_bytes = sum(t.numel() * t.element_size() for t in inner)
    head_bytes = model.head.numel() * model.head.element_size()

    def decode(batch: int, steps: int, warmup: int):
        ids = [f"d{batch}_{i}" for i in range(batch)]
        start = args.context - (steps + warmup)
        assert start > 0
        for rid in ids:
            cache.admit(rid)
            cache.reserve(rid, start)
            cache.commit(rid, start)   # the context's keys and values are the random fill
        toks = torch.randint(0, V, (batch,), generator=gen).tolist()

        def one(toks):
            logits = runner.step([StepEntry(rid, [t], [0]) for rid, t in zip(ids, toks)])
            return sampler.sample(logits, [(greedy, i, 0) for i in range(batch)])

        for _ in range(warmup):
            toks = one(toks)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(steps):
            toks = one(toks)
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        ctx_mean = args.context - steps / 2.0
        for rid in ids:
            cache.release(rid)
        ms = dt / steps * 1e3
        kv_bytes = batch * ctx_mean * cache.bytes_per_token()
        step_bytes = layer_weight_bytes + head_bytes + batch * H * esize + kv_bytes
        return {"tok_s": batch * steps / dt, "ms": ms, "bytes": step_bytes, "gbs": step_bytes / (dt / steps) / 1e9}

    def prefill():
        # one prompt of T tokens in one step, logits at its last place
        T = args.prefill_tokens
        prompt = torch.randint(0, V, (T,), generator=gen).tolist()
        times = []
        passes = 7 if dtype == "bfloat16" else 3
        for i in range(passes + 1):   # the first pass warms up (the library chooses its kernels there)
            rid = f"p{i}"
            cache.admit(rid)
            torch.cuda.synchronize()
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            e0.record()
            logits = runner.step([StepEntry(rid, prompt, [T - 1])])
            sampler.sample(logits, [(greedy, 0, 0)])
            e1.record()
            torch.cuda.synchronize()
            times.append(e0.elapsed_time(e1) * 1e-3)
            cache.release(rid)
        pt = sorted(times[1:])[len(times[1:]) // 2]   # the median
        mat_params = sum(t.numel() for t in inner if t.dim() == 2)
        flops = 2.0 * T * mat_params + 4.0 * T * T / 2.0 * cfg["num_attention_heads"] * cfg["head_dim"] * L + 2.0 * V * H
        return {"value": round(T / pt, 1), "tokens": T, "ms": round(pt * 1e3, 3), "frac": round(flops / pt / FLOP_PEAK[dkey], 4)}

    if args.prefill_only:
        return {"prefill": prefill()}
    main_pt = decode(args.batch, args.steps, args.warmup)
    record = {
        "metric": "decode tokens/s, MiniCPM4-8B shape, batch %d, context %d" % (args.batch, args.context),
        "value": round(main_pt["tok_s"], 2), "unit": "tokens/s", "n_gpus": 1, "steps": args.steps,
        "warmup": args.warmup, "ms_per_step": round(main_pt["ms"], 4), "higher_is_better": True, "scaling": "weak",
        "vs_baseline": None, "dtype": dkey, "data": "synthetic: random weights, random token ids, random-filled cache",
        "config": {"model": "MiniCPM4-8B shape (random weights)", "global_batch": args.batch, "seq_len": args.context,
                   "parallelism": "single-gpu", "num_hidden_layers": FULL_LAYERS, "layers_run": L, "hidden_size": H,
                   "num_attention_heads": 32, "num_key_value_heads": 2, "head_dim": 128, "intermediate_size": 16384,
                   "vocab_size": V, "rope": "longrope, 64 factors", "tied_head": False, "page_size": ps,
                   "prefill_tokens": args.prefill_tokens},
        "roofline": {"bound": "hbm", "achieved": round(main_pt["gbs"], 1), "peak": HBM_PEAK / 1e9, "unit": "GB/s",
                     "frac": round(main_pt["gbs"] * 1e9 / HBM_PEAK, 4)},
    }
    if not args.no_points:
        k = max(8, args.steps // 2)
        if full:
            pts = {b: decode(b, k, args.warmup) for b in (1, 32, 64)}
            record["points"] = {f"decode_b{b}": round(p["tok_s"], 2) for b, p in pts.items()}
            # the same pricing as `roofline` for each point: bytes the step has to read / its time / the HBM peak
            record["points_frac"] = {f"decode_b{b}": round(p["gbs"] * 1e9 / HBM_PEAK, 4) for b, p in pts.items()}
        record["prefill"] = prefill()
    del runner, cache, model
    return record


if __name__ == "__main__":
    sys.exit(main())
