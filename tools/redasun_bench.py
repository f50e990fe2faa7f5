"""`bench.py --redasun`: prefill and decode throughput of the looped sandwich-norm decoder (Redasun: a centred norm into and out of every
sublayer, the difference of two softmax maps over all earlier keys, GELU-gated feed-forwards, group-limited sigmoid router with a shared
expert, a loop that reads the embedding in every pass) at layer sizes that resemble a real model's, beside the repository's closest model,
the looped pre-norm hybrid decoder (Piladra: one softmax map with a sink, SiLU-gated feed-forwards, input-weighted experts with a shared
expert, a loop with a learned step vector) of equal width, depth, loop, head count, head size, experts and feed-forward widths, and each
kernel alone against its roofline beside its like kernel.

Random weights, synthetic token ids, bf16.  One JSON line on stdout; does not touch bench.py's default workload.

    python bench.py --redasun [--redasun-args --sizes s m --prompt 2048 --batch 32 --steps 20 --no-twin --no-kernels]
"""
from __future__ import annotations

import argparse
import json

import torch

from tools.hybrid_bench import HBM_TBS, MFMA_TFLOPS, VALU_TFLOPS, _time_us, run_engine

# name -> (width, feed-forwards: D = dense, M = mixture; heads, key heads, head size (values; two maps of half of it for keys), loop, dense ff,
#          experts, chosen, groups, kept groups, expert ff, shared ff, vocab)
SIZES = {
    "s": (1024, "DMDM", 8, 2, 128, (1, 3, 2), 2048, 16, 2, 4, 2, 512, 1024, 32000),
    "m": (2048, "DMMDMM", 16, 4, 128, (1, 4, 2), 4096, 64, 6, 8, 4, 512, 1024, 32000),
}
KEYS = ("width", "feed_forwards", "heads", "kv_heads", "head", "loop", "ff", "experts", "top", "groups", "keep", "expert_ff", "shared_ff", "vocab")


def redasun_json(name: str) -> dict:
    W, order, H, G, D, loop, ff, E, top, groups, keep, eff, sff, V = SIZES[name]
    moe = {"kind": "moe", "expert": {"ff": eff}, "shared": {"ff": sff},
           "router": {"experts": E, "top": top, "scale": 2.0, "groups": {"count": groups, "keep": keep}}}
    mixer = {"heads": H, "kv_heads": G, "dim": D // 2, "vdim": D, "scale": (D // 2) ** -0.5, "diff": 0.4, "rot": {"base": 1e5, "dims": D // 2}}
    layers = [{"type": "attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if c == "D" else moe} for c in order]
    return {"architecture": "Redasun", "layers": layers, "norm": {"eps": 1e-5}, "embedding": {"scale": W ** 0.5},
            "loop": dict(zip(("start", "stop", "times"), loop)), "vocab": V, "width": W}


def twin_json(name: str) -> dict:
    W, order, H, G, D, loop, ff, E, top, groups, keep, eff, sff, V = SIZES[name]
    moe = {"kind": "moe", "expert": {"ff": eff}, "shared": {"ff": sff}, "router": {"experts": E, "top": top}}
    mixer = {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "rot": {"base": 1e5, "dims": D}}
    layers = [{"type": "attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if c == "D" else moe} for c in order]
    return {"architecture": "Piladra", "layers": layers, "norm": {"eps": 1e-5, "groups": 1}, "residual_mult": 1.0,
            "loop": dict(zip(("start", "stop", "times"), loop)), "vocab": V, "width": W}


def _entry(us: float, flops: float, byts: float, flop_peak: float) -> dict:
    return {"us": round(us, 1), "tflops": round(flops / us / 1e6, 2), "tb_s": round(byts / us / 1e6, 3),
            "of_roofline": round(max(flops / us / 1e6 / flop_peak, byts / us / 1e6 / HBM_TBS), 4)}


def kernel_rooflines(name: str, prompt: int, batch: int, device) -> dict:
    """Each kernel of the design alone at the size's shapes, beside its like kernel of the other hybrid decoders: microseconds and the share
    of the roofline that bounds it (matrix cores for a prompt portion's products, HBM for what a decode step streams and for row kernels)."""
    from mini_sglang_amd import mixops

    W, order, H, G, D, loop, ff, E, top, groups, keep, eff, sff, V = SIZES[name]
    bf, f32 = torch.bfloat16, torch.float32
    out = {}

    def rnd(*shape, dtype=bf, scale=1.0):
        return (torch.randn(shape, device=device, dtype=f32) * scale).to(dtype)

    def i32(v):
        return torch.tensor(v, dtype=torch.int32, device=device)

    for phase, T, reqs, ctx in (("prefill", prompt, 1, prompt), ("prefill x 4", 4 * prompt, 4, prompt), ("decode", batch, batch, prompt)):
        q_len = T // reqs
        cu, seq, rows = i32([i * q_len for i in range(reqs + 1)]), i32([ctx] * reqs), i32(list(range(reqs)))
        slots = reqs * ctx
        table = torch.arange(slots, dtype=torch.int32, device=device).view(reqs, ctx)
        first = ctx - q_len
        pos = i32([first + i for _ in range(reqs) for i in range(q_len)])

        def put(label, fn, flops, byts, peak=MFMA_TFLOPS):
            out[f"{phase}.{label}"] = _entry(_time_us(fn), flops, byts, peak)

        # --- attention: two maps of half the head size (like: one map of the whole head size, same cache bytes)
        d = D // 2
        q2, q1 = rnd(T, H * D, dtype=f32, scale=0.1), rnd(T, H * D, dtype=f32, scale=0.1)
        kc, vc = rnd(slots, G * D), rnd(slots, G * D)
        lam, sink = torch.full((1,), 0.4, device=device), torch.zeros(H, device=device)
        o = torch.empty(T, H * D, dtype=bf, device=device)
        sp = mixops.sink_attn_splits(reqs, T, H, G, 0, ctx) if q_len <= 16 else 1
        pairs = reqs * sum(first + i + 1 for i in range(q_len))
        # a pair costs 2 x 2 d for the scores of its maps and 2 x 2 D for their two products with the values
        put("diff_attn", lambda: mixops.diff_attn(o, q2, kc, vc, table, rows, seq, cu, reqs, H, G, d, D, d ** -0.5, 0, 0, lam, 0.6, 1e-5, splits=sp),
            pairs * H * (4.0 * d + 4.0 * D), slots * 2 * G * D * 2 + T * H * D * (4 + 2))
        put("sink_attn (like)", lambda: mixops.sink_attn(o, q1, kc, vc, table, rows, seq, cu, reqs, H, G, D, D, D ** -0.5, 0, sink, splits=sp),
            4.0 * pairs * H * D, slots * 2 * G * D * 2 + T * H * D * (4 + 2))
        # --- q / k preparation with a weighted norm per map row (like: one row per head, no norm, unit values)
        proj, loc = rnd(T, (H + 2 * G) * D), table[:, first:].reshape(-1).contiguous()
        ang, ang2, nw = torch.rand(ctx, d, device=device), torch.rand(ctx, D, device=device), (rnd(d), rnd(d))
        byts = T * ((H + 2 * G) * D * 2 + H * D * 4 + 2 * G * D * 2)
        put("qk_prep (weighted norm)", lambda: mixops.qk_prep(proj, None, kc, vc, loc, pos, ang, 1e-5, 2 * H, 2 * G, d, D, interleaved=False, unit=False,
                                                              norm_w=nw, value_heads=G), 0.0, byts)
        put("qk_prep (like)", lambda: mixops.qk_prep(proj, None, kc, vc, loc, pos, ang2, 1e-5, H, G, D, D, interleaved=False, unit=False, unit_v=True), 0.0, byts)
        # --- residual sum and norms (like: one norm in front of the sublayer, none behind it)
        x1, x2, y, h = rnd(T, W, dtype=f32), torch.empty(T, W, device=device), rnd(T, W), torch.empty(T, W, dtype=bf, device=device)
        w1, w2 = rnd(W), rnd(W)
        jn = dict(dtype=bf, centre=True, w_in=w1, x_out=x2)
        put("join_norm (one part)", lambda: mixops.join_norm(x1, 1e-5, y=y, w_out=w2, h_out=h, **jn), 0.0, T * W * (4 + 2 + 4 + 2))
        put("norm_conv (one part, like)", lambda: mixops.norm_conv(x1, w2, 1e-5, 1, h, parts=(y,), x_out=x2), 0.0, T * W * (4 + 2 + 4 + 2))
        yk, gw = rnd(T, top, W), torch.rand(T, top, device=device)
        put("join_norm (experts + shared)", lambda: mixops.join_norm(x1, 1e-5, y=yk, gate=gw, y2=y, w_out=w2, h_out=h, **jn), 0.0, T * W * (4 + 2 * top + 2 + 4 + 2))
        put("norm_conv (experts + shared, like)", lambda: mixops.norm_conv(x1, w2, 1e-5, 1, h, parts=(yk, y), x_out=x2), 0.0, T * W * (4 + 2 * top + 2 + 4 + 2))
        wide = torch.empty(T, 2 * W, dtype=bf, device=device)
        put("join_norm (stream as product rows)", lambda: mixops.join_norm(x1, 1e-5, y=y, raw=(wide[:, :W],), **jn), 0.0, T * W * (4 + 2 + 4 + 2))
        # --- the product that opens a pass, fp32 result (like: the same product with a 16-bit result)
        win = rnd(W, 2 * W, scale=W ** -0.5)
        put("loop product (fp32 result)", lambda: mixops.linear(wide, win, out=x2), 4.0 * T * W * W, W * W * 4 + T * W * (4 + 4))
        put("loop product (16-bit result, like)", lambda: mixops.linear(wide, win, out=h), 4.0 * T * W * W, W * W * 4 + T * W * (4 + 2))
        # --- router (like: largest logits, sigmoid weights; in short steps expert inputs scaled in the same launch)
        router, corr = rnd(E, W, scale=W ** -0.5), rnd(E, scale=0.1)
        rule = (top, groups, keep, True, 2, 2.0)
        if T <= 128:
            byts = T * W * (4 + 2 + 4 + 2) + E * W * 2
            put("join_norm + choice", lambda: mixops.join_norm(x1, 1e-5, y=y, w_out=w2, h_out=h, route=(router, corr) + rule, **jn), 0.0, byts)

            def like():
                mixops.norm_conv(x1, w2, 1e-5, 1, h, parts=(y,), x_out=x2)
                mixops.route_scale(h, router, top)

            put("norm_conv, route_scale (like)", like, 0.0, byts + T * top * W * 2)
        else:
            byts = T * W * 2 + E * W * 2 + T * E * 8
            put("route", lambda: mixops.route(h, router, corr, top, groups, keep, sigmoid=True, group_best=2, scale=2.0), 2.0 * T * W * E, byts)

            put("route_sigmoid (like)", lambda: mixops.route_sigmoid(h, router, top), 2.0 * T * W * E, byts)
        # --- gated activation (like: the clamped gate)
        gu = rnd(T, 2 * ff)
        put("gate_mul (gelu)", lambda: mixops.gate_mul(gu, mixops.GATE_MUL_GELU_TANH), 0.0, T * ff * 6)
        put("clamp_gate (like)", lambda: mixops.clamp_gate(gu, 7.0, 1.702), 0.0, T * ff * 6)
        print(f"[redasun bench] {name} {phase}: " + json.dumps({k.split(".", 1)[1]: (v["us"], v["of_roofline"]) for k, v in out.items() if k.startswith(phase + ".")}),
              flush=True)
    return out


def main(argv=None) -> None:
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", nargs="*", default=["s", "m"], choices=sorted(SIZES))
    ap.add_argument("--prompt", type=int, default=2048)
    ap.add_argument("--batch", type=int, default=32)
    ap.add_argument("--steps", type=int, default=20)
    ap.add_argument("--warmup", type=int, default=3)
    ap.add_argument("--no-twin", action="store_true", help="skip the looped pre-norm hybrid decoder of equal size")
    ap.add_argument("--no-kernels", action="store_true")
    ap.add_argument("--no-engine", action="store_true", help="kernel rooflines only")
    args = ap.parse_args(argv)
    from mini_sglang_amd.hybrid import piladra_config, redasun_config

    device = torch.device("cuda:0")
    torch.cuda.set_device(device)
    report = {"metric": "redasun_decoder_throughput", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1,
              "prompt": args.prompt, "batch": args.batch, "steps": args.steps, "sizes": {}}
    if not args.no_engine:  # the process's first engine pays for library loading and allocator growth: one untimed pass
        run_engine(redasun_config(redasun_json(args.sizes[0])), args.prompt, args.batch, 1, 1, device)
    for name in args.sizes:
        entry = {"shape": dict(zip(KEYS, SIZES[name]))}
        if not args.no_engine:
            entry["redasun"] = run_engine(redasun_config(redasun_json(name)), args.prompt, args.batch, args.steps, args.warmup, device)
            print(f"[redasun bench] {name}: " + json.dumps(entry["redasun"]), flush=True)
            if not args.no_twin:
                entry["pre_norm_hybrid"] = run_engine(piladra_config(twin_json(name)), args.prompt, args.batch, args.steps, args.warmup, device)
                print(f"[redasun bench] {name} twin: " + json.dumps(entry["pre_norm_hybrid"]), flush=True)
        if not args.no_kernels:
            entry["kernels"] = kernel_rooflines(name, args.prompt, args.batch, device)
        report["sizes"][name] = entry
    print(json.dumps(report))


if __name__ == "__main__":
    main()
