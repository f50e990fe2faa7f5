"""`bench.py --nagezen`: prefill and decode throughput of the multi-stream hybrid decoder (Nagezen: several residual streams, retention,
gated linear attention, the difference of two softmax maps over a window with kept first tokens, clamped gated feed-forwards) at layer
sizes that resemble a real model's, beside the repository's closest model, the looped pre-norm hybrid decoder (Piladra: selective scan
where this one has retention or gated linear attention, windowed attention with a sink where it has two maps, dense gated
feed-forwards) of equal width, depth, head count, head size, window and feed-forward width, and each new kernel alone against its
roofline beside its like kernel.

Random weights, synthetic token ids, bf16.  One JSON line on stdout; does not touch bench.py's default workload.

    python bench.py --nagezen [--nagezen-args --sizes s m --prompt 2048 --batch 32 --steps 20 --no-twin --no-kernels]
"""
from __future__ import annotations

import argparse
import json

import torch

from tools.hybrid_bench import HBM_TBS, MFMA_TFLOPS, VALU_TFLOPS, _time_us, run_engine

# name -> (width, layers: R = retention, G = gated linear attention, A = two-map attention; heads, key heads of the attention, head size
#          (values; q and k of R and G; two maps of half of it in A), decay rank of G, window, kept first tokens, streams, ff, vocab)
SIZES = {
    "s": (1024, "GRAR", 8, 2, 128, 16, 1024, 64, 4, 2048, 32000),
    "m": (2048, "GRAGRA", 16, 4, 128, 16, 2048, 64, 4, 4096, 32000),
}


def nagezen_json(name: str) -> dict:
    W, order, H, G, D, rank, window, keep, streams, ff, V = SIZES[name]
    mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
    layers = []
    for c in order:
        if c == "R":
            decay = [1.0 - 2.0 ** (-5.0 - 7.0 * h / max(H - 1, 1)) for h in range(H)]
            layers.append({"type": "retention", "mixer": {"heads": H, "dim": D, "vdim": D, "decay": decay, "rot": {"base": 1e4, "dims": D}}, "mlp": mlp})
        elif c == "G":
            layers.append({"type": "gla", "mixer": {"heads": H, "dim": D, "vdim": D, "tau": 16.0}, "mlp": mlp})
        else:
            rot = {"base": 1e6, "dims": D // 2, "scaling": {"factor": 4.0, "fast": 32.0, "slow": 1.0, "original": 8192}}
            layers.append({"type": "attention", "mlp": mlp,
                           "mixer": {"heads": H, "kv_heads": G, "dim": D // 2, "vdim": D, "scale": (D // 2) ** -0.5, "diff": 0.4,
                                     "mask": {"size": window, "keep_first": keep}, "rot": rot}})
    return {"architecture": "Nagezen", "layers": layers, "norm": {"eps": 1e-5}, "streams": streams, "logit_scale": 1.0, "vocab": V, "width": W}


def twin_json(name: str) -> dict:
    W, order, H, G, D, rank, window, keep, streams, ff, V = SIZES[name]
    dense = {"kind": "dense", "ff": ff}
    layers = []
    for c in order:
        if c == "A":
            rot = {"base": 1e6, "dims": D, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 8192}}
            layers.append({"type": "attention", "mlp": dense,
                           "mixer": {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "mask": {"size": window}, "rot": rot}})
        else:
            layers.append({"type": "mamba1", "mixer": {"inner": 2 * W, "state": 16, "dt_rank": W // 16, "conv": 4}, "mlp": dense})
    return {"architecture": "Piladra", "layers": layers, "norm": {"eps": 1e-6, "groups": 1}, "residual_mult": 1.0, "vocab": V, "width": W}


def _entry(us: float, flops: float, byts: float, flop_peak: float) -> dict:
    return {"us": round(us, 1), "tflops": round(flops / us / 1e6, 2), "tb_s": round(byts / us / 1e6, 3),
            "of_roofline": round(max(flops / us / 1e6 / flop_peak, byts / us / 1e6 / HBM_TBS), 4)}


def kernel_rooflines(name: str, prompt: int, batch: int, device, chunk: int = 0) -> dict:
    """Each new kernel alone at the size's shapes, beside its like kernel of the other hybrid decoders: microseconds and the share
    of the roofline that bounds it (matrix cores for a prompt portion's attention products, the fp32 rate -- 157 TFLOP/s on the vector
    units and on the matrix cores alike -- for the recurrences, HBM for everything a decode step streams and for the row kernels)."""
    from mini_sglang_amd import mixops
    from mini_sglang_amd.attention import MixAttnBackend

    W, order, H, G, D, rank, window, keep, streams, ff, V = SIZES[name]
    bf, f32 = torch.bfloat16, torch.float32
    out = {}

    def rnd(*shape, dtype=bf, scale=1.0):
        return (torch.randn(shape, device=device, dtype=f32) * scale).to(dtype)

    def i32(v):
        return torch.tensor(v, dtype=torch.int32, device=device)

    def chunk_list(q_len, reqs, size):
        if q_len < 2 * size:
            return None
        n = -(-q_len // size)
        items = i32([[b, c * size, min((c + 1) * size, q_len)] for b in range(reqs) for c in range(n)]).view(-1)
        return items, i32([b * n for b in range(reqs + 1)]), reqs * n

    for phase, T, reqs, ctx in (("prefill", prompt, 1, prompt), ("prefill x 4", 4 * prompt, 4, prompt), ("decode", batch, batch, prompt)):
        q_len = T // reqs
        cu, seq, rows = i32([i * q_len for i in range(reqs + 1)]), i32([ctx] * reqs), i32(list(range(reqs)))
        slots = reqs * ctx
        table = torch.arange(slots, dtype=torch.int32, device=device).view(reqs, ctx)
        first = ctx - q_len
        pos = i32([first + i for _ in range(reqs) for i in range(q_len)])
        # --- attention: two maps of half the head size (like: one map of the whole head size), all keys visible and half the window
        d = D // 2
        q2, q1 = rnd(T, H * D, dtype=f32, scale=0.1), rnd(T, H * D, dtype=f32, scale=0.1)
        kc, vc = rnd(slots, G * D), rnd(slots, G * D)
        gate = rnd(T, 2 * H * D)[:, H * D:]
        lam, sink = torch.full((1,), 0.4, device=device), torch.zeros(H, device=device)
        o = torch.empty(T, H * D, dtype=bf, device=device)
        for label, win, kf in (("", 0, 0), (" (window %d)" % (window // 2), window // 2, keep)):
            keys = lambda p: min(p + 1, win + min(kf, max(p + 1 - win, 0))) if win else p + 1  # noqa: E731
            read = reqs * (min(ctx, win + kf + q_len) if win else ctx)
            sp = mixops.sink_attn_splits(reqs, T, H, G, win, ctx, kf) if q_len <= 16 else 1
            pairs = reqs * sum(keys(first + i) for i in range(q_len))
            us = _time_us(lambda: mixops.diff_attn(o, q2, kc, vc, table, rows, seq, cu, reqs, H, G, d, D, d ** -0.5, win, kf, lam, 0.6, 1e-5, gate=gate, splits=sp))
            # a pair costs 2 x 2 d for the scores of its maps and 2 x 2 D for their two products with the values
            out[f"{phase}.diff_attn{label}"] = _entry(us, pairs * H * (4.0 * d + 4.0 * D), read * 2 * G * D * 2 + T * H * D * (4 + 2 + 2), MFMA_TFLOPS)
            us = _time_us(lambda: mixops.sink_attn(o, q1, kc, vc, table, rows, seq, cu, reqs, H, G, D, D, D ** -0.5, win, sink, splits=sp, keep=kf))
            out[f"{phase}.sink_attn{label} (like)"] = _entry(us, 4.0 * pairs * H * D, read * 2 * G * D * 2 + T * H * D * (4 + 2), MFMA_TFLOPS)
        # --- q / k preparation with a weighted norm before the rotation (like: without it, same kernel)
        proj, bias = rnd(T, (2 * H + 2 * G) * D), torch.zeros((H + 2 * G) * D, device=device)
        ang = torch.rand(ctx, d, device=device)
        nw = (rnd(d), rnd(d))
        loc = table[:, first:].reshape(-1).contiguous()
        us = _time_us(lambda: mixops.qk_prep(proj, bias, kc, vc, loc, pos, ang, 1e-5, 2 * H, 2 * G, d, D, interleaved=False, unit=False, norm_w=nw, value_heads=G))
        byts = T * ((H + 2 * G) * D * 2 + H * D * 4 + 2 * G * D * 2)
        out[f"{phase}.qk_prep (weighted norm)"] = _entry(us, 0.0, byts, VALU_TFLOPS)
        ang2 = torch.rand(ctx, D, device=device)
        us = _time_us(lambda: mixops.qk_prep(proj, None, kc, vc, loc, pos, ang2, 1e-5, H, G, D, D, interleaved=False, unit=False, unit_v=True))
        out[f"{phase}.qk_prep (like)"] = _entry(us, 0.0, byts, VALU_TFLOPS)
        # --- recurrences with head norm and gate (like: the lightning recurrence and its gated norm; the channel-wise delta rule)
        pr = rnd(T, 4 * H * D, scale=0.5)
        cols = [pr[:, i * H * D: (i + 1) * H * D] for i in range(4)]
        state = torch.zeros(reqs, H, D, D, device=device)
        decay = torch.tensor([1.0 - 2.0 ** (-5.0 - 7.0 * h / max(H - 1, 1)) for h in range(H)], device=device)
        tab = torch.rand(ctx, D, device=device)
        byts = 2 * reqs * H * D * D * 4 + T * H * D * 2 * 5
        flops = 4.0 * T * H * D * D  # the update and the read of the state; what a piece does besides is the kernel's own choice
        ch = chunk_list(q_len, reqs, chunk or MixAttnBackend.decay_chunk(T, H))
        us = _time_us(lambda: mixops.decay_attn(*cols, state, cu, seq, rows, reqs, 1e-5, decay=decay, k_scale=D ** -0.5, cos_sin=tab, positions=pos, chunks=ch))
        out[f"{phase}.decay_attn (per head)"] = _entry(us, flops, byts, VALU_TFLOPS)
        z, zb, w = rnd(T, H * D), torch.ones(H * D, device=device), rnd(D)
        us = _time_us(lambda: mixops.decay_attn(*cols, state, cu, seq, rows, reqs, 1e-5, z=z, z_bias=zb, tau=16.0, q_scale=D ** -0.5, weight=w, chunks=ch))
        out[f"{phase}.decay_attn (per channel)"] = _entry(us, flops, byts + T * H * D * 2, VALU_TFLOPS)
        o32, gw = torch.empty(T, H * D, device=device), rnd(H * D)
        lch = chunk_list(q_len, reqs, MixAttnBackend.RECURRENT_CHUNK)

        def lightning():
            mixops.lightning(o32, pr, state, decay, cu, seq, rows, reqs, chunks=lch)
            mixops.gated_norm(o32, cols[3], gw, 1e-5)

        out[f"{phase}.lightning + gated_norm (like)"] = _entry(_time_us(lightning), flops, byts, VALU_TFLOPS)
        # --- residual streams (like: sum of one part + grouped norm, one stream)
        xs, y, h = rnd(T, streams, W, dtype=f32), rnd(T, W), torch.empty(T, W, dtype=bf, device=device)
        mix, vec = torch.eye(streams, device=device), torch.full((streams,), 1.0 / streams, device=device)
        sq = (rnd(W), rnd(W), torch.full((1,), 0.5, device=device))
        us = _time_us(lambda: mixops.stream_norm(xs, streams, y=y, mix=mix, out_w=vec, x_out=xs, read=vec, norm=sq, h_out=h))
        out[f"{phase}.stream_norm ({streams} streams)"] = _entry(us, 0.0, T * W * (8 * streams + 2 + 2), VALU_TFLOPS)
        x1, x2 = rnd(T, W, dtype=f32), torch.empty(T, W, device=device)
        us = _time_us(lambda: mixops.norm_conv(x1, sq[0], 1e-6, 1, h, parts=(y,), x_out=x2))
        out[f"{phase}.norm_conv (like)"] = _entry(us, 0.0, T * W * (4 + 2 + 4 + 2), VALU_TFLOPS)
        # --- clamped gate (like: SiLU gate)
        gu = rnd(T, 2 * ff)
        us = _time_us(lambda: mixops.clamp_gate(gu, 7.0, 1.702))
        out[f"{phase}.clamp_gate"] = _entry(us, 0.0, T * ff * 6, VALU_TFLOPS)
        us = _time_us(lambda: mixops.silu_mul(gu))
        out[f"{phase}.silu_mul (like)"] = _entry(us, 0.0, T * ff * 6, VALU_TFLOPS)
        print(f"[nagezen bench] {name} {phase}: " + json.dumps({k.split(".", 1)[1]: (v["us"], v["of_roofline"]) for k, v in out.items() if k.startswith(phase + ".")}),
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
    ap.add_argument("--chunk", type=int, default=0, help="piece size of long portions in the recurrences' own measurement")
    args = ap.parse_args(argv)
    from mini_sglang_amd.hybrid import nagezen_config, piladra_config

    device = torch.device("cuda:0")
    torch.cuda.set_device(device)
    report = {"metric": "nagezen_decoder_throughput", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1,
              "prompt": args.prompt, "batch": args.batch, "steps": args.steps, "sizes": {}}
    keys = ("width", "layers", "heads", "kv_heads", "head", "decay_rank", "window", "keep_first", "streams", "ff", "vocab")

    def config_of(name):
        W, order, rank = SIZES[name][0], SIZES[name][1], SIZES[name][5]
        return nagezen_config(nagezen_json(name), {f"l{i}.mix.a1": (rank, W) for i, c in enumerate(order) if c == "G"})

    if not args.no_engine:  # the process's first engine pays for library loading and allocator growth: one untimed pass
        run_engine(config_of(args.sizes[0]), args.prompt, args.batch, 1, 1, device)
    for name in args.sizes:
        entry = {"shape": dict(zip(keys, SIZES[name]))}
        if not args.no_engine:
            entry["nagezen"] = run_engine(config_of(name), args.prompt, args.batch, args.steps, args.warmup, device)
            print(f"[nagezen bench] {name}: " + json.dumps(entry["nagezen"]), flush=True)
            if not args.no_twin:
                entry["pre_norm_hybrid"] = run_engine(piladra_config(twin_json(name)), args.prompt, args.batch, args.steps, args.warmup, device)
                print(f"[nagezen bench] {name} twin: " + json.dumps(entry["pre_norm_hybrid"]), flush=True)
        if not args.no_kernels:
            entry["kernels"] = kernel_rooflines(name, args.prompt, args.batch, device, args.chunk)
        report["sizes"][name] = entry
    print(json.dumps(report))


if __name__ == "__main__":
    main()
