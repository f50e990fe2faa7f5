"""The looped sandwich-norm decoder (Redasun: a centred norm into and out of every sublayer, the difference of two softmax maps over all
earlier keys, GELU-gated feed-forwards, group-limited sigmoid router with a shared expert, a loop that reads the embedding in every pass)
on the GPU against the plain restatement in tests/redasun_oracle.py: small configurations and random weights made here, the engine's own
step function, cache and kernels on one side, whole-sequence float64 arithmetic on the other.

fp32 engines are held to 2e-4 of the largest reference value (the sharp test); bf16 engines to the rounding of a 16-bit product chain, with
corrections spaced so widely that a rounded router picks the same experts.  Where random weights would hide a fault the inputs are built
so that it shows: one key far back whose score stands far above all others, choice scores that are all negative, groups whose best expert
and whose best pair disagree, rows with a mean a thousand times their deviation.
"""
from __future__ import annotations

import json
import math

import pytest
import torch

import redasun_oracle as O
from test_gpu_hybrid import alone, rel, replay, tokens_of

pytestmark = pytest.mark.gpu

FP32_TOL = 2e-4
BF16_TOL = 6e-2


# ----------------------------------------------------------------------------------------- configurations
def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=8, top=3, ff=20, count=4, keep=2, scale=1.3, shared=24):
    r = {"experts": experts, "top": top, "scale": scale}
    if count:
        r["groups"] = {"count": count, "keep": keep}
    m = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def att(heads=6, kv_heads=2, dim=12, vdim=20, dims=8, base=500.0, scale=0.3, diff=0.35, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if dims:
        m["rot"] = {"base": base, "dims": dims}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def config(layers, width=48, vocab=80, eps=1e-5, embed=2.5, loop=None):
    c = {"architecture": "Redasun", "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": embed}, "vocab": vocab, "width": width}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


FULL = config([att(mlp=dense()), att(heads=3, kv_heads=3, dim=8, vdim=8, dims=4, diff=0.1, mlp=moe()),
               att(heads=4, kv_heads=1, dim=16, vdim=40, dims=16, base=77.0, mlp=dense(ff=40)), att(dims=0, mlp=None)], loop=(1, 3, 2))


# ----------------------------------------------------------------------------------------- harness
_ENGINES: dict = {}


def engine_for(cfg_json, dtype, max_tokens=512, rows=4, page_size=16, graphs=None, seed=5, spaced=False):
    """(engine, checkpoint-named weights on the host) for a configuration; engines are kept for the session.  spaced: the router's
    corrections lie 1.5 apart in a shuffled order (scores lie in (0, 1): no rounding changes a choice)."""
    from mini_sglang_amd.engine import Engine, EngineConfig
    from mini_sglang_amd.hybrid import redasun_config

    key = (json.dumps(cfg_json, sort_keys=True), dtype, max_tokens, rows, page_size, tuple(graphs or ()), seed, spaced)
    if key not in _ENGINES:
        pages = max_tokens // page_size
        eng = Engine(EngineConfig(model=redasun_config(cfg_json), dtype=dtype, max_running_req=rows, page_size=page_size,
                                  num_page_override=pages, max_seq_len_override=pages * page_size, cuda_graph_bs=list(graphs or []),
                                  gemm_tune="off", refine_in_graph=False, seed=seed), torch.device("cuda:0"))
        state = eng.model.export_state()
        if spaced:
            g = torch.Generator().manual_seed(seed)
            for name, t in state.items():
                if name.endswith("correction"):
                    state[name] = (1.5 * (torch.randperm(t.numel(), generator=g) - t.numel() // 2)).to(t.dtype)
            eng.model.load_state(state)
        _ENGINES[key] = (eng, state)
    return _ENGINES[key]


def check(eng_state, cfg_json, steps, seqs, tol):
    """Every position of every request within `tol` of the restatement."""
    eng, state = eng_state
    got = replay(eng, steps)
    for rid, toks in seqs.items():
        ref = O.forward(cfg_json, state, toks)[0]
        assert got[rid].shape == ref.shape
        per = (got[rid] - ref).abs().amax(1) / ref.abs().max()
        bad = (per > tol).nonzero().flatten().tolist()
        assert not bad, f"request {rid}: {len(bad)} of {len(toks)} positions above {tol} (worst {float(per.max()):.3e}, first at {bad[0]})"
    return got


@pytest.fixture(scope="module")
def dev():
    return torch.device("cuda:0")


# ----------------------------------------------------------------------------------------- each mechanism alone
@pytest.mark.parametrize("layer", [
    att(), att(heads=3, kv_heads=3, dim=10, vdim=6, dims=10), att(heads=6, kv_heads=2, dim=8, vdim=72, dims=0), att(heads=1, kv_heads=1, dim=40, vdim=8, dims=2),
    att(heads=34, kv_heads=1, dim=8, vdim=8, dims=4), att(dims=10, base=3e6, diff=0.9), att(diff=0.0, scale=2.0), att(heads=2, kv_heads=1, dim=140, vdim=33, dims=64),
    att(heads=2, kv_heads=2, dim=9, vdim=264, dims=6), att(heads=1, kv_heads=1, dim=1, vdim=1, dims=0),
], ids=["grouped", "ungrouped", "wide-v-no-rotation", "one-head", "34-per-key-head", "all-rotated", "no-constant", "keys-140", "values-264", "ones"])
def test_attention_alone_fp32(layer):
    cfg = config([layer])
    toks = tokens_of(70, cfg["vocab"], 1)
    check(engine_for(cfg, torch.float32), cfg, alone("a", toks, [70]), {"a": toks}, FP32_TOL)
    check(engine_for(cfg, torch.float32), cfg, alone("a", toks, [50, 1, 1, 2]), {"a": toks}, FP32_TOL)


@pytest.mark.parametrize("mlp", [
    dense(), dense(ff=301), dense(ff=1), None, moe(), moe(experts=6, top=6, count=1, keep=1), moe(experts=6, top=2, count=6, keep=3),
    moe(experts=12, top=1, count=2, keep=1, shared=0), moe(experts=10, top=2, count=0, scale=1.0), moe(experts=70, top=9, count=7, keep=3, ff=9, scale=0.4, shared=33),
    moe(experts=1, top=1, count=1, keep=1), moe(experts=16, top=8, count=4, keep=2)],
    ids=["dense", "dense-301", "dense-1", "none", "moe", "every-expert", "groups-of-one", "top-1-no-shared", "no-groups", "70-experts", "one-expert", "all-of-the-kept"])
def test_feed_forward_alone_fp32(mlp):
    cfg = config([att(heads=1, kv_heads=1, dim=4, vdim=4, dims=2, mlp=mlp)])
    toks = tokens_of(150, cfg["vocab"], 2)  # more tokens than one launch routes beside the norm, then fewer
    check(engine_for(cfg, torch.float32), cfg, alone("a", toks, [140, 10]), {"a": toks}, FP32_TOL)


@pytest.mark.parametrize("kw", [dict(loop=(0, 2, 2)), dict(loop=(1, 2, 1)), dict(loop=(0, 1, 4)), dict(loop=(1, 3, 3)), dict(loop=(0, 3, 1)), dict(loop=None),
                                dict(loop=(2, 3, 2), embed=1.0), dict(loop=(1, 2, 2), width=50), dict(loop=(1, 2, 2), width=36, eps=0.3), dict(width=7, loop=(0, 3, 2))],
                         ids=["first-two", "one-pass", "one-layer-four-times", "to-the-end", "all-once", "no-loop", "last-unscaled", "width-50", "width-36-large-eps", "width-7"])
def test_loops_and_widths_fp32(kw):
    cfg = config([att(mlp=dense()), att(mlp=moe()), att(heads=2, kv_heads=1, mlp=None)], **kw)
    toks = tokens_of(40, cfg["vocab"], 3)
    check(engine_for(cfg, torch.float32), cfg, alone("a", toks, [1, 2, 7, 1, 29]), {"a": toks}, FP32_TOL)


def test_layer_outputs_fp32():
    """The stream after every layer run, not only the logits."""
    for cfg in (FULL, config([att(mlp=dense()), att(mlp=moe())], loop=(0, 2, 2))):
        eng, state = engine_for(cfg, torch.float32)
        toks = tokens_of(40, cfg["vocab"], 3)
        mine: list = []
        orig = eng.model.forward
        eng.model.forward = lambda ctx, batch, logits_out=None: orig(ctx, batch, logits_out, layer_outputs=mine)
        try:
            replay(eng, alone("a", toks, [40]))
        finally:
            eng.model.forward = orig
        ref = O.forward(cfg, state, toks)[1]
        assert len(mine) == ref.shape[0] == len(O.layer_runs(cfg))
        for i, a in enumerate(mine):
            assert rel(a.double().cpu(), ref[i]) < FP32_TOL, f"run {i}"


def test_every_term_matters_fp32():
    """Weights set so that a dropped term shows, and proof that the restatement itself moves when the term goes."""
    cfg = config([att(mlp=dense()), att(mlp=moe())], loop=(1, 2, 2))
    eng, state = engine_for(cfg, torch.float32, seed=6)
    state = {k: v.clone() for k, v in state.items()}
    state["l0.mix.lq1"], state["l0.mix.lk1"] = torch.full((12,), 0.2), torch.full((12,), 0.3)      # exp(0.72)
    state["l0.mix.lq2"], state["l0.mix.lk2"] = torch.full((12,), -0.4), torch.full((12,), 0.25)    # exp(-1.2)
    state["l0.mix.q.norm"], state["l0.mix.k.norm"] = torch.linspace(0.3, 2.0, 12), torch.linspace(2.0, 0.2, 12)
    state["l1.mlp.correction"] = torch.tensor([-3.0, 1.0, -2.0, 0.4, 0.5, -0.6, 0.7, 0.2])
    for n in ("l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l1.norm2b", "final.norm"):
        state[n] = torch.linspace(0.2, 2.0, 48).roll(7 * len(n))
    eng.model.load_state(state)  # this engine (its own seed) serves no other test
    toks = tokens_of(45, cfg["vocab"], 13)
    got = check((eng, eng.model.export_state()), cfg, alone("a", toks, [20, 1, 24]), {"a": toks}, FP32_TOL)["a"]
    z, one = torch.zeros_like, torch.ones_like
    edits = {n: one(state[n]) for n in ("l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l1.norm2b", "final.norm", "l0.mix.q.norm", "l0.mix.k.norm")}
    edits.update({n: z(state[n]) for n in ("l0.mix.lq1", "l0.mix.lk2", "l1.mlp.correction", "l1.mlp.shared.down", "l1.mlp.e6.down")})
    edits["loop.in"] = torch.cat((state["loop.in"][:, :48], z(state["loop.in"][:, 48:])), 1)
    edits["l0.mix.k"] = state["l0.mix.k"].view(2, 2, 12, 48).flip(1).reshape(48, 48)  # a head's two maps change places
    for name, val in edits.items():
        assert rel(O.forward(cfg, dict(state, **{name: val}), toks)[0], got) > 20 * FP32_TOL, name
    for edit in (lambda c: c["embedding"].update(scale=1.0), lambda c: c["loop"].update(times=1), lambda c: c["layers"][1]["mlp"]["router"].update(scale=1.0),
                 lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=4), lambda c: c["layers"][0]["mixer"].update(diff=0.0),
                 lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6), lambda c: c["layers"][0]["mixer"].update(scale=0.2)):
        other = json.loads(json.dumps(cfg))
        edit(other)
        assert rel(O.forward(other, state, toks)[0], got) > 20 * FP32_TOL, other


# ----------------------------------------------------------------------------------------- kernels on built inputs
def _norm_ref(v, w, eps, centre):
    return O.centred_norm(v, w, eps) if centre else O.rms_unit(v, eps) * w


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("rows,W", [(3, 48), (1, 2048), (5, 2056), (2, 8200), (4, 7), (3, 1001), (1030, 200), (1029, 1000), (1027, 2048), (1025, 40)],
                         ids=["48", "2048", "2056", "8200", "7", "1001", "wave-200", "wave-1000", "wave-2048", "wave-40"])
def test_join_norm(dev, dtype, rows, W):
    """Weighted parts and a plain part, normed onto the stream, the next norm, copies beside each other in one wide row; rows whose mean is
    far above their deviation; every way to leave a piece out; out of place and in place."""
    from mini_sglang_amd import mixops

    g = torch.Generator().manual_seed(rows + W)
    eps = 1e-5

    def rnd(*shape, scale=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g, dtype=torch.float64) * scale + mean).to(dtype)

    x = (torch.randn(rows, W, generator=g, dtype=torch.float64) + torch.where(torch.arange(rows) % 2 == 0, 300.0, 0.0)[:, None]).float()
    y, y2 = rnd(rows, 3, W, mean=20.0), rnd(rows, W)
    gate = torch.rand(rows, 3, generator=g).float()
    w_in, w_out = rnd(W, scale=0.3, mean=1.0), rnd(W, scale=0.3, mean=1.0)
    to = lambda t: t.to(dev)  # noqa: E731
    tol = 1e-5 if dtype == torch.float32 else 8e-3
    for centre, use_gate, use_y2, use_w_in, in_place in ((True, True, True, True, True), (False, True, False, True, False), (True, False, True, False, True),
                                                         (True, False, False, True, False)):
        s = (y.double() * (gate.double()[:, :, None] if use_gate else 1.0)).sum(1) + (y2.double() if use_y2 else 0.0)
        want = x.double() + (_norm_ref(s, w_in.double(), eps, centre) if use_w_in else s)
        xd = to(x).clone()
        x_out = xd if in_place else torch.empty_like(xd)
        h = torch.empty((rows, W), dtype=dtype, device=dev)
        wide = torch.zeros((rows, 2 * W), dtype=dtype, device=dev)
        mixops.join_norm(xd, eps, dtype=dtype, centre=centre, y=to(y), gate=to(gate) if use_gate else None, y2=to(y2) if use_y2 else None,
                         w_in=to(w_in) if use_w_in else None, x_out=x_out, raw=(wide[:, W:], wide[:, :W]), w_out=to(w_out), h_out=h)
        assert rel(x_out.double().cpu(), want) < 1e-5
        got = x_out.double().cpu()  # what the second norm saw
        ref = _norm_ref(got, w_out.double(), eps, centre)
        assert rel(h.double().cpu(), ref) < (2e-4 if dtype == torch.float32 else 8e-3)
        assert rel(wide.double().cpu(), torch.cat((got, got), 1)) < tol
    # embedding rows in the place of the stream, no parts; then the stream alone
    table, ids = rnd(31, W), torch.randint(0, 31, (rows,), generator=g, dtype=torch.int32)
    want = table.double()[ids.long()] * 1.7
    x_out, h = torch.empty((rows, W), device=dev), torch.empty((rows, W), dtype=dtype, device=dev)
    wide = torch.zeros((rows, 2 * W), dtype=dtype, device=dev)
    mixops.join_norm(None, eps, dtype=dtype, centre=True, embed=(to(table), to(ids), 1.7), x_out=x_out, raw=(wide[:, W:],), w_out=to(w_out), h_out=h)
    assert rel(x_out.double().cpu(), want) < 1e-6 and rel(h.double().cpu(), O.centred_norm(want, w_out.double(), eps)) < tol
    assert rel(wide.double().cpu()[:, W:], want) < tol and float(wide[:, :W].abs().max()) == 0.0
    h2 = torch.empty_like(h)
    mixops.join_norm(x_out, eps, dtype=dtype, centre=True, w_out=to(w_out), h_out=h2)
    assert torch.equal(h2, h)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("E,top,groups,keep,W,bias", [(15, 5, 3, 2, 64, "mixed"), (8, 2, 4, 1, 40, "negative"), (9, 3, 9, 4, 72, "mixed"), (160, 8, 8, 4, 256, "negative"),
                                                      (6, 6, 1, 1, 30, None), (64, 1, 2, 1, 2048, "mixed"), (200, 20, 20, 3, 128, "negative")])
def test_expert_choice(dev, dtype, E, top, groups, keep, W, bias):
    """The router in the norm's launch and on product-kernel logits, against the choice token by token; corrections that make every choice
    score negative (a dropped group must not win with zeros) and groups whose best expert and whose best pair disagree."""
    from mini_sglang_amd import mixops

    g = torch.Generator().manual_seed(E + W)
    rows = 40
    x = torch.randn(rows, W, generator=g).float().to(dev)
    router = (torch.randn(E, W, generator=g) * 2.0 * W ** -0.5).to(dtype)
    b = None
    if bias is not None:
        b = torch.randn(E, generator=g) * 0.6 - (4.0 if bias == "negative" else 0.0)
        b[:: E // groups] += 0.5  # every group's first expert stands out: its best and its best pair need not agree with the others'
        b = b.to(dtype)
    w = torch.ones(W, dtype=dtype, device=dev)
    h = torch.empty((rows, W), dtype=dtype, device=dev)
    rule = (top, groups, keep, True, 2, 2.5)
    ids, wts = mixops.join_norm(x, 1e-5, dtype=dtype, centre=True, w_out=w, h_out=h, route=(router.to(dev), None if b is None else b.to(dev)) + rule)
    ids2, wts2 = mixops.route(h, router.to(dev), None if b is None else b.to(dev), top, groups, keep, sigmoid=True, group_best=2, scale=2.5)
    scores = 1.0 / (1.0 + torch.exp(-(h.double().cpu() @ router.double().T)))
    corr = torch.zeros(E, dtype=torch.float64) if b is None else b.double()
    differs, sure = 0, 0
    for t in range(rows):
        want = O.choose(scores[t], corr, top, groups, keep)
        c = scores[t] + corr
        n = E // groups
        best1 = sorted(range(groups), key=lambda q: -float(c[q * n: (q + 1) * n].max()))[:keep]
        differs += set(e // n for e in want) - set(best1) != set()
        worth = sorted((float(c[q * n: (q + 1) * n].sort(descending=True).values[:2].sum()) for q in range(groups)), reverse=True)
        inside = sorted((float(c[e]) for e in range(E) if e // n in {e2 // n for e2 in want}), reverse=True)
        gaps = [worth[keep - 1] - worth[keep]] if keep < groups else []
        gaps += [inside[k] - inside[k + 1] for k in range(min(top, len(inside) - 1))]
        if min(gaps, default=1.0) < 1e-5:
            continue  # too close to call in fp32
        sure += 1
        sw = torch.stack([scores[t, e] for e in want])
        sw = sw / (sw.sum() + 1e-20) * 2.5
        for i, wt in ((ids, wts), (ids2, wts2)):
            assert i[t].cpu().tolist() == want, t
            assert rel(wt[t].double().cpu(), sw) < 1e-5
    assert sure >= rows // 2
    if groups > keep and E // groups > 1:
        assert differs > 0  # the pair rule decided somewhere


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("rows,N", [(3, 64), (700, 96), (5, 13), (1, 1), (33, 4096)])
def test_gated_activations(dev, dtype, rows, N):
    from mini_sglang_amd import mixops

    g = torch.Generator().manual_seed(N)
    gu = (torch.randn(rows, 2 * N, generator=g) * torch.tensor([0.1, 3.0, 40.0]).repeat(rows)[:rows, None]).to(dtype)
    z, u = gu.double()[:, :N], gu.double()[:, N:]
    for act, fn in ((mixops.GATE_MUL_SILU, O.silu), (mixops.GATE_MUL_GELU_TANH, O.gelu_tanh)):
        got = mixops.gate_mul(gu.to(dev), act).double().cpu()
        assert bool(torch.isfinite(got).all())
        ref = fn(z) * u
        assert float(((got - ref).abs() / (ref.abs() + 1e-3)).max()) < (2e-5 if dtype == torch.float32 else 6e-3), act


@pytest.mark.parametrize("M,N,K", [(1, 256, 512), (7, 48, 96), (130, 50, 100), (300, 1024, 2048), (33, 7, 14)])
def test_product_with_fp32_result(dev, M, N, K):
    """bf16 operands, fp32 result: closer to the exact product than one rounding to bf16 could be."""
    from mini_sglang_amd import mixops

    g = torch.Generator().manual_seed(M)
    x, w = torch.randn(M, K, generator=g).bfloat16(), (torch.randn(N, K, generator=g) * K ** -0.5).bfloat16()
    out = torch.empty((M, N), device=dev)
    mixops.linear(x.to(dev), w.to(dev), out=out)
    assert rel(out.double().cpu(), x.double() @ w.double().T) < 3e-6


def _paged(dev, T, k, v, dtype, g, slots_total=2048):
    slots = torch.randperm(slots_total, generator=g)[:T].to(torch.int32)
    table = torch.zeros((3, 2048), dtype=torch.int32)
    table[2, :T] = slots
    kc = torch.zeros((slots_total, k[0].numel()), dtype=dtype, device=dev)
    vc = torch.zeros((slots_total, v[0].numel()), dtype=dtype, device=dev)
    kc[slots.long().to(dev)] = k.reshape(T, -1).to(dtype).to(dev)
    vc[slots.long().to(dev)] = v.reshape(T, -1).to(dtype).to(dev)
    return table.to(dev), kc, vc


def _diff_ref(q, k, v, scale, lam, post, eps):
    a = [O.causal_softmax(q[:, :, m], k[:, :, m], v, scale) for m in range(2)]
    return O.rms_unit(a[0] - lam * a[1], eps) * post


def _run_diff(dev, dtype, q, table, kc, vc, G, dv, scale, lam, post, eps, splits, pieces):
    from mini_sglang_amd import mixops

    T, H, _, d = q.shape
    got = torch.empty((T, H * dv), dtype=dtype, device=dev)
    qd = q.reshape(T, -1).float().to(dev)
    for lo, hi in pieces:
        part = torch.empty((hi - lo, H * dv), dtype=dtype, device=dev)
        mixops.diff_attn(part, qd[lo:hi].contiguous(), kc, vc, table, torch.tensor([2], dtype=torch.int32, device=dev),
                         torch.tensor([hi], dtype=torch.int32, device=dev), torch.tensor([0, hi - lo], dtype=torch.int32, device=dev), 1, H, G, d, dv,
                         scale, 0, 0, torch.tensor([lam], dtype=torch.float32, device=dev), post, eps, splits=splits)
        got[lo:hi] = part
    return got.double().cpu().view(T, H, dv)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("loud_map", [0, 1])
@pytest.mark.parametrize("loud", [0, 1, 15, 16, 63, 64, 127, 512, 1023, 1024, 1149])
def test_one_loud_key_far_back(dev, dtype, loud, loud_map):
    """In one map one key scores far above all others, at page and tile borders and a thousand tokens back: every later query, in prompt
    portions and decoded alone, with the keys in one range and in several, returns that key's value (less the other map's share)."""
    H, G, d, dv, scale, lam, eps, T = 6, 2, 16, 24, 0.5, 0.4, 1e-5, 1150
    g = torch.Generator().manual_seed(loud)
    q = torch.randn(T, H, 2, d, generator=g, dtype=torch.float64) * 0.3
    k = torch.randn(T, G, 2, d, generator=g, dtype=torch.float64) * 0.3
    v = torch.randn(T, G, dv, generator=g, dtype=torch.float64)
    k[:, :, loud_map, 0] = 0.0
    k[loud, :, loud_map, 0] = 12.0
    q[:, :, loud_map, 0] = 5.0
    q, k, v = (t.to(dtype).double() for t in (q, k, v))
    ref = _diff_ref(q, k, v, scale, lam, 0.65, eps)
    table, kc, vc = _paged(dev, T, k, v, dtype, g)
    pieces = [(0, 600)] + [(t, t + 1) for t in range(600, 606)] + [(606, 608), (608, 1142)] + [(t, t + 1) for t in range(1142, T)]
    sign = 1.0 if loud_map == 0 else -1.0
    want = v[loud].repeat_interleave(H // G, 0) * sign
    for splits in (1, 4):
        got = _run_diff(dev, dtype, q, table, kc, vc, G, dv, scale, lam, 0.65, eps, splits, pieces)
        assert rel(got, ref) < (2e-5 if dtype == torch.float32 else 3e-2), splits

        def aligned(t):  # cosine between the output and the loud key's value, per head
            return float(((got[t] * want).sum(-1) / (got[t].norm(dim=-1) * want.norm(dim=-1))).min())

        if loud_map == 0 or loud > 0:
            for t in {min(loud + 40, T - 1), T - 1}:
                assert aligned(t) > 0.6, (splits, t)
        if loud > 0:
            assert aligned(loud - 1) < 0.6, "a key after the query was read"


@pytest.mark.parametrize("H,G,d,dv", [(4, 4, 32, 64), (8, 2, 64, 64), (6, 3, 40, 40), (3, 1, 64, 128), (16, 2, 128, 128), (2, 1, 100, 104), (8, 1, 128, 256),
                                      (5, 5, 72, 136), (2, 1, 160, 96), (4, 2, 7, 9), (2, 1, 20, 300), (5, 1, 44, 92), (7, 1, 24, 48), (1, 1, 130, 520), (34, 1, 16, 32), (40, 2, 64, 112)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
def test_two_map_attention_head_sizes(dev, dtype, H, G, d, dv):
    """Every matrix-core instance (and the plain kernel beside it): a portion, single tokens, a portion of two, the rest; keys in one range and in three."""
    T, scale, lam, eps = 330, d ** -0.5, 0.7, 1e-5
    g = torch.Generator().manual_seed(d + dv)
    q, k, v = (torch.randn(T, *w, generator=g, dtype=torch.float64).to(dtype).double() for w in ((H, 2, d), (G, 2, d), (G, dv)))
    ref = _diff_ref(q, k, v, scale, lam, 0.7, eps)
    table, kc, vc = _paged(dev, T, k, v, dtype, g)
    for splits in (1, 3):
        got = _run_diff(dev, dtype, q, table, kc, vc, G, dv, scale, lam, 0.7, eps, splits, [(0, 200), (200, 201), (201, 202), (202, 204), (204, T)])
        assert rel(got, ref) < (2e-5 if dtype == torch.float32 else 3e-2), splits


# ----------------------------------------------------------------------------------------- schedules
@pytest.mark.parametrize("dtype,tol", [(torch.float32, FP32_TOL), (torch.bfloat16, BF16_TOL)], ids=["fp32", "bf16"])
def test_whole_prompt(dtype, tol):
    toks = tokens_of(150, FULL["vocab"], 21)
    check(engine_for(FULL, dtype, spaced=dtype == torch.bfloat16), FULL, alone("a", toks, [150]), {"a": toks}, tol)


def test_prefill_against_token_by_token_fp32():
    eng = engine_for(FULL, torch.float32)
    toks = tokens_of(60, FULL["vocab"], 22)
    whole = check(eng, FULL, alone("a", toks, [60]), {"a": toks}, FP32_TOL)["a"]
    single = check(eng, FULL, alone("a", toks, [1]), {"a": toks}, FP32_TOL)["a"]
    assert rel(single, whole) < FP32_TOL


@pytest.mark.parametrize("sizes", [[2], [3, 1], [5, 2, 17], [16], [64, 1, 1, 2], [33, 31]], ids=["twos", "3-1", "5-2-17", "pages", "64-then-short", "33-31"])
def test_portions_fp32(sizes):
    """Prompts cut anywhere: inside a page, a key tile, between the passes' caches; portions down to two tokens and one."""
    toks = tokens_of(100, FULL["vocab"], 23)
    check(engine_for(FULL, torch.float32), FULL, alone("a", toks, sizes), {"a": toks}, FP32_TOL)


def test_long_sequence_fp32():
    """A thousand tokens in long portions, single tokens between them: keys far away, many tiles, router logits from the product kernel."""
    cfg = config([att(mlp=dense()), att(heads=2, kv_heads=1, scale=0.6, mlp=moe())], loop=(0, 2, 2))
    toks = tokens_of(1050, cfg["vocab"], 24)
    eng = engine_for(cfg, torch.float32, max_tokens=1152)
    got = check(eng, cfg, alone("a", toks, [700, 1, 1, 2, 346]), {"a": toks}, FP32_TOL)["a"]
    assert rel(replay(eng[0], alone("a", toks, [1050]))["a"], got) < FP32_TOL


def test_long_decoding_fp32():
    toks = tokens_of(170, FULL["vocab"], 25)
    check(engine_for(FULL, torch.float32), FULL, alone("a", toks, [20] + [1] * 150), {"a": toks}, FP32_TOL)


def test_first_tokens_fp32():
    """Sequences of one, two and three tokens."""
    eng = engine_for(FULL, torch.float32)
    for n in (1, 2, 3):
        toks = tokens_of(n, FULL["vocab"], 30 + n)
        check(eng, FULL, alone("a", toks, [n]), {"a": toks}, FP32_TOL)
        check(eng, FULL, alone("a", toks, [1]), {"a": toks}, FP32_TOL)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, FP32_TOL), (torch.bfloat16, BF16_TOL)], ids=["fp32", "bf16"])
def test_mixed_batches_against_each_alone(dtype, tol):
    """Four requests of unequal length: portions of some beside single tokens of others, requests that sit out steps."""
    eng = engine_for(FULL, dtype, spaced=dtype == torch.bfloat16)
    seqs = {r: tokens_of(n, FULL["vocab"], 40 + i) for i, (r, n) in enumerate((("a", 90), ("b", 37), ("c", 5), ("d", 61)))}
    a, b, c, d = (seqs[r] for r in "abcd")
    steps = [[("a", a[:50], False), ("b", b[:2], False)],
             [("a", a[50:51], False), ("b", b[2:30], False), ("c", c[:3], False)],
             [("d", d[:40], False), ("a", a[51:52], False), ("c", c[3:4], False)],
             [("a", a[52:88], False), ("b", b[30:], True), ("c", c[4:], True), ("d", d[40:41], False)],
             [("d", d[41:], True), ("a", a[88:], True)]]
    got = check(eng, FULL, steps, seqs, tol)
    for r, toks in seqs.items():
        assert rel(replay(eng[0], alone(r, toks, [len(toks)]))[r], got[r]) < tol, r


def test_pages_used_again_fp32():
    """A pool of six pages and two request rows serving six requests in turn: every page is handed on with its last owner's contents."""
    eng = engine_for(FULL, torch.float32, max_tokens=96, rows=2)
    steps, seqs = [], {}
    for i in range(6):
        r, toks = f"r{i}", tokens_of(30 + 3 * i, FULL["vocab"], 50 + i)
        seqs[r] = toks
        steps += alone(r, toks, [17, 1, 40])
    check(eng, FULL, steps, seqs, FP32_TOL)


def test_other_orders_and_sizes():
    """Head sizes that are no powers of two, three key heads, a mixture in front, a layer without feed-forward inside the loop; two
    requests whose portions and single tokens share steps."""
    cfg = config([att(heads=6, kv_heads=3, dim=40, vdim=56, dims=24, mlp=moe(experts=15, top=2, count=3, keep=2, ff=48, shared=72)),
                  att(heads=4, kv_heads=4, dim=32, vdim=64, dims=32, mlp=None), att(heads=8, kv_heads=2, dim=64, vdim=128, dims=10, mlp=dense(ff=200))],
                 width=192, vocab=333, loop=(0, 2, 3), embed=13.0)
    a, b = tokens_of(120, 333, 63), tokens_of(70, 333, 64)
    steps = [[("a", a[:64], False)], [("a", a[64:65], False), ("b", b[:50], False)], [("a", a[65:66], False), ("b", b[50:51], False)],
             [("a", a[66:], True), ("b", b[51:], True)]]
    check(engine_for(cfg, torch.bfloat16, spaced=True), cfg, steps, {"a": a, "b": b}, BF16_TOL)
    check(engine_for(cfg, torch.float32), cfg, steps, {"a": a, "b": b}, FP32_TOL)


@pytest.mark.parametrize("graphs", [None, [1, 2, 4]], ids=["eager", "graphs"])
def test_greedy_generation_through_the_scheduler(graphs):
    """OfflineRunner.generate (chunked prefill with a small budget, continuous decode, the sampler's argmax, captured decode graphs)
    against greedy decoding with the restatement, on weights loaded AFTER the graphs were captured; a step whose two best logits are
    closer than the fp32 tolerance ends the comparison for that request."""
    from mini_sglang_amd.core import SamplingParams
    from mini_sglang_amd.offline import OfflineRunner

    eng, _ = engine_for(FULL, torch.float32, max_tokens=512, graphs=graphs, seed=11)
    _, state = engine_for(FULL, torch.float32, max_tokens=96, rows=2)
    eng.model.load_state(state)
    prompts = [tokens_of(n, FULL["vocab"], 60 + n) for n in (9, 31, 47)]
    run = OfflineRunner(eng, max_extend_tokens=32, seed=2)
    n_new = 12
    run.generate(prompts, [SamplingParams(temperature=0.0, max_tokens=n_new, ignore_eos=True)] * len(prompts))
    compared = 0
    for p, st in zip(prompts, run.last_states):
        out = run.output_ids(st)
        assert len(out) == n_new
        seq = list(p)
        for tok in out:
            lg = O.forward(FULL, state, seq)[0][-1]
            top2 = lg.topk(2).values
            if float(top2[0] - top2[1]) < 1e-3 * float(lg.abs().max()):
                break
            assert tok == int(lg.argmax()), (len(seq), tok)
            seq.append(tok)
            compared += 1
    assert compared >= 2 * n_new


WIDE = config([att(heads=8, kv_heads=2, dim=64, vdim=128, dims=64, mlp=dense(ff=2048)),
               att(heads=4, kv_heads=4, dim=32, vdim=64, dims=32, mlp=moe(experts=16, top=4, count=4, keep=2, ff=256, shared=512))],
              width=1024, vocab=1500, loop=(0, 2, 2), embed=30.0)


@pytest.mark.parametrize("cfg", [FULL, WIDE], ids=["small", "wide"])
def test_decode_graph_replays_bf16(cfg):
    """Captured decode steps replayed several times, eager steps and synchronizations between, draw the tokens the eager steps draw."""
    from mini_sglang_amd.core import SamplingParams
    from mini_sglang_amd.offline import OfflineRunner

    eng, _ = engine_for(cfg, torch.bfloat16, graphs=[2], seed=12, spaced=True)
    prompts = [tokens_of(20, cfg["vocab"], 80), tokens_of(27, cfg["vocab"], 81)]
    gr = eng.graph_runner
    captured = gr.can_use_cuda_graph
    outs = []
    try:
        for use in (True, False, True, True, False):
            gr.can_use_cuda_graph = captured if use else (lambda batch: False)
            run = OfflineRunner(eng, max_extend_tokens=64, seed=2)
            run.generate(prompts, [SamplingParams(temperature=0.0, max_tokens=16, ignore_eos=True)] * 2)
            outs.append([run.output_ids(st) for st in run.last_states])
            torch.cuda.synchronize()
    finally:
        gr.can_use_cuda_graph = captured
    assert all(o == outs[0] for o in outs[1:])


def test_generate_command(tmp_path, capsys):
    """The command line's `generate` on a checkpoint folder written here, in this process."""
    from safetensors.torch import save_file

    from mini_sglang_amd import cli
    from mini_sglang_amd.hybrid import HybridDecoder, redasun_config

    cfg = config([att(mlp=moe()), att(heads=2, kv_heads=1, mlp=dense(ff=24))], width=64, vocab=97, loop=(0, 1, 2))
    state = HybridDecoder(redasun_config(cfg), dtype=torch.bfloat16, device=torch.device("cpu"), seed=9).export_state()
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(state, str(tmp_path / "model.safetensors"))
    prompts = [tokens_of(5, 97, 1), tokens_of(23, 97, 2)]
    args = ["generate", "--model", str(tmp_path), "--dtype", "float32", "--max-tokens", "5", "--no-graphs"]
    for p in prompts:
        args += ["--prompt", ",".join(map(str, p))]
    assert cli.main(args) == 0
    lines = [json.loads(ln) for ln in capsys.readouterr().out.splitlines() if ln.startswith("{")]
    assert [ln["prompt"] for ln in lines] == prompts and all(len(ln["output"]) == 5 for ln in lines)
    for p, ln in zip(prompts, lines):
        lg = O.forward(cfg, state, p)[0][-1]
        top2 = lg.topk(2).values
        if float(top2[0] - top2[1]) > 1e-3 * float(lg.abs().max()):
            assert ln["output"][0] == int(lg.argmax())


def test_trace_command_line(tmp_path):
    """bin/trace_run end to end in its own process on a checkpoint folder written here: the model class comes from config.json."""
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np
    from safetensors.torch import save_file

    from mini_sglang_amd.hybrid import HybridDecoder, redasun_config

    cfg = config([att(heads=3, kv_heads=1, dim=10, vdim=14, dims=4, mlp=dense(ff=44)), att(heads=2, kv_heads=2, dim=14, vdim=7, dims=6, mlp=moe(ff=10))],
                 width=100, vocab=131, loop=(1, 2, 3))
    model = HybridDecoder(redasun_config(cfg), dtype=torch.bfloat16, device=torch.device("cpu"), seed=9)
    state = {k: (v.to(torch.bfloat16) if v.is_floating_point() else v) for k, v in model.export_state().items()}
    mdir, out = tmp_path / "model", tmp_path / "out"
    mdir.mkdir()
    (mdir / "config.json").write_text(json.dumps(cfg))
    save_file(state, str(mdir / "model.safetensors"))
    a, b = tokens_of(45, cfg["vocab"], 70), tokens_of(9, cfg["vocab"], 71)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:8], "want": []}, {"id": "a", "tokens": a[30:31], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[31:], "want": [13]}, {"id": "b", "tokens": b[8:], "want": [0]}], "end": ["a", "b"]}]
    root = Path(__file__).resolve().parent.parent
    pr = subprocess.run([sys.executable, str(root / "bin" / "trace_run"), "--model", str(mdir), "--dtype", "float32", "--out", str(out),
                         "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n", text=True, capture_output=True,
                        timeout=110)
    assert pr.returncode == 0, pr.stderr[-2000:]
    assert [ln for ln in pr.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    ra, rb = O.forward(cfg, state, a)[0], O.forward(cfg, state, b)[0]
    got0, got1, got2 = (torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(n, -1)).double() for i, n in ((0, 2), (1, 1), (2, 2)))
    scale = float(ra.abs().max())
    assert float((got0 - ra[[0, 29]]).abs().max()) < FP32_TOL * scale
    assert float((got1 - ra[[30]]).abs().max()) < FP32_TOL * scale
    assert float((got2[0] - ra[44]).abs().max()) < FP32_TOL * scale and float((got2[1] - rb[8]).abs().max()) < FP32_TOL * scale
