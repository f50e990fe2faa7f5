"""The multi-stream hybrid decoder (Nagezen: several residual streams joined by small matrices, an element-wise squashing in the place
of norms, retention, gated linear attention, the difference of two softmax maps over a window with kept first tokens, clamped gated
feed-forwards) on the GPU against the plain restatement in tests/nagezen_oracle.py: small configurations and random weights made
here, the engine's own step function, cache, state slots and kernels on one side, whole-sequence float64 arithmetic on the other.

fp32 engines are held to 2e-4 of the largest reference value (the sharp test); bf16 engines to the rounding of a 16-bit product
chain.  Where random weights would hide a fault the inputs are built so that it shows: one key whose score stands far above all others
just inside and just outside a window, decays that forget within a token and decays that never forget, state rows that still hold
their last owner's state.
"""
from __future__ import annotations

import json

import pytest
import torch

import nagezen_oracle as O
from test_gpu_hybrid import alone, rel, replay, tokens_of

pytestmark = pytest.mark.gpu

FP32_TOL = 2e-4
BF16_TOL = 6e-2


# ----------------------------------------------------------------------------------------- configurations
def dense(ff=56, limit=1.1):
    return {"kind": "dense", "ff": ff, "limit": limit}


def ret(heads=3, dim=20, vdim=28, dims=12, base=900.0, decay=None, mlp=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay or [0.6 + 0.395 * (i + 1) / heads for i in range(heads)]}
    if dims:
        m["rot"] = {"base": base, "dims": dims}
    return {"type": "retention", "mixer": m, "mlp": mlp}


def gla(heads=2, dim=24, vdim=20, tau=8.0, mlp=None):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": mlp}


SCALING = {"factor": 4.0, "fast": 4.0, "slow": 1.0, "original": 64}


def att(heads=6, kv_heads=2, dim=12, vdim=20, dims=8, base=500.0, scale=0.3, window=9, keep=3, diff=0.35, scaling=SCALING, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if dims:
        m["rot"] = {"base": base, "dims": dims}
        if scaling:
            m["rot"]["scaling"] = scaling
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def config(layers, width=48, vocab=80, eps=1e-5, streams=2, logit_scale=1.6):
    return {"architecture": "Nagezen", "layers": layers, "norm": {"eps": eps}, "streams": streams, "logit_scale": logit_scale, "vocab": vocab,
            "width": width}


FULL = config([ret(mlp=dense()), att(mlp=dense(ff=40, limit=0.4)), gla(mlp=dense()), att(heads=3, kv_heads=3, dim=8, vdim=8, dims=4, window=20,
               keep=0, diff=0.1, scaling=None, mlp=None), gla(heads=4, dim=8, vdim=40, tau=2.0, mlp=None),
               ret(heads=1, dim=8, vdim=70, dims=0, decay=[0.99], mlp=dense(ff=24, limit=3.0))], streams=4)


# ----------------------------------------------------------------------------------------- harness
_ENGINES: dict = {}


def shapes_of(cfg_json, rank=5):
    return {f"l{i}.mix.a1": (rank + i, cfg_json["width"]) for i, e in enumerate(cfg_json["layers"]) if e["type"] == "gla"}


def engine_for(cfg_json, dtype, max_tokens=512, rows=4, page_size=16, graphs=None, seed=5):
    """(engine, checkpoint-named weights on the host) for a configuration; engines are kept for the session."""
    from mini_sglang_amd.engine import Engine, EngineConfig
    from mini_sglang_amd.hybrid import nagezen_config

    key = (json.dumps(cfg_json, sort_keys=True), dtype, max_tokens, rows, page_size, tuple(graphs or ()), seed)
    if key not in _ENGINES:
        pages = max_tokens // page_size
        eng = Engine(EngineConfig(model=nagezen_config(cfg_json, shapes_of(cfg_json)), dtype=dtype, max_running_req=rows, page_size=page_size,
                                  num_page_override=pages, max_seq_len_override=pages * page_size, cuda_graph_bs=list(graphs or []),
                                  gemm_tune="off", refine_in_graph=False, seed=seed), torch.device("cuda:0"))
        _ENGINES[key] = (eng, eng.model.export_state())
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
    ret(), ret(heads=1, dim=16, vdim=16, dims=16, decay=[1.0]), ret(heads=5, dim=6, vdim=100, dims=2, base=3.0), ret(heads=2, dim=130, vdim=40, dims=64),
    ret(heads=2, dim=48, vdim=264, dims=10), ret(heads=2, dim=9, vdim=7, dims=0, decay=[0.05, 0.9999]), ret(heads=2, dim=200, vdim=180, dims=200),
    gla(), gla(heads=1, dim=16, vdim=16, tau=1.0), gla(heads=5, dim=7, vdim=100, tau=16.0), gla(heads=2, dim=140, vdim=33, tau=0.2),
    gla(heads=2, dim=100, vdim=200, tau=3.0), gla(heads=1, dim=33, vdim=300, tau=4.0), gla(heads=3, dim=64, vdim=64, tau=100.0),
    att(), att(heads=3, kv_heads=3, dim=10, vdim=6, dims=10, scaling=None), att(heads=6, kv_heads=2, dim=8, vdim=72, dims=0, window=0),
    att(heads=1, kv_heads=1, dim=40, vdim=8, dims=2, scale=1.0, window=1, keep=1), att(heads=34, kv_heads=1, dim=8, vdim=8, dims=4, window=64),
    att(window=200, keep=7, base=2.0, scaling={"factor": 16.0, "fast": 9.0, "slow": 0.5, "original": 300}), att(window=4, keep=40, diff=0.0),
    att(dims=12, base=1e6, diff=0.9, scaling={"factor": 1.0, "fast": 32.0, "slow": 1.0, "original": 128}),
], ids=["retention", "retention-one-head-no-decay", "retention-wide-v", "retention-wide-k", "retention-v-264", "retention-odd-no-rotation",
        "retention-200", "gla", "gla-one-head-tau-1", "gla-wide-v", "gla-fast-decays", "gla-100-200", "gla-v-300", "gla-slow-decays", "attention",
        "attention-ungrouped-unscaled", "attention-wide-v-no-rotation-no-window", "attention-window-1-keep-1", "attention-34-per-key-head",
        "attention-wide-window-other-ramp", "attention-more-kept-than-window", "attention-factor-1"])
def test_mixer_alone_fp32(layer):
    cfg = config([layer])
    toks = tokens_of(70, cfg["vocab"], 1)
    check(engine_for(cfg, torch.float32), cfg, alone("a", toks, [70]), {"a": toks}, FP32_TOL)


@pytest.mark.parametrize("mlp", [dense(), dense(ff=301, limit=0.05), dense(limit=50.0), None], ids=["clamped", "odd-tight", "never-clamped", "none"])
def test_feed_forward_alone_fp32(mlp):
    cfg = config([ret(heads=1, dim=4, vdim=4, dims=2, mlp=mlp)])
    toks = tokens_of(50, cfg["vocab"], 2)
    check(engine_for(cfg, torch.float32), cfg, alone("a", toks, [50]), {"a": toks}, FP32_TOL)


@pytest.mark.parametrize("kw", [dict(streams=1), dict(streams=3), dict(streams=5), dict(streams=9), dict(streams=16, width=40), dict(width=50),
                                dict(logit_scale=0.3), dict(eps=1e-2)],
                         ids=["one", "three", "five", "nine", "sixteen", "width-50", "logits-scaled-down", "large-eps"])
def test_stream_variants_fp32(kw):
    cfg = config([gla(mlp=dense()), att(mlp=dense())], **kw)
    toks = tokens_of(40, cfg["vocab"], 3)
    check(engine_for(cfg, torch.float32), cfg, alone("a", toks, [1, 2, 7, 1, 29]), {"a": toks}, FP32_TOL)


def test_layer_outputs_fp32():
    """The sum of the streams after every layer, not only the logits."""
    eng, state = engine_for(FULL, torch.float32)
    toks = tokens_of(40, FULL["vocab"], 3)
    mine: list = []
    orig = eng.model.forward
    eng.model.forward = lambda ctx, batch, logits_out=None: orig(ctx, batch, logits_out, layer_outputs=mine)
    try:
        replay(eng, alone("a", toks, [40]))
    finally:
        eng.model.forward = orig
    ref = O.forward(FULL, state, toks)[1]
    assert len(mine) == ref.shape[0] == len(FULL["layers"])
    for i, a in enumerate(mine):
        assert rel(a.double().cpu(), ref[i]) < FP32_TOL, f"layer {i}"


def test_every_term_matters_fp32():
    """Weights set so that a dropped term shows, and proof that the restatement itself moves when the term goes."""
    cfg = config([att(mlp=dense()), gla(mlp=dense()), ret(mlp=None)], streams=3)
    eng, state = engine_for(cfg, torch.float32, seed=6)
    state = {k: v.clone() for k, v in state.items()}
    state["l0.mix.lq1"], state["l0.mix.lk1"] = torch.full((12,), 0.2), torch.full((12,), 0.3)      # exp(0.72)
    state["l0.mix.lq2"], state["l0.mix.lk2"] = torch.full((12,), -0.4), torch.full((12,), 0.25)    # exp(-1.2)
    state["l0.mix.g"] = state["l0.mix.g"] * 8.0
    state["l0.mix.q.b"], state["l0.mix.k.b"] = torch.linspace(-1, 1, 144), torch.linspace(2, -1, 48)
    state["l0.mix.v.b"] = torch.linspace(-2, 2, 40)
    state["l0.mix.q.norm"], state["l0.mix.k.norm"] = torch.linspace(0.3, 2.0, 12), torch.linspace(2.0, 0.2, 12)
    state["l1.mix.a2.b"] = torch.linspace(-6, 4, 48)
    state["l1.mix.norm"] = torch.linspace(0.2, 2.0, 20)
    state["l0.norm1.alpha"] = torch.tensor(2.2)
    state["final.norm.b"] = torch.linspace(-1, 1, 48)
    eng.model.load_state(state)  # this engine (its own seed) serves no other test
    toks = tokens_of(45, cfg["vocab"], 13)
    got = check((eng, eng.model.export_state()), cfg, alone("a", toks, [20, 1, 24]), {"a": toks}, FP32_TOL)["a"]
    z = torch.zeros_like
    edits = {"l0.mix.lq1": z(state["l0.mix.lq1"]), "l0.mix.lk2": z(state["l0.mix.lk2"]), "l0.mix.g": z(state["l0.mix.g"]),
             "l0.mix.q.b": z(state["l0.mix.q.b"]), "l0.mix.k.b": z(state["l0.mix.k.b"]), "l0.mix.v.b": z(state["l0.mix.v.b"]),
             "l0.mix.q.norm": torch.ones(12), "l0.mix.k.norm": torch.ones(12), "l1.mix.a2.b": z(state["l1.mix.a2.b"]),
             "l1.mix.norm": torch.ones(20), "l0.norm1.alpha": torch.tensor(1.0), "l2.norm1.b": z(state["l2.norm1.b"]),
             "final.norm.b": torch.zeros(48), "l1.hc1.in": torch.ones(3), "l1.hc2.out": torch.ones(3), "l2.hc1.mix": torch.eye(3),
             "l0.hc2.mix": state["l0.hc2.mix"].T.contiguous()}
    for name, val in edits.items():
        other = dict(state)
        other[name] = val
        assert rel(O.forward(cfg, other, toks)[0], got) > 20 * FP32_TOL, name


# ----------------------------------------------------------------------------------------- kernels on built inputs
def _paged(dev, T, k, v, dtype, g):
    slots = torch.randperm(1024, generator=g)[:T].to(torch.int32)
    table = torch.zeros((3, 640), dtype=torch.int32)
    table[2, :T] = slots
    kc = torch.zeros((1024, k[0].numel()), dtype=dtype, device=dev)
    vc = torch.zeros((1024, v[0].numel()), dtype=dtype, device=dev)
    kc[slots.long().to(dev)] = k.reshape(T, -1).to(dtype).to(dev)
    vc[slots.long().to(dev)] = v.reshape(T, -1).to(dtype).to(dev)
    return table.to(dev), kc, vc


def _pieces(T, cut, singles):
    end = min(T, cut + singles)
    return [(0, cut)] + [(t, t + 1) for t in range(cut, end)] + ([(end, T)] if end < T else [])


def _diff_ref(q, k, v, scale, window, keep, lam, post, eps, gate):
    a = [O.masked_softmax(q[:, :, m], k[:, :, m], v, scale, window, keep) for m in range(2)]
    return O.rms_unit(a[0] - lam * a[1], eps) * post * O.sigmoid(gate)


def _run_diff(dev, dtype, q, gate, table, kc, vc, G, scale, window, keep, lam, post, eps, splits, pieces):
    from mini_sglang_amd import mixops

    T, H, _, d = q.shape
    dv = gate.shape[2]
    got = torch.empty((T, H * dv), dtype=dtype, device=dev)
    qd, gd = q.reshape(T, -1).float().to(dev), torch.cat([torch.zeros(T, 8), gate.reshape(T, -1).float()], 1).to(dtype).to(dev)
    for lo, hi in pieces:
        part = torch.empty((hi - lo, H * dv + 8), dtype=dtype, device=dev)[:, : H * dv]  # views with a row stride
        mixops.diff_attn(part, qd[lo:hi].contiguous(), kc, vc, table, torch.tensor([2], dtype=torch.int32, device=dev),
                         torch.tensor([hi], dtype=torch.int32, device=dev), torch.tensor([0, hi - lo], dtype=torch.int32, device=dev), 1, H, G, d,
                         dv, scale, window, keep, torch.tensor([lam], dtype=torch.float32, device=dev), post, eps, gate=gd[lo:hi, 8:], splits=splits)
        got[lo:hi] = part
    return got.double().cpu().view(T, H, dv)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("splits", [1, 3], ids=["one-range", "three-ranges"])
@pytest.mark.parametrize("loud,window,keep", [(0, 64, 1), (15, 64, 0), (16, 17, 17), (16, 17, 16), (63, 64, 64), (63, 64, 63), (64, 65, 65),
                                              (100, 1, 5), (255, 96, 20), (256, 40, 100), (299, 300, 4), (200, 0, 0), (5, 30, 9)])
def test_diff_attention_one_loud_key(dev, dtype, splits, loud, window, keep):
    """In the first map one key scores far above all others: every query that sees it (those up to `window - 1` tokens later, or every
    later one when it is among the kept first keys) returns its value less the second map's share; the first query that does not see it
    returns something else.  The sequence is a prompt portion, single decoded tokens, a second portion, on slots scattered over the
    pool, so edges fall inside portions and among decoded tokens; the keys of a step in one range and cut into three."""
    H, G, d, dv, scale, lam, eps = 6, 2, 16, 24, 0.5, 0.4, 1e-5
    T = 420
    g = torch.Generator().manual_seed(loud + window)
    q = torch.randn(T, H, 2, d, generator=g, dtype=torch.float64) * 0.3
    k = torch.randn(T, G, 2, d, generator=g, dtype=torch.float64) * 0.3
    v = torch.randn(T, G, dv, generator=g, dtype=torch.float64)
    gate = torch.randn(T, H, dv, generator=g, dtype=torch.float64)
    k[:, :, 0, 0] = 0.0
    k[loud, :, 0, 0] = 12.0
    q[:, :, 0, 0] = 5.0
    q, k, v, gate = (t.to(dtype).double() for t in (q, k, v, gate))
    ref = _diff_ref(q, k, v, scale, window, keep, lam, 0.65, eps, gate)
    table, kc, vc = _paged(dev, T, k, v, dtype, g)
    got = _run_diff(dev, dtype, q, gate, table, kc, vc, G, scale, window, keep, lam, 0.65, eps, splits, _pieces(T, 290, 40))
    assert rel(got, ref) < (2e-5 if dtype == torch.float32 else 3e-2)
    last = T - 1 if window == 0 or loud < keep else min(T - 1, loud + window - 1)
    ungated = got / O.sigmoid(gate)
    want = v[loud].repeat_interleave(H // G, 0)

    def aligned(t):  # cosine between the output and the loud key's value, per head
        o = ungated[t]
        return float(((o * want).sum(-1) / (o.norm(dim=-1) * want.norm(dim=-1))).min())

    for t in {loud, min(loud + 1, last), last}:
        assert aligned(t) > 0.7, t
    if last + 1 < T:
        assert aligned(last + 1) < 0.6, "the key just outside the window was read"


@pytest.mark.parametrize("H,G,d,dv", [(4, 4, 32, 64), (8, 2, 64, 64), (6, 3, 40, 40), (3, 1, 64, 128), (16, 2, 128, 128), (2, 1, 100, 104), (8, 1, 128, 256),
                                      (5, 5, 72, 136), (2, 1, 160, 96), (4, 2, 7, 9)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
def test_diff_attention_head_sizes(dev, dtype, H, G, d, dv):
    """Every matrix-core instance (and the plain kernel beside it), a window that ends inside a tile, kept first keys, a portion after a
    cached prefix and single tokens, keys in one range and in two."""
    T, window, keep, scale, lam, eps = 150, 45, 13, d ** -0.5, 0.3, 1e-5
    g = torch.Generator().manual_seed(d + dv)
    q, k, v, gate = (torch.randn(T, *w, generator=g, dtype=torch.float64).to(dtype).double() for w in ((H, 2, d), (G, 2, d), (G, dv), (H, dv)))
    ref = _diff_ref(q, k, v, scale, window, keep, lam, 0.7, eps, gate)
    table, kc, vc = _paged(dev, T, k, v, dtype, g)
    for splits in (1, 2):
        got = _run_diff(dev, dtype, q, gate, table, kc, vc, G, scale, window, keep, lam, 0.7, eps, splits, _pieces(T, 70, 30))
        assert rel(got, ref) < (2e-5 if dtype == torch.float32 else 3e-2), splits


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
def test_diff_attention_batches(dev, dtype):
    """Three requests of unequal length in one launch: a portion that continues a cached prefix, a fresh prompt, one decoded token."""
    from mini_sglang_amd import mixops

    H, G, d, dv, scale, window, keep, lam, eps = 3, 3, 20, 40, 0.4, 33, 6, 0.5, 1e-4
    g = torch.Generator().manual_seed(5)
    lens, new = [150, 47, 90], [60, 47, 1]
    seqs = [tuple(torch.randn(n, *w, generator=g, dtype=torch.float64).to(dtype).double() for w in ((H, 2, d), (G, 2, d), (G, dv), (H, dv))) for n in lens]
    kc = torch.zeros((1024, G * 2 * d), dtype=dtype, device=dev)
    vc = torch.zeros((1024, G * dv), dtype=dtype, device=dev)
    table = torch.zeros((4, 256), dtype=torch.int32)
    perm = torch.randperm(1024, generator=g).to(torch.int32)
    at = 0
    for b, (_, k, v, _) in enumerate(seqs):
        sl = perm[at: at + lens[b]]
        at += lens[b]
        table[b + 1, : lens[b]] = sl
        kc[sl.long().to(dev)] = k.reshape(lens[b], -1).to(dtype).to(dev)
        vc[sl.long().to(dev)] = v.reshape(lens[b], -1).to(dtype).to(dev)
    qd, gd = (torch.cat([s[i][n - m:].reshape(m, -1) for s, n, m in zip(seqs, lens, new)]) for i in (0, 3))
    cu = torch.tensor([0, 60, 107, 108], dtype=torch.int32, device=dev)
    for splits in (1, 2):
        out = torch.empty((108, H * dv), dtype=dtype, device=dev)
        mixops.diff_attn(out, qd.float().to(dev), kc, vc, table.to(dev), torch.tensor([1, 2, 3], dtype=torch.int32, device=dev),
                         torch.tensor(lens, dtype=torch.int32, device=dev), cu, 3, H, G, d, dv, scale, window, keep,
                         torch.tensor([lam], dtype=torch.float32, device=dev), 1.0, eps, gate=gd.to(dtype).to(dev), splits=splits)
        got, at = out.double().cpu().view(108, H, dv), 0
        for (q, k, v, gate), n, m in zip(seqs, lens, new):
            ref = _diff_ref(q, k, v, scale, window, keep, lam, 1.0, eps, gate)[n - m:]
            assert rel(got[at: at + m], ref) < (2e-5 if dtype == torch.float32 else 3e-2)
            at += m


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("keep", [0, 1, 30, 64, 90, 500])
def test_single_map_attention_keeps_first_keys(dev, dtype, keep):
    """The one-map kernels of the same attention with kept first keys."""
    from mini_sglang_amd import mixops

    H, G, d, dv, T, window, scale = 6, 2, 24, 40, 260, 41, 0.6
    g = torch.Generator().manual_seed(keep)
    q, k, v = (torch.randn(T, n, w, generator=g, dtype=torch.float64).to(dtype).double() for n, w in ((H, d), (G, d), (G, dv)))
    ref = O.masked_softmax(q, k, v, scale, window, keep)
    table, kc, vc = _paged(dev, T, k, v, dtype, g)
    qd = q.reshape(T, -1).float().to(dev)
    for splits in (1, 3):
        got = torch.empty((T, H * dv), dtype=dtype, device=dev)
        for lo, hi in _pieces(T, 190, 10):
            part = torch.empty((hi - lo, H * dv), dtype=dtype, device=dev)
            mixops.sink_attn(part, qd[lo:hi].contiguous(), kc, vc, table, torch.tensor([2], dtype=torch.int32, device=dev),
                             torch.tensor([hi], dtype=torch.int32, device=dev), torch.tensor([0, hi - lo], dtype=torch.int32, device=dev), 1, H, G,
                             d, dv, scale, window, None, splits=splits, keep=keep)
            got[lo:hi] = part
        assert rel(got.double().cpu().view(T, H, dv), ref) < (1e-5 if dtype == torch.float32 else 2e-2), splits


def _chunk_list(cuts, chunk, dev):
    items, firsts = [], [0]
    for b, (s, e) in cuts.items():
        items += [[b, c, min(c + chunk, e - s)] for c in range(0, e - s, chunk)]
        firsts.append(len(items))
    return (torch.tensor(items, dtype=torch.int32, device=dev).view(-1), torch.tensor(firsts, dtype=torch.int32, device=dev), len(items))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("chunk", [0, 1, 5, 16, 21], ids=["whole", "chunks-of-1", "chunks-of-5", "chunks-of-16", "chunks-of-21"])
@pytest.mark.parametrize("channel", [False, True], ids=["per-head", "per-channel"])
def test_decay_attention_kernel_state_slots_and_cuts(dev, dtype, channel, chunk):
    """The recurrence kernel alone, every size class: two requests in one launch on state rows that hold garbage, then continued in a
    second launch; whole portions, and portions cut into pieces that run in parallel and are joined; inputs as column blocks of one
    row; decays from 'forgets at once' to 'never forgets' in one launch (per channel: also far beyond what exp(-log decay) could hold
    over 16 tokens, where the scores are summed pair by pair)."""
    from mini_sglang_amd import mixops

    for H, d, dv, tau in ((2, 20, 28, 8.0), (1, 32, 64, 0.05), (3, 50, 30, 2.0), (2, 64, 100, 16.0), (2, 72, 40, 1.0), (1, 128, 128, 4.0), (1, 100, 250, 1.0),
                          (1, 250, 128, 8.0), (1, 160, 150, 3.0), (1, 40, 300, 0.3)):
        g = torch.Generator().manual_seed(d)
        lens = [61, 18]

        def make(n, w):
            return torch.randn(n, w, generator=g, dtype=torch.float64).to(dtype).double()

        seq = {b: {k: make(n, H * w) for k, w in (("q", d), ("k", d), ("v", dv), ("g", dv), ("z", d))} for b, n in enumerate(lens)}
        if channel:
            for s in seq.values():
                s["z"] = (s["z"] * 4.0).to(dtype).double()
        zb = torch.linspace(-3.0, 6.0, H * d, dtype=torch.float64).float().double()
        decay = torch.tensor([0.9, 1.0, 1e-3][:H]).double()
        w = (1.0 + 0.3 * torch.randn(dv, generator=g, dtype=torch.float64)).to(dtype).double() if channel else None
        rd = 0 if channel else d // 2 // 2 * 2
        freqs, amp = O.rotary(rd, 300.0, {"factor": 2.0, "fast": 8.0, "slow": 1.0, "original": 100}) if rd else (torch.zeros(0), 1.0)
        ang = torch.arange(64, dtype=torch.float64)[:, None] * freqs[None, :]
        table = torch.cat((ang.cos() * amp, ang.sin() * amp), 1).float().to(dev).contiguous() if rd else None
        state = torch.randn((3, H, d, dv), generator=g, dtype=torch.float32).to(dev)  # garbage: a fresh request must not read it
        outs = {b: [] for b in seq}
        for lo, hi in ((0.0, 0.6), (0.6, 1.0)):
            cuts = {b: (int(lo * n), int(hi * n)) for b, n in enumerate(lens)}
            wide = torch.cat([torch.cat([seq[b][n][s:e] for n in ("q", "k", "v", "g", "z")], 1) for b, (s, e) in cuts.items()]).to(dtype).to(dev)
            cols = torch.split(wide, [H * d, H * d, H * dv, H * dv, H * d], dim=1)
            n0 = cuts[0][1] - cuts[0][0]
            cu = torch.tensor([0, n0, wide.shape[0]], dtype=torch.int32, device=dev)
            pos = torch.cat([torch.arange(s, e) for s, e in cuts.values()]).to(torch.int32).to(dev)
            kw = dict(z=cols[4], z_bias=zb.float().to(dev), tau=tau, weight=w.to(dtype).to(dev)) if channel else \
                dict(decay=decay.float().to(dev), cos_sin=table, positions=pos)
            out = mixops.decay_attn(cols[0], cols[1], cols[2], cols[3], state, cu, torch.tensor([cuts[0][1], cuts[1][1]], dtype=torch.int32, device=dev),
                                    torch.tensor([2, 0], dtype=torch.int32, device=dev), 2, 1e-5, q_scale=0.7, k_scale=d ** -0.5,
                                    chunks=_chunk_list(cuts, chunk, dev) if chunk else None, **kw)
            outs[0].append(out[:n0].cpu())
            outs[1].append(out[n0:].cpu())
        for b, n in enumerate(lens):
            s = {k: v.reshape(n, H, -1) for k, v in seq[b].items()}
            p = torch.arange(n)
            qq, kk = (O.rotate(s[x], freqs, amp, p) for x in ("q", "k"))
            a = O.sigmoid(s["z"] + zb.reshape(H, d)) ** (1.0 / tau) if channel else decay[None, :, None].expand(n, H, d)
            o, S = O.decayed_outer_sum(qq * 0.7, kk * d ** -0.5, s["v"], a)
            o = O.rms_unit(o, 1e-5) * (w if channel else 1.0) * O.silu(s["g"])
            # a request's first tokens hold one or two outer products: their unit-RMS rows carry the rounding of a single score
            assert rel(torch.cat(outs[b]).double(), o.reshape(n, -1)) < (5e-5 if dtype == torch.float32 else 1e-2), (H, d, dv, b)
            assert rel(state[[2, 0][b]].double().cpu(), S) < (1e-5 if dtype == torch.float32 else 2e-5), (H, d, dv, b)


def test_decay_attention_kernel_interleaved_rotation(dev):
    from mini_sglang_amd import mixops

    H, d, dv, n, rd = 2, 24, 24, 40, 10
    g = torch.Generator().manual_seed(3)
    q, k, v, gate = (torch.randn(n, H, w, generator=g, dtype=torch.float64).float().double() for w in (d, d, dv, dv))
    freqs, _ = O.rotary(rd, 50.0, None)
    ang = torch.arange(n, dtype=torch.float64)[:, None] * freqs[None, :]

    def turn(x):
        y = x.clone()
        c, s = ang.cos()[:, None], ang.sin()[:, None]
        y[..., 0:rd:2], y[..., 1:rd:2] = x[..., 0:rd:2] * c - x[..., 1:rd:2] * s, x[..., 1:rd:2] * c + x[..., 0:rd:2] * s
        return y

    decay = torch.tensor([0.7, 0.97]).double()
    ref = O.rms_unit(O.decayed_outer_sum(turn(q), turn(k), v, decay[None, :, None].expand(n, H, d))[0], 1e-5) * O.silu(gate)
    wide = torch.cat([t.reshape(n, -1) for t in (q, k, v, gate)], 1).float().to(dev)
    cols = torch.split(wide, [H * d, H * d, H * dv, H * dv], dim=1)
    i32 = dict(dtype=torch.int32, device=dev)
    out = mixops.decay_attn(*cols, torch.zeros((1, H, d, dv), device=dev), torch.tensor([0, n], **i32), torch.tensor([n], **i32), torch.tensor([0], **i32), 1,
                            1e-5, decay=decay.float().to(dev), cos_sin=torch.cat((ang.cos(), ang.sin()), 1).float().to(dev).contiguous(),
                            positions=torch.arange(n, **i32), interleaved=True)
    assert rel(out.double().cpu(), ref.reshape(n, -1)) < 5e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("s,W", [(1, 64), (2, 36), (3, 50), (4, 128), (7, 24), (16, 20)])
def test_stream_kernel(dev, dtype, s, W):
    """Update, read and squashing; in place and out of place; one row standing for all streams; without an update; without a norm."""
    from mini_sglang_amd import mixops

    T = 9
    g = torch.Generator().manual_seed(s)
    x, x0 = torch.randn(T, s, W, generator=g), torch.randn(T, W, generator=g)
    y, w, b = (torch.randn(*n, generator=g).to(dtype) for n in ((T, W), (W,), (W,)))
    mix, ow, rd = torch.randn(s, s, generator=g), torch.randn(s, generator=g), torch.randn(s, generator=g)
    alpha = torch.tensor([0.8])
    tol = 2e-6 if dtype == torch.float32 else 5e-3
    to = lambda t: t.to(dev)  # noqa: E731
    for src in (x, x0):
        xs = (src if src.dim() == 3 else src[:, None].expand(T, s, W)).permute(1, 0, 2).double()
        new = O.streams_write(xs, mix.double(), ow.double(), y.double())
        h_ref = O.tanh_norm(O.streams_read(new, rd.double()), alpha.double(), w.double(), b.double()) * 1.7
        for inplace in ([False, True] if src is x else [False]):
            xin = to(src).clone()
            xo = xin if inplace else torch.empty((T, s, W), device=dev)
            h = torch.empty((T, W), dtype=dtype, device=dev)
            mixops.stream_norm(xin, s, y=to(y), mix=to(mix), out_w=to(ow), x_out=xo, read=to(rd), norm=(to(w), to(b), to(alpha)), scale=1.7, h_out=h)
            assert rel(xo.double().cpu().permute(1, 0, 2), new) < 2e-6
            assert rel(h.double().cpu(), h_ref) < tol
        h = torch.empty((T, W), dtype=dtype, device=dev)
        mixops.stream_norm(to(src).contiguous(), s, norm=(to(w), to(b), to(alpha)), h_out=h)
        assert rel(h.double().cpu(), O.tanh_norm(xs.sum(0), alpha.double(), w.double(), b.double())) < tol
        xo = torch.empty((T, s, W), device=dev)
        mixops.stream_norm(to(src).contiguous(), s, y=to(y), mix=to(mix), out_w=to(ow), x_out=xo)
        assert rel(xo.double().cpu().permute(1, 0, 2), new) < 2e-6


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("N", [8, 56, 33])
def test_clamped_gate_kernel(dev, dtype, N):
    from mini_sglang_amd import mixops

    gu = (torch.randn(11, 2 * N, generator=torch.Generator().manual_seed(N)) * 3).to(dtype)
    got = mixops.clamp_gate(gu.to(dev), 1.3, 1.5).double().cpu()
    a, u = gu.double()[:, :N].clamp(max=1.3), gu.double()[:, N:].clamp(-1.3, 1.3)
    assert rel(got, a * O.sigmoid(1.5 * a) * (u + 1.0)) < (1e-6 if dtype == torch.float32 else 5e-3)


# ----------------------------------------------------------------------------------------- schedules
@pytest.mark.parametrize("dtype,tol", [(torch.float32, FP32_TOL), (torch.bfloat16, BF16_TOL)], ids=["fp32", "bf16"])
def test_whole_prompt(dtype, tol):
    toks = tokens_of(150, FULL["vocab"], 21)
    check(engine_for(FULL, dtype), FULL, alone("a", toks, [150]), {"a": toks}, tol)


def test_prefill_against_token_by_token_fp32():
    eng = engine_for(FULL, torch.float32)
    toks = tokens_of(60, FULL["vocab"], 22)
    whole = check(eng, FULL, alone("a", toks, [60]), {"a": toks}, FP32_TOL)["a"]
    single = check(eng, FULL, alone("a", toks, [1]), {"a": toks}, FP32_TOL)["a"]
    assert rel(single, whole) < FP32_TOL


@pytest.mark.parametrize("sizes", [[2], [3, 1], [5, 2, 17], [16], [64, 1, 1, 2], [33, 31]],
                         ids=["twos", "3-1", "5-2-17", "pages", "64-then-short", "33-31"])
def test_portions_fp32(sizes):
    """Prompts cut anywhere: inside a page, a window, a 16-token piece of a recurrence; portions down to two tokens and one."""
    toks = tokens_of(100, FULL["vocab"], 23)
    check(engine_for(FULL, torch.float32), FULL, alone("a", toks, sizes), {"a": toks}, FP32_TOL)


def test_long_portions_run_as_parallel_chunks_fp32():
    """Portions long enough that the recurrences run as parallel pieces joined by a second launch, continued from a carried state."""
    cfg = config([gla(mlp=dense()), att(window=150, keep=30, mlp=None), ret(decay=[0.9, 0.999, 0.99999], mlp=None), gla(heads=1, dim=40, vdim=70, tau=0.5)])
    toks = tokens_of(1300, cfg["vocab"], 24)
    eng = engine_for(cfg, torch.float32, max_tokens=1536)
    got = check(eng, cfg, alone("a", toks, [1100, 3, 197]), {"a": toks}, FP32_TOL)["a"]
    again = replay(eng[0], alone("a", toks, [150, 640, 510]))["a"]
    assert rel(again, got) < FP32_TOL


def test_long_decoding_fp32():
    """A short prompt, then 150 tokens one by one: the windows pass over decoded tokens, the states are carried 150 times."""
    toks = tokens_of(170, FULL["vocab"], 25)
    check(engine_for(FULL, torch.float32), FULL, alone("a", toks, [20] + [1] * 150), {"a": toks}, FP32_TOL)


def test_first_tokens_fp32():
    """Sequences of one, two and three tokens: shorter than the windows, the kept keys and a page."""
    eng = engine_for(FULL, torch.float32)
    for n in (1, 2, 3):
        toks = tokens_of(n, FULL["vocab"], 30 + n)
        check(eng, FULL, alone("a", toks, [n]), {"a": toks}, FP32_TOL)
        check(eng, FULL, alone("a", toks, [1]), {"a": toks}, FP32_TOL)


def test_mixed_batches_against_each_alone_fp32():
    """Four requests of unequal length: portions of some beside single tokens of others, requests that sit out steps."""
    eng = engine_for(FULL, torch.float32)
    seqs = {r: tokens_of(n, FULL["vocab"], 40 + i) for i, (r, n) in enumerate((("a", 90), ("b", 37), ("c", 5), ("d", 61)))}
    a, b, c, d = (seqs[r] for r in "abcd")
    steps = [[("a", a[:50], False), ("b", b[:2], False)],
             [("a", a[50:51], False), ("b", b[2:30], False), ("c", c[:3], False)],
             [("d", d[:40], False), ("a", a[51:52], False), ("c", c[3:4], False)],
             [("a", a[52:88], False), ("b", b[30:], True), ("c", c[4:], True), ("d", d[40:41], False)],
             [("d", d[41:], True), ("a", a[88:], True)]]
    got = check(eng, FULL, steps, seqs, FP32_TOL)
    for r, toks in seqs.items():
        assert rel(replay(eng[0], alone(r, toks, [len(toks)]))[r], got[r]) < FP32_TOL, r


def test_mixed_batches_with_chunks_fp32():
    """A portion long enough for parallel pieces beside single tokens and short portions of other requests in one step."""
    eng = engine_for(FULL, torch.float32, max_tokens=1024)
    a, b, c = tokens_of(400, FULL["vocab"], 45), tokens_of(60, FULL["vocab"], 46), tokens_of(9, FULL["vocab"], 47)
    steps = [[("b", b[:40], False), ("c", c[:8], False)], [("b", b[40:41], False), ("a", a[:350], False), ("c", c[8:], True)],
             [("a", a[350:351], False), ("b", b[41:], True)], [("a", a[351:], True)]]
    check(eng, FULL, steps, {"a": a, "b": b, "c": c}, FP32_TOL)


def test_pages_and_state_slots_used_again_fp32():
    """A pool of six pages and two request rows serving six requests in turn: every page and every state row is handed on with its
    last owner's contents."""
    eng = engine_for(FULL, torch.float32, max_tokens=96, rows=2)
    steps, seqs = [], {}
    for i in range(6):
        r, toks = f"r{i}", tokens_of(30 + 3 * i, FULL["vocab"], 50 + i)
        seqs[r] = toks
        steps += alone(r, toks, [17, 1, 40])
    check(eng, FULL, steps, seqs, FP32_TOL)


def test_other_orders_and_sizes_bf16():
    cfg = config([gla(heads=4, dim=64, vdim=64, mlp=dense(ff=128)), att(heads=8, kv_heads=2, dim=32, vdim=32, dims=16, window=40, mlp=dense(ff=96)),
                  ret(heads=4, dim=32, vdim=128, dims=32, mlp=dense(ff=160)), gla(heads=1, dim=128, vdim=128, mlp=None)], width=128, vocab=200, streams=4)
    a, b = tokens_of(340, 200, 61), tokens_of(33, 200, 62)
    steps = [[("a", a[:300], False)], [("a", a[300:301], False), ("b", b[:20], False)], [("a", a[301:], True), ("b", b[20:], True)]]
    check(engine_for(cfg, torch.bfloat16), cfg, steps, {"a": a, "b": b}, BF16_TOL)


def test_wider_model_with_odd_head_sizes():
    """Head sizes that are no powers of two, three key heads, five streams; two requests whose portions and single tokens share steps."""
    cfg = config([att(heads=6, kv_heads=3, dim=40, vdim=56, dims=24, window=33, keep=5, mlp=dense(ff=200)), ret(heads=3, dim=72, vdim=88, dims=36, mlp=None),
                  gla(heads=5, dim=24, vdim=136, mlp=dense(ff=104))], width=192, vocab=333, streams=5)
    a, b = tokens_of(120, 333, 63), tokens_of(70, 333, 64)
    steps = [[("a", a[:64], False)], [("a", a[64:65], False), ("b", b[:50], False)], [("a", a[65:66], False), ("b", b[50:51], False)],
             [("a", a[66:], True), ("b", b[51:], True)]]
    check(engine_for(cfg, torch.bfloat16), cfg, steps, {"a": a, "b": b}, BF16_TOL)
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


def test_trace_command_line(tmp_path):
    """bin/trace_run end to end in its own process on a checkpoint folder written here: the model class comes from config.json, the inner
    size of the decay projection from the checkpoint."""
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np
    from safetensors.torch import save_file

    from mini_sglang_amd.hybrid import HybridDecoder, nagezen_config

    cfg = config([att(heads=3, kv_heads=1, dim=10, vdim=14, dims=4, window=12, mlp=dense(ff=44)), gla(heads=3, dim=10, vdim=18, mlp=None),
                  ret(heads=2, dim=14, vdim=7, dims=6, mlp=dense(ff=20))], width=100, vocab=131, streams=3)
    model = HybridDecoder(nagezen_config(cfg, shapes_of(cfg)), dtype=torch.bfloat16, device=torch.device("cpu"), seed=9)
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
