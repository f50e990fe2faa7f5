"""CPU-side tests of the looped sandwich-norm decoder (Redasun): configuration reader, registry, checkpoint round trip, cache layout and
byte counts, and the plain restatement by hand (tests/redasun_oracle.py).  No GPU."""
from __future__ import annotations

import json
import math

import pytest
import torch

import redasun_oracle as O


def _cfg():
    mixer = {"heads": 6, "kv_heads": 3, "dim": 10, "vdim": 14, "scale": 0.4, "diff": 0.3, "rot": {"base": 300.0, "dims": 6}}
    other = {"heads": 2, "dim": 8, "vdim": 5, "scale": 0.5, "diff": 0.1, "rot": {"base": 50.0, "dims": 8}}
    moe = {"kind": "moe", "expert": {"ff": 12}, "router": {"experts": 8, "top": 3, "scale": 1.7, "groups": {"count": 4, "keep": 2}}, "shared": {"ff": 18}}
    layers = [{"type": "attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": 20}}, {"type": "attention", "mixer": other, "mlp": moe},
              {"type": "attention", "mixer": mixer, "mlp": None}]
    return {"architecture": "Redasun", "vocab": 50, "width": 24, "norm": {"eps": 1e-4}, "embedding": {"scale": 3.0}, "layers": layers,
            "loop": {"start": 0, "stop": 2, "times": 3}}


def _model(seed, raw=None):
    from mini_sglang_amd.hybrid import HybridDecoder, redasun_config

    return HybridDecoder(redasun_config(raw or _cfg()), dtype=torch.float32, device=torch.device("cpu"), seed=seed)


def test_config_reader_and_registry(tmp_path):
    from safetensors.torch import save_file

    from mini_sglang_amd.hybrid import DenseFfSpec, HybridConfig, HybridDecoder, MoeSpec, redasun_config
    from mini_sglang_amd.registry import architecture_of, load_model_dir, model_class

    raw = _cfg()
    assert architecture_of(raw) == "Redasun"
    cfg = redasun_config(raw)
    assert isinstance(cfg, HybridConfig) and cfg.residual == "sandwich" and cfg.norm_centre and model_class(cfg) is HybridDecoder
    assert (cfg.vocab_size, cfg.hidden_size, cfg.rms_norm_eps, cfg.embed_scale, cfg.loop) == (50, 24, 1e-4, 3.0, (0, 2, 3))
    a, b, c = cfg.layers
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.diff, a.maps) == ("diff_attention", 6, 3, 10, 14, 0.4, 0.3, 2)
    assert (a.rot_dims, a.rot_base, a.rot_scaling, a.window, a.keep_first, a.out_gate, a.proj_bias, a.recurrent) == (6, 300.0, None, 0, 0, False, False, False)
    assert b.kv_heads == 2  # as many key heads as heads where config.json names none
    assert a.mlp == DenseFfSpec(ff=20, act="gelu_gate") and a.mlp.gated and c.mlp is None
    assert b.mlp == MoeSpec(experts=8, top=3, ff=12, groups=4, keep=2, gated=True, pick="sigmoid_scores", group_best=2, scale=1.7, shared_ff=18)
    assert cfg.runs == ((0, 0), (1, None), (0, 1), (1, None), (0, 2), (1, None), (2, None)) and len(cfg.cache_layers) == 7
    (tmp_path / "config.json").write_text(json.dumps(raw))
    save_file(_model(1).export_state(), str(tmp_path / "model.safetensors"))
    assert load_model_dir(tmp_path) == (cfg, "Redasun")
    plain = _cfg()
    del plain["loop"], plain["embedding"], plain["layers"][1]["mlp"]["shared"], plain["layers"][1]["mlp"]["router"]["groups"]
    del plain["layers"][1]["mlp"]["router"]["scale"], plain["layers"][2]["mixer"]
    plain["layers"][2]["mixer"] = {"heads": 1, "dim": 4, "vdim": 4, "scale": 1.0, "diff": 0.0}
    c2 = redasun_config(plain)
    m2 = c2.layers[1].mlp
    assert (c2.loop, c2.embed_scale, m2.groups, m2.keep, m2.scale, m2.shared_ff, c2.layers[2].rot_dims) == (None, 1.0, 1, 1, 1.0, 0, 0)
    for edit in (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=12),
                 lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3), lambda c: c["layers"][0].update(type="lightning"),
                 lambda c: c["layers"][0]["mlp"].update(kind="sparse"), lambda c: c["loop"].update(stop=4), lambda c: c["loop"].update(start=2),
                 lambda c: c["loop"].update(times=0), lambda c: c["layers"][1]["mlp"]["router"].update(experts=9),
                 lambda c: c["layers"][1]["mlp"]["router"].update(top=5), lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=5)):
        bad = json.loads(json.dumps(_cfg()))
        edit(bad)
        with pytest.raises(ValueError):
            redasun_config(bad)


def test_checkpoint_round_trip_and_cache_layout():
    from mini_sglang_amd.kvcache import HybridCache

    a, b = _model(1), _model(2)
    state = a.export_state()
    assert "head" not in state and state["loop.in"].shape == (24, 48) and state["final.norm"].shape == (24,)
    assert state["l0.mix.q"].shape == (120, 24) and state["l0.mix.k"].shape == (60, 24) and state["l0.mix.v"].shape == (42, 24)
    assert state["l0.mix.q.norm"].shape == (10,) and state["l0.mix.lk2"].shape == (10,) and state["l0.mix.o"].shape == (24, 84)
    assert "l0.mix.g" not in state and "l0.mix.q.b" not in state and "l2.norm2" not in state and "l2.norm2b" not in state and "l2.norm1b" in state
    assert state["l1.mlp.router"].shape == (8, 24) and state["l1.mlp.correction"].shape == (8,) and state["l1.mlp.e7.down"].shape == (24, 12)
    assert state["l1.mlp.shared.gate"].shape == (18, 24) and state["l0.mlp.up"].shape == (20, 24)
    assert a.weight_bytes() == sum(4 * v.numel() for v in state.values())
    where = b.layers[0].lam_now.data_ptr()
    b.load_state(state)
    again = b.export_state()
    assert set(again) == set(state)
    for k, v in state.items():
        assert torch.equal(again[k], v), k
    # what a captured graph reads is written where it was
    assert b.layers[0].lam_now.data_ptr() == where and abs(float(b.layers[0].lam_now) - O.second_map_weight(state, "l0.mix.", 0.3)) < 1e-6
    with pytest.raises(ValueError):
        b.load_state(dict(state, **{"l0.norm1b": torch.zeros(23)}))
    layers = a.cfg.cache_layers  # one entry per layer RUN
    kv = HybridCache(layers, num_pages=4, page_size=16, state_rows=3, dtype=torch.bfloat16, device=torch.device("cpu"))
    assert [kv.kv_rows(i)[0].shape[1] for i in range(7)] == [60, 32, 60, 32, 60, 32, 60]
    assert kv.kv_rows(0)[1].shape == (64, 42) and kv.kv_rows(2)[0].data_ptr() != kv.kv_rows(0)[0].data_ptr()
    assert HybridCache.bytes_per_page(layers, 16, torch.bfloat16) == 2 * 16 * (4 * (60 + 42) + 3 * (32 + 10))
    assert HybridCache.state_bytes(layers, 3, torch.bfloat16) == 0


def test_restatement_by_hand():
    f = torch.float64
    # rows 1, 3: mean 2, deviations -1, 1, variance 1
    assert torch.allclose(O.centred_norm(torch.tensor([1.0, 3.0], dtype=f), torch.tensor([2.0, 5.0], dtype=f), 3.0), torch.tensor([-1.0, 2.5], dtype=f))
    z = torch.tensor([0.0, 1.0, -3.0], dtype=f)
    want = [0.5 * v * (1 + math.tanh(math.sqrt(2 / math.pi) * (v + 0.044715 * v ** 3))) for v in (0.0, 1.0, -3.0)]
    assert torch.allclose(O.gelu_tanh(z), torch.tensor(want, dtype=f))
    # two groups of three: the largest choice is in the first, the larger sum of two in the second; all choices negative
    s = torch.tensor([0.9, 0.1, 0.1, 0.6, 0.7, 0.2], dtype=f)
    assert O.choose(s, torch.full((6,), -2.0, dtype=f), 2, 2, 1) == [4, 3]
    assert O.choose(s, torch.tensor([0.0, 0.6, 0.0, -1.0, 0.0, 0.0], dtype=f), 3, 2, 1) == [0, 1, 2]
    assert O.choose(s, torch.zeros(6, dtype=f), 2, 6, 3) == [0, 4]  # groups of one
    assert O.choose(s, torch.tensor([0.0, 0.0, 0.0, 0.0, 0.0, 9.0], dtype=f), 2, 1, 1) == [5, 0]
    # weights: scores without the correction over their sum, times the scale
    eye = torch.eye(2, dtype=f)
    st = {"p.router": torch.tensor([[0.0, 0.0], [math.log(3.0), 0.0], [-50.0, 0.0]], dtype=f), "p.correction": torch.tensor([0.0, 0.0, -9.0], dtype=f)}
    for e, k in ((0, 1.0), (1, 10.0), (2, 1000.0)):
        st[f"p.e{e}.gate"], st[f"p.e{e}.up"], st[f"p.e{e}.down"] = eye, eye, k * eye
    h = torch.tensor([[1.0, 2.0]], dtype=f)
    one = O.silu(h) * h
    got = O.mixture(h, st, "p.", {"router": {"experts": 3, "top": 2, "scale": 5.0}})
    assert torch.allclose(got, one * 5.0 * (0.5 * 1.0 + 0.75 * 10.0) / 1.25)
    q = torch.zeros(3, 1, 1, dtype=f)
    v = torch.tensor([4.0, 6.0, 8.0], dtype=f).view(3, 1, 1)
    assert O.causal_softmax(q, q, v, 1.0).flatten().tolist() == [4.0, 5.0, 6.0]
    turned = O.rotate(torch.tensor([[[1.0, 0.0, 7.0]], [[1.0, 0.0, 7.0]]], dtype=f), 2, 10.0)
    assert torch.allclose(turned[1, 0], torch.tensor([math.cos(1.0), math.sin(1.0), 7.0], dtype=f)) and torch.equal(turned[0, 0], torch.tensor([1.0, 0.0, 7.0], dtype=f))
    assert O.layer_runs({"layers": [0, 0, 0, 0], "loop": {"start": 1, "stop": 3, "times": 2}}) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert O.layer_runs({"layers": [0, 0]}) == [(0, False), (1, False)]


def test_restatement_is_causal_and_reads_the_embedding_in_every_pass():
    raw = _cfg()
    state = _model(3).export_state()
    toks = torch.randint(0, 50, (20,), generator=torch.Generator().manual_seed(1)).tolist()
    logits, after = O.forward(raw, state, toks)
    assert logits.shape == (20, 50) and after.shape == (7, 20, 24)
    head, _ = O.forward(raw, state, toks[:13])
    assert torch.allclose(head, logits[:13], atol=1e-9)
    # with the embedding's half of the joining matrix gone, a later pass no longer sees it
    half = dict(state, **{"loop.in": torch.cat((state["loop.in"][:, :24], torch.zeros(24, 24)), 1)})
    assert float((O.forward(raw, half, toks)[1][2] - after[2]).abs().max()) > 1e-2
