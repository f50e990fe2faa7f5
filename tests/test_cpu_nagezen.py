"""CPU-side tests of the multi-stream hybrid decoder (Nagezen): configuration reader, registry, rotary table, checkpoint round trip,
cache layout and byte counts, and the plain restatement's own consistency (tests/nagezen_oracle.py).  No GPU."""
from __future__ import annotations

import json
import math

import pytest
import torch

import nagezen_oracle as O


def _cfg():
    dense = {"kind": "dense", "ff": 20, "limit": 0.9}
    att = {"type": "attention", "mlp": dense,
           "mixer": {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 6, "scale": 0.35, "diff": 0.2, "mask": {"size": 7, "keep_first": 2},
                     "rot": {"base": 100.0, "dims": 4, "scaling": {"factor": 4.0, "fast": 2.0, "slow": 0.5, "original": 16}}}}
    ret = {"type": "retention", "mlp": None, "mixer": {"heads": 3, "dim": 6, "vdim": 10, "decay": [0.5, 0.9, 0.99], "rot": {"base": 77.0, "dims": 6}}}
    gla = {"type": "gla", "mlp": dense, "mixer": {"heads": 2, "dim": 5, "vdim": 9, "tau": 3.0}}
    return {"architecture": "Nagezen", "vocab": 50, "width": 24, "norm": {"eps": 1e-5}, "layers": [gla, att, ret], "streams": 3, "logit_scale": 0.7}


SHAPES = {"l0.mix.a1": (7, 24)}


def _model(seed):
    from mini_sglang_amd.hybrid import HybridDecoder, nagezen_config

    return HybridDecoder(nagezen_config(_cfg(), SHAPES), dtype=torch.float32, device=torch.device("cpu"), seed=seed)


def test_config_reader_and_registry(tmp_path):
    from safetensors.torch import save_file

    from mini_sglang_amd.hybrid import DenseFfSpec, HybridConfig, HybridDecoder, nagezen_config
    from mini_sglang_amd.registry import architecture_of, load_model_dir, model_class

    raw = _cfg()
    assert architecture_of(raw) == "Nagezen"
    cfg = nagezen_config(raw, SHAPES)
    assert isinstance(cfg, HybridConfig) and cfg.residual == "streams" and model_class(cfg) is HybridDecoder
    assert (cfg.streams, cfg.logit_scale, cfg.vocab_size, cfg.hidden_size, cfg.rms_norm_eps) == (3, 0.7, 50, 24, 1e-5)
    g, a, r = cfg.layers
    assert (g.kind, g.heads, g.dim, g.vdim, g.tau, g.decay_rank, g.recurrent) == ("gla", 2, 5, 9, 3.0, 7, True)
    assert (a.kind, a.heads, a.kv_heads, a.maps, a.window, a.keep_first, a.diff, a.scale) == ("diff_attention", 4, 2, 2, 7, 2, 0.2, 0.35)
    assert dict(a.rot_scaling) == {"factor": 4.0, "fast": 2.0, "slow": 0.5, "original": 16.0} and not a.recurrent
    assert (r.kind, r.decay, r.rot_dims, r.rot_base, r.mlp, r.recurrent) == ("retention", (0.5, 0.9, 0.99), 6, 77.0, None, True)
    assert isinstance(a.mlp, DenseFfSpec) and (a.mlp.act, a.mlp.limit, a.mlp.slope, a.mlp.gated) == ("clamp_gate", 0.9, 1.702, True)
    # the inner size of the decay projection comes from the checkpoint's header
    (tmp_path / "config.json").write_text(json.dumps(raw))
    save_file(_model(1).export_state(), str(tmp_path / "model.safetensors"))
    got, name = load_model_dir(tmp_path)
    assert name == "Nagezen" and got == cfg
    plain = _cfg()
    del plain["streams"], plain["logit_scale"], plain["layers"][1]["mixer"]["mask"], plain["layers"][1]["mixer"]["rot"], plain["layers"][2]["mixer"]["rot"]
    c2 = nagezen_config(plain)
    assert (c2.streams, c2.logit_scale, c2.layers[1].window, c2.layers[1].keep_first, c2.layers[1].rot_dims, c2.layers[2].rot_dims) == (1, 1.0, 0, 0, 0, 0)
    for edit in (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), lambda c: c["layers"][2]["mixer"].update(heads=2),
                 lambda c: c["layers"][2]["mixer"]["rot"].update(dims=8), lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3),
                 lambda c: c["layers"][0].update(type="lightning"), lambda c: c["layers"][0]["mlp"].update(kind="moe"), lambda c: c.update(streams=0)):
        bad = json.loads(json.dumps(_cfg()))
        edit(bad)
        with pytest.raises(ValueError):
            nagezen_config(bad)


@pytest.mark.parametrize("dims,base,sc", [(12, 50.0, {"factor": 8.0, "fast": 4.0, "slow": 1.0, "original": 64}), (4, 1e6, None),
                                          (8, 10.0, {"factor": 2.0, "fast": 1.0, "slow": 1.0, "original": 700}),
                                          (16, 1e4, {"factor": 3.0, "fast": 1e6, "slow": 1e-9, "original": 512})])
def test_rotary_table_with_ramped_frequencies(dims, base, sc):
    from mini_sglang_amd.hybrid import LayerSpec, rotary_table

    spec = LayerSpec(kind="diff_attention", heads=1, dim=dims, vdim=4, rot_dims=dims, rot_base=base, rot_scaling=tuple(sorted(sc.items())) if sc else None)
    f, amp = O.rotary(dims, base, sc)
    ang = torch.arange(40, dtype=torch.float64)[:, None] * f
    assert torch.allclose(rotary_table(spec, 40, "cpu").double(), torch.cat((ang.cos() * amp, ang.sin() * amp), 1), atol=1e-6)
    plain, one = O.rotary(dims, base, None)
    assert one == 1.0
    if sc:
        assert bool(((f <= plain * (1 + 1e-12)) & (f >= plain / sc["factor"] * (1 - 1e-12))).all())


def test_checkpoint_round_trip_and_cache_layout():
    from mini_sglang_amd.kvcache import HybridCache

    a, b = _model(1), _model(2)
    state = a.export_state()
    assert state["head"].shape == (50, 24) and state["final.norm"].shape == (24,) and state["final.norm.alpha"].shape == ()
    assert state["l0.mix.q"].shape == (10, 24) and state["l0.mix.v"].shape == (18, 24) and state["l0.mix.a1"].shape == (7, 24)
    assert state["l0.mix.a2"].shape == (10, 7) and state["l0.mix.a2.b"].shape == (10,) and state["l0.mix.norm"].shape == (9,)
    assert state["l1.mix.q"].shape == (64, 24) and state["l1.mix.k"].shape == (32, 24) and state["l1.mix.v"].shape == (12, 24)
    assert state["l1.mix.q.b"].shape == (64,) and state["l1.mix.k.norm"].shape == (8,) and state["l1.mix.lk2"].shape == (8,)
    assert state["l1.mix.g"].shape == (24, 24) and state["l1.mlp.gate"].shape == (20, 24) and state["l1.hc2.mix"].shape == (3, 3)
    assert state["l2.mix.o"].shape == (24, 30) and "l2.norm2" not in state and "l2.hc2.in" not in state and "l2.mix.norm" not in state
    assert a.weight_bytes() == sum(4 * v.numel() for v in state.values())
    where = b.layers[1].lam_now.data_ptr()
    b.load_state(state)
    again = b.export_state()
    assert set(again) == set(state)
    for k, v in state.items():
        assert torch.equal(again[k], v), k
    # what a captured graph reads is written where it was
    assert b.layers[1].lam_now.data_ptr() == where and abs(float(b.layers[1].lam_now) - O.difference_weight(state, "l1.mix.", 0.2)) < 1e-6
    layers = a.cfg.cache_layers
    kv = HybridCache(layers, num_pages=4, page_size=16, state_rows=3, dtype=torch.bfloat16, device=torch.device("cpu"))
    assert kv.state(0).shape == (3, 2, 5, 9) and kv.state(2).shape == (3, 3, 6, 10) and kv.state(2).dtype == torch.float32
    k1, v1 = kv.kv_rows(1)
    assert k1.shape == (64, 32) and v1.shape == (64, 12)
    assert HybridCache.bytes_per_page(layers, 16, torch.bfloat16) == 2 * (32 + 12) * 16
    assert HybridCache.state_bytes(layers, 3, torch.bfloat16) == 4 * 3 * (2 * 5 * 9 + 3 * 6 * 10)


def test_piece_size_of_the_recurrences():
    from mini_sglang_amd.attention import MixAttnBackend

    for tokens, heads in ((1, 1), (300, 3), (2048, 8), (8192, 16), (65536, 64)):
        c = MixAttnBackend.decay_chunk(tokens, heads)
        assert c % 16 == 0 and 32 <= c <= 512
        assert c == 512 or -(-tokens // c) * heads <= 512 or c == 32
    assert MixAttnBackend.decay_chunk(2048, 16) == 64


def test_restatement_by_hand():
    f = torch.float64
    # two streams, (1, 10) and (2, 20): read (0.5, 2); mixing rows are where a stream comes FROM
    xs = torch.tensor([[[1.0, 10.0]], [[2.0, 20.0]]], dtype=f)
    assert torch.equal(O.streams_read(xs, torch.tensor([0.5, 2.0], dtype=f)), torch.tensor([[4.5, 45.0]], dtype=f))
    got = O.streams_write(xs, torch.tensor([[1.0, 3.0], [0.0, 2.0]], dtype=f), torch.tensor([1.0, -1.0], dtype=f), torch.tensor([[100.0, 0.0]], dtype=f))
    assert torch.equal(got, torch.tensor([[[101.0, 10.0]], [[3 + 4 - 100.0, 30 + 40.0]]], dtype=f))
    assert torch.allclose(O.tanh_norm(torch.tensor([0.0, 1e9], dtype=f), torch.tensor(2.0, dtype=f), torch.tensor([5.0, 3.0], dtype=f),
                                      torch.tensor([1.0, -1.0], dtype=f)), torch.tensor([1.0, 2.0], dtype=f))
    assert O.visible(6, 3, 2) == [0, 1, 4, 5, 6] and O.visible(2, 3, 2) == [0, 1, 2] and O.visible(3, 0, 0) == [0, 1, 2, 3] and O.visible(4, 1, 0) == [4]
    # one head, one key channel: S = 2 * 3, then 0.5 * 6 + 1 * 4
    o, S = O.decayed_outer_sum(torch.ones(2, 1, 1, dtype=f), torch.tensor([2.0, 1.0], dtype=f).view(2, 1, 1), torch.tensor([3.0, 4.0], dtype=f).view(2, 1, 1),
                               torch.full((2, 1, 1), 0.5, dtype=f))
    assert o.flatten().tolist() == [6.0, 7.0] and float(S) == 7.0
    q = torch.zeros(3, 1, 1, dtype=f)
    v = torch.tensor([4.0, 6.0, 8.0], dtype=f).view(3, 1, 1)
    assert O.masked_softmax(q, q, v, 1.0, 1, 1).flatten().tolist() == [4.0, 5.0, 6.0]
    h, st = torch.tensor([[10.0], [-10.0]], dtype=f), {"p.gate": torch.ones(1, 1), "p.up": torch.ones(1, 1), "p.down": torch.ones(1, 1)}
    sg = lambda z: 1 / (1 + math.exp(-z))  # noqa: E731
    assert torch.allclose(O.clamped_ff(h, st, "p.", 2.0).flatten(), torch.tensor([2 * sg(3.404) * 3, -10 * sg(-17.02) * -1.0], dtype=f))


def test_restatement_is_causal():
    raw = _cfg()
    state = _model(3).export_state()
    g = torch.Generator().manual_seed(1)
    toks = torch.randint(0, 50, (20,), generator=g).tolist()
    logits, after = O.forward(raw, state, toks)
    assert logits.shape == (20, 50) and after.shape == (3, 20, 24)
    head, _ = O.forward(raw, state, toks[:13])
    assert torch.allclose(head, logits[:13], atol=1e-9)
    q, k, v = (torch.randn(9, 2, n, generator=g, dtype=torch.float64) for n in (3, 3, 4))
    a = torch.rand(9, 2, 3, generator=g, dtype=torch.float64)
    whole, S = O.decayed_outer_sum(q, k, v, a)
    o1, S1 = O.decayed_outer_sum(q[:4], k[:4], v[:4], a[:4])
    o2, S2 = O.decayed_outer_sum(q[4:], k[4:], v[4:], a[4:], S0=S1)
    assert torch.allclose(torch.cat([o1, o2]), whole, atol=1e-12) and torch.allclose(S2, S, atol=1e-12)
