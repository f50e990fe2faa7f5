"""A plain, slow restatement of the Nagezen design in float64 torch: one function per mechanism, whole sequences only, token
loops where the design has a recurrence.  It shares no code with the product path; tests hand it a configuration dictionary
(the layout of the design's config.json) and a checkpoint dictionary (checkpoint tensor names) and compare.

Notation: T tokens of one sequence, positions 0 .. T - 1; W = width; every weight matrix is [out, in] and applied as x @ M^T.
"""
from __future__ import annotations

import math
from typing import Any, Dict, List, Optional, Tuple

import torch

F64 = torch.float64


def _w(state: Dict[str, torch.Tensor], name: str) -> torch.Tensor:
    return state[name].to(F64)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over the root of its mean square along the last axis, eps under the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def tanh_norm(x: torch.Tensor, alpha: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """An element-wise squashing in the place of a norm: no statistic of the row enters."""
    return torch.tanh(alpha * x) * w + b


def streams_read(xs: torch.Tensor, read: torch.Tensor) -> torch.Tensor:
    """xs [s, T, W], read [s] -> the row a sublayer gets: the streams weighed by `read`."""
    return (xs * read[:, None, None]).sum(dim=0)


def streams_write(xs: torch.Tensor, mix: torch.Tensor, out: torch.Tensor, y: torch.Tensor) -> torch.Tensor:
    """new stream t = sum over streams s of mix[s, t] (row: from, column: to) times the old stream s, plus out[t] y."""
    new = []
    for t in range(xs.shape[0]):
        row = out[t] * y
        for s in range(xs.shape[0]):
            row = row + mix[s, t] * xs[s]
        new.append(row)
    return torch.stack(new)


def rotary(dims: int, base: float, scaling: Optional[Dict[str, float]]) -> Tuple[torch.Tensor, float]:
    """-> (angle per position of every pair, factor on cos and sin)."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return torch.tensor(f, dtype=F64), 1.0
    factor, orig = float(scaling["factor"]), float(scaling["original"])

    def where(turns: float) -> float:  # the (fractional) pair that makes `turns` turns over the original context
        return dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(where(float(scaling["fast"]))), 0)
    hi = min(math.ceil(where(float(scaling["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(factor) + 1.0


def rotate(v: torch.Tensor, freqs: torch.Tensor, amp: float, pos: torch.Tensor) -> torch.Tensor:
    """v [T, heads, n]: the first 2 * len(freqs) entries of each head turn, entry i paired with entry i + len(freqs)."""
    half = freqs.shape[0]
    if half == 0:
        return v
    a = pos.to(F64)[:, None, None] * freqs[None, None, :]
    c, s = torch.cos(a) * amp, torch.sin(a) * amp
    u, w = v[..., :half], v[..., half: 2 * half]
    return torch.cat((u * c - w * s, w * c + u * s, v[..., 2 * half:]), dim=-1)


def decayed_outer_sum(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor,
                      S0: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """q, k, decay [T, H, d], v [T, H, dv]:  S <- diag(decay_t) S + k_t v_t^T,  o_t = S^T q_t  -> (o [T, H, dv], last S)."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64) if S0 is None else S0.clone()
    o = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(dim=1)
    return o, S


def retention(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ _w(st, p + "q").T).reshape(T, H, d)
    k = (h @ _w(st, p + "k").T).reshape(T, H, d)
    v = (h @ _w(st, p + "v").T).reshape(T, H, dv)
    rot = m.get("rot") or {}
    if rot.get("dims"):
        freqs, amp = rotary(int(rot["dims"]), float(rot["base"]), rot.get("scaling"))
        q, k = rotate(q, freqs, amp, torch.arange(T)), rotate(k, freqs, amp, torch.arange(T))
    decay = torch.tensor([float(x) for x in m["decay"]], dtype=F64)[None, :, None].expand(T, H, d)
    o, _ = decayed_outer_sum(q, k * d ** -0.5, v, decay)
    return (rms_unit(o, eps).reshape(T, H * dv) * silu(h @ _w(st, p + "g").T)) @ _w(st, p + "o").T


def channel_decay(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, m: Dict[str, Any]) -> torch.Tensor:
    """-> [T, H, d] decays in (0, 1): the tau-th root of a sigmoid of a two-step projection with a bias."""
    z = (h @ _w(st, p + "a1").T) @ _w(st, p + "a2").T + _w(st, p + "a2.b")
    return (sigmoid(z) ** (1.0 / float(m["tau"]))).reshape(h.shape[0], int(m["heads"]), int(m["dim"]))


def gla(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ _w(st, p + "q").T).reshape(T, H, d) * d ** -0.5
    k = (h @ _w(st, p + "k").T).reshape(T, H, d)
    v = (h @ _w(st, p + "v").T).reshape(T, H, dv)
    o, _ = decayed_outer_sum(q, k, v, channel_decay(h, st, p, m))
    o = rms_unit(o, eps) * _w(st, p + "norm")
    return (o.reshape(T, H * dv) * silu(h @ _w(st, p + "g").T)) @ _w(st, p + "o").T


def visible(i: int, window: int, keep_first: int) -> List[int]:
    """The keys token i sees: the last `window` ones (all when 0), itself included, and the first `keep_first` of the sequence."""
    return [j for j in range(i + 1) if window <= 0 or i - j < window or j < keep_first]


def masked_softmax(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, window: int, keep_first: int) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv], query head h on key head h // (H / G)."""
    T, H, _ = q.shape
    G, dv = k.shape[1], v.shape[2]
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        js = torch.tensor(visible(i, window, keep_first))
        for hh in range(H):
            g = hh // (H // G)
            out[i, hh] = torch.softmax((k[js, g] @ q[i, hh]) * scale, dim=0) @ v[js, g]
    return out


def difference_weight(st: Dict[str, torch.Tensor], p: str, diff: float) -> float:
    a = torch.exp((_w(st, p + "lq1") * _w(st, p + "lk1")).sum())
    b = torch.exp((_w(st, p + "lq2") * _w(st, p + "lk2")).sum())
    return float(a - b) + diff


def differential_attention(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m["vdim"])
    q = (h @ _w(st, p + "q").T + _w(st, p + "q.b")).reshape(T, H, 2, d)
    k = (h @ _w(st, p + "k").T + _w(st, p + "k.b")).reshape(T, G, 2, d)
    v = (h @ _w(st, p + "v").T + _w(st, p + "v.b")).reshape(T, G, dv)
    q, k = rms_unit(q, eps) * _w(st, p + "q.norm"), rms_unit(k, eps) * _w(st, p + "k.norm")
    rot = m.get("rot") or {}
    freqs, amp = rotary(int(rot["dims"]), float(rot["base"]), rot.get("scaling")) if rot.get("dims") else (torch.zeros(0, dtype=F64), 1.0)
    mask = m.get("mask") or {}
    maps = []
    for a in range(2):
        qa, ka = rotate(q[:, :, a], freqs, amp, torch.arange(T)), rotate(k[:, :, a], freqs, amp, torch.arange(T))
        maps.append(masked_softmax(qa, ka, v, float(m["scale"]), int(mask.get("size", 0)), int(mask.get("keep_first", 0))))
    diff = float(m["diff"])
    o = maps[0] - difference_weight(st, p, diff) * maps[1]
    o = rms_unit(o, eps) * (1.0 - diff)
    return (o.reshape(T, H * dv) * sigmoid(h @ _w(st, p + "g").T)) @ _w(st, p + "o").T


def clamped_ff(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, limit: float) -> torch.Tensor:
    g = torch.clamp(h @ _w(st, p + "gate").T, max=limit)
    u = torch.clamp(h @ _w(st, p + "up").T, min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ _w(st, p + "down").T


MIXERS = {"retention": retention, "gla": gla, "attention": differential_attention}


def forward(cfg: Dict[str, Any], st: Dict[str, torch.Tensor], tokens) -> Tuple[torch.Tensor, torch.Tensor]:
    """-> (logits [T, vocab], the sum of the streams after every layer [layers, T, W]) in float64."""
    eps, n = float(cfg["norm"]["eps"]), int(cfg["streams"])

    def norm(x, name):
        return tanh_norm(x, _w(st, name + ".alpha"), _w(st, name), _w(st, name + ".b"))

    xs = _w(st, "embed")[torch.as_tensor(tokens, dtype=torch.long)][None].repeat(n, 1, 1)
    after = []
    for i, entry in enumerate(cfg["layers"]):
        hc = f"l{i}.hc1."
        y = MIXERS[entry["type"]](norm(streams_read(xs, _w(st, hc + "in")), f"l{i}.norm1"), st, f"l{i}.mix.", entry["mixer"], eps)
        xs = streams_write(xs, _w(st, hc + "mix"), _w(st, hc + "out"), y)
        if entry.get("mlp") is not None:
            hc = f"l{i}.hc2."
            y = clamped_ff(norm(streams_read(xs, _w(st, hc + "in")), f"l{i}.norm2"), st, f"l{i}.mlp.", float(entry["mlp"]["limit"]))
            xs = streams_write(xs, _w(st, hc + "mix"), _w(st, hc + "out"), y)
        after.append(xs.sum(dim=0))
    logits = norm(xs.sum(dim=0), "final.norm") @ _w(st, "head").T * float(cfg.get("logit_scale", 1.0))
    return logits, torch.stack(after)
