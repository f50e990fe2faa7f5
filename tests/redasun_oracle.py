"""A plain, slow restatement of the Redasun design in float64 torch: one function per mechanism, whole sequences only, one token at a
time where a choice is made.  It shares no code with the product path; tests hand it a configuration dictionary (the layout of the
design's config.json) and a checkpoint dictionary (checkpoint tensor names) and compare.

Notation: T tokens of one sequence, positions 0 .. T - 1; W = width; every weight matrix is [out, in] and applied as x @ M^T.
"""
from __future__ import annotations

import math
from typing import Any, Dict, List, Tuple

import torch

F64 = torch.float64


def _w(state: Dict[str, torch.Tensor], name: str) -> torch.Tensor:
    return state[name].to(F64)


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over the root of its mean square along the last axis, eps under the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def centred_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """The row's mean taken off, the rest over the root of its mean square (eps under the root), times w."""
    return rms_unit(x - x.mean(dim=-1, keepdim=True), eps) * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1.0 + torch.exp(-z))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def gated_ff(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, act) -> torch.Tensor:
    return (act(h @ _w(st, p + "gate").T) * (h @ _w(st, p + "up").T)) @ _w(st, p + "down").T


def rotate(v: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """v [T, heads, n]: entries i and i + dims / 2 (i < dims / 2) of every head turn by position * base^(-2i / dims)."""
    out = v.clone()
    half = dims // 2
    for i in range(half):
        a = torch.arange(v.shape[0], dtype=F64)[:, None] * float(base) ** (-2.0 * i / dims)
        out[..., i] = v[..., i] * torch.cos(a) - v[..., i + half] * torch.sin(a)
        out[..., i + half] = v[..., i + half] * torch.cos(a) + v[..., i] * torch.sin(a)
    return out


def causal_softmax(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; query head h reads key head h // (H / G), token i the keys 0 .. i."""
    T, H, _ = q.shape
    G = k.shape[1]
    later = torch.ones(T, T, dtype=torch.bool).triu(1)
    heads = []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T * scale).masked_fill(later, -math.inf)
        heads.append(torch.softmax(s, dim=1) @ v[:, g])
    return torch.stack(heads, dim=1)


def second_map_weight(st: Dict[str, torch.Tensor], p: str, diff: float) -> float:
    a = math.exp(float((_w(st, p + "lq1") * _w(st, p + "lk1")).sum()))
    b = math.exp(float((_w(st, p + "lq2") * _w(st, p + "lk2")).sum()))
    return a - b + diff


def differential_attention(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m["vdim"])
    q = rms_unit((h @ _w(st, p + "q").T).reshape(T, H, 2, d), eps) * _w(st, p + "q.norm")
    k = rms_unit((h @ _w(st, p + "k").T).reshape(T, G, 2, d), eps) * _w(st, p + "k.norm")
    v = (h @ _w(st, p + "v").T).reshape(T, G, dv)
    rot = m.get("rot") or {}
    turn = (lambda t: rotate(t, int(rot["dims"]), float(rot["base"]))) if rot.get("dims") else (lambda t: t)
    a1, a2 = (causal_softmax(turn(q[:, :, i]), turn(k[:, :, i]), v, float(m["scale"])) for i in range(2))
    diff = float(m["diff"])
    o = rms_unit(a1 - second_map_weight(st, p, diff) * a2, eps) * (1.0 - diff)
    return o.reshape(T, H * dv) @ _w(st, p + "o").T


def choose(scores: torch.Tensor, correction: torch.Tensor, top: int, groups: int, keep: int) -> List[int]:
    """scores, correction [E] of ONE token -> the chosen experts: `top` largest corrected scores among the experts of the `keep`
    groups whose two largest corrected scores have the largest sum."""
    c = (scores + correction).tolist()
    n = len(c) // groups
    worth = [sum(sorted(c[g * n: (g + 1) * n], reverse=True)[:2]) for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: -worth[g])[:keep]
    allowed = [e for e in range(len(c)) if e // n in kept]
    return sorted(allowed, key=lambda e: -c[e])[:top]


def mixture(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, m: Dict[str, Any]) -> torch.Tensor:
    r = m["router"]
    g = r.get("groups") or {}
    count = int(g.get("count", 1))
    scores = 1.0 / (1.0 + torch.exp(-(h @ _w(st, p + "router").T)))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        picks = choose(scores[t], _w(st, p + "correction"), int(r["top"]), count, int(g.get("keep", count)))
        total = sum(float(scores[t, e]) for e in picks) + 1e-20
        for e in picks:
            out[t] += float(scores[t, e]) / total * float(r.get("scale", 1.0)) * gated_ff(h[t][None], st, f"{p}e{e}.", silu)[0]
    if m.get("shared"):
        out = out + gated_ff(h, st, p + "shared.", silu)
    return out


def feed_forward(h: torch.Tensor, st: Dict[str, torch.Tensor], p: str, m: Dict[str, Any]) -> torch.Tensor:
    return gated_ff(h, st, p, gelu_tanh) if m["kind"] == "dense" else mixture(h, st, p, m)


def layer_runs(cfg: Dict[str, Any]) -> List[Tuple[int, bool]]:
    """(layer, does it open a pass of the loop) in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    return [(i, False) for i in range(a)] + [(i, i == a) for _ in range(int(loop["times"])) for i in range(a, b)] + [(i, False) for i in range(b, n)]


def forward(cfg: Dict[str, Any], st: Dict[str, torch.Tensor], tokens) -> Tuple[torch.Tensor, torch.Tensor]:
    """-> (logits [T, vocab], the residual stream after every layer run [runs, T, W]) in float64."""
    eps = float(cfg["norm"]["eps"])

    def norm(x, name):
        return centred_norm(x, _w(st, name), eps)

    x0 = _w(st, "embed")[torch.as_tensor(tokens, dtype=torch.long)] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    x, after = x0, []
    for i, opens in layer_runs(cfg):
        entry, l = cfg["layers"][i], f"l{i}."
        if opens:
            x = torch.cat((x, x0), dim=1) @ _w(st, "loop.in").T
        x = x + norm(differential_attention(norm(x, l + "norm1"), st, l + "mix.", entry["mixer"], eps), l + "norm1b")
        if entry.get("mlp") is not None:
            x = x + norm(feed_forward(norm(x, l + "norm2"), st, l + "mlp.", entry["mlp"]), l + "norm2b")
        after.append(x)
    return norm(x, "final.norm") @ _w(st, "embed").T, torch.stack(after) if after else torch.zeros(0, len(tokens), x.shape[1], dtype=F64)
