"""A plain, slow statement of the Nuzivik decoder in float64 torch on the CPU: one function per
mechanism, whole sequences, no cache and no state.  It shares nothing with the product path; the
tests hold the framework to it.

The stream starts as the embedded row times a constant.  Every sublayer stands between two
pointwise norms, ``x <- x + n_b(f(n_a(x)))``, each a saturating map ``tanh(alpha x) w + b`` that
looks at no other place of the row.  The attention divides every query and key head by its root
mean square, has no values of its own (a kv head's values are its keys before that division), adds
a learned bias by distance to the scaled scores, sees a sliding window and the first tokens of the
sequence, and has a learned sink per head in the softmax's denominator.  The feed-forward is a
mixture of SiLU-gated experts whose router squashes each logit by itself, chooses by the squashed
score plus a correction, within the best groups of experts only, and weighs by the score without
the correction.  The logits are products with the embedding table.

``rounding=torch.bfloat16`` rounds where a bfloat16 run rounds (inputs and outputs of matrix
products), which gives the yardstick for the error that rounding alone costs.
"""
from __future__ import annotations

import math
from typing import Dict, List

import torch

F64 = torch.float64


def _r(x: torch.Tensor, rounding) -> torch.Tensor:
    return x if rounding is None else x.to(rounding).to(F64)


def matmul(x, w, rounding=None):
    """``x [T, in] -> [T, out]`` with ``w [out, in]``."""
    return _r(_r(x, rounding) @ w.to(F64).T, rounding)


def silu(z):
    return z * torch.sigmoid(z)


def saturating_norm(x, t: Dict[str, torch.Tensor], name: str):
    """``tanh(alpha x) w + b`` place by place, with one ``alpha`` for the whole row."""
    return (torch.tanh(t[name + ".alpha"].to(F64) * x) * t[name].to(F64)
            + t[name + ".b"].to(F64))


def unit_rms(x, eps: float):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def bucket_of(n: int, rows: int, far: float) -> int:
    """The bias table's row for distance ``n``: one row a distance in the first half of the table,
    then rows on a logarithmic scale."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half)
                                           * (rows - half)))


def seen(T: int, size, keep: int) -> torch.Tensor:
    """[T, T] bool: whether query i sees key j (``size`` None: every key up to its own)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    if size is not None:
        ok &= (i - j < size) | (j < keep)
    return ok


def sink_softmax(scores, ok, sink):
    """``scores [H, T, T]`` -> weights over the keys seen, with ``exp(sink[h])`` beside them in the
    denominator."""
    scores = scores.masked_fill(~ok, -math.inf)
    m = torch.maximum(scores.max(dim=-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(scores - m)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink[:, None, None] - m))


def attention(h, t: Dict[str, torch.Tensor], p: str, m: dict, eps: float, rounding=None):
    """The attention on ``h [T, width]`` with the tensors ``p + name``."""
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q = matmul(h, t[p + "q"], rounding).reshape(T, H, d)
    v = matmul(h, t[p + "k"], rounding).reshape(T, G, d)
    q, k = _r(unit_rms(q, eps), rounding), _r(unit_rms(v, eps), rounding)
    k, v = (x.repeat_interleave(H // G, dim=1) for x in (k, v))
    scores = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    table = t[p + "rel"].to(F64)
    rows = torch.tensor([bucket_of(n, table.shape[0], m["bias_max"]) for n in range(T)])
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).clamp_min(0)
    scores = scores + table[rows[dist]].permute(2, 0, 1)
    mask = m.get("mask") or {}
    ok = seen(T, mask.get("size"), mask.get("keep_first", 0))
    w = sink_softmax(scores, ok, t[p + "sink"].to(F64))
    ctx = _r(torch.einsum("hij,jhd->ihd", w, v), rounding)
    return matmul(ctx.reshape(T, H * d), t[p + "o"], rounding)


def expert(h, t, p: str, rounding=None):
    act = silu(matmul(h, t[p + "gate"], rounding)) * matmul(h, t[p + "up"], rounding)
    return matmul(act, t[p + "down"], rounding)


def choose(scores, correction, router: dict):
    """One row's chosen experts, best first: by score plus correction, among the groups whose two
    best sums are largest.  Also returns how far the choice stands from another one (the gap at
    the last group kept and at the last expert chosen, whichever is smaller)."""
    E, top = router["experts"], router["top"]
    c = (scores + correction).tolist()
    allowed, gap = list(range(E)), math.inf
    if router.get("groups"):
        n, keep = router["groups"]["count"], router["groups"]["keep"]
        size = E // n
        rank = sorted(((sum(sorted(c[g * size:(g + 1) * size])[-2:]), -g) for g in range(n)),
                      reverse=True)
        if keep < n:
            gap = rank[keep - 1][0] - rank[keep][0]
        kept = {-g for _, g in rank[:keep]}
        allowed = [e for e in range(E) if e // size in kept]
    order = sorted(allowed, key=lambda e: (-c[e], e))
    if top < len(order):
        gap = min(gap, c[order[top - 1]] - c[order[top]])
    return order[:top], gap


def moe_ff(h, t, p: str, mlp: dict, rounding=None, margins: list = None):
    """``margins``: gets, row by row, how far the choice stands from another one."""
    router = mlp["router"]
    s = torch.sigmoid(_r(h, rounding) @ t[p + "router"].to(F64).T)
    corr = t[p + "correction"].to(F64)
    out, gaps = torch.zeros_like(h), []
    for i in range(h.shape[0]):
        order, gap = choose(s[i], corr, router)
        gaps.append(gap)
        for e in order:
            w = s[i, e] * router.get("scale", 1.0)
            out[i] += w * expert(h[i:i + 1], t, f"{p}e{e}.", rounding)[0]
    if margins is not None:
        margins.append(torch.tensor(gaps, dtype=F64))
    return out


def forward(cfg: dict, t: Dict[str, torch.Tensor], tokens: List[int], rounding=None,
            layers_out: list = None, margins: list = None):
    """Float64 logits [len(tokens), vocab].  ``layers_out``: gets the stream after every layer;
    ``margins``: gets every router's margins (``moe_ff``)."""
    eps = cfg["norm"]["eps"]
    x = t["embed"].to(F64)[torch.tensor(tokens, dtype=torch.long)]
    x = x * (cfg.get("embedding") or {}).get("scale", 1.0)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        if layer["type"] != "attention":
            raise ValueError(f"unknown layer type {layer['type']!r}")
        h = attention(saturating_norm(x, t, p + "norm1"), t, p + "mix.", layer["mixer"], eps,
                      rounding)
        x = x + saturating_norm(h, t, p + "norm1b")
        if layer.get("mlp") is not None:
            h = moe_ff(saturating_norm(x, t, p + "norm2"), t, p + "mlp.", layer["mlp"], rounding,
                       margins)
            x = x + saturating_norm(h, t, p + "norm2b")
        if layers_out is not None:
            layers_out.append(x)
    return matmul(saturating_norm(x, t, "final.norm"), t["embed"], rounding)
