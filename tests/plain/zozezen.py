"""A plain, slow statement of the Zozezen decoder in float64 torch on the CPU: one function per
mechanism, whole sequences, no cache and no state handed on.  It shares nothing with the product
path; the tests hold the framework to it.

Every sublayer stands between two RMS norms whose weights are stored around zero, ``x <- x +
n_b(f(n_a(x)))``.  The mixer is a grouped-query attention (per-head norms, a rotation over the
first places, a one in the softmax's denominator, one sigmoid gate a head; it may read the keys
and values of an earlier layer instead of making its own) or a state-space layer with one decay a
head and token (S <- a S + (dt B) x^T).  The feed-forward is a mixture of experts with clamped
gates: the router takes a softmax over all experts, the last of which may hand their input on
unchanged; it chooses by the score plus a correction within the best groups and weighs by the
score; a shared expert runs for every row behind a gate of its own.

``rounding=torch.bfloat16`` rounds where a bfloat16 run rounds (inputs and outputs of matrix
products and of the short convolution), which gives the yardstick for the error that rounding
alone costs.
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


def unit_rms(x, eps: float):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def one_plus_norm(x, w, eps: float):
    return unit_rms(x, eps) * (1.0 + w.to(F64))


def rotate(x, base: float, dims: int):
    """``x [T, heads, d]``, row t at position t: the pair of places (i, i + dims / 2) turns by
    ``t * base^(-2 i / dims)``; places from ``dims`` on stay."""
    half = dims // 2
    f = base ** (-2.0 * torch.arange(half, dtype=F64) / dims)
    a = torch.arange(x.shape[0], dtype=F64)[:, None, None] * f
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a),
                      x[..., dims:]], dim=-1)


def plus_one_softmax(scores):
    """Weights over the last axis with a one beside the exponentials in the denominator; scores of
    minus infinity are not seen."""
    m = scores.max(dim=-1, keepdim=True).values.clamp_min(0.0)
    e = torch.exp(scores - m)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(-m))


def heads_of(h, t, p: str, which: str, n: int, m: dict, eps: float, rounding=None):
    """The ``n`` query or key heads (``which`` "q" or "k"): projected, normed, rotated."""
    x = matmul(h, t[p + which], rounding).reshape(h.shape[0], n, m["dim"])
    x = unit_rms(x, eps) * t[p + which + ".norm"].to(F64)
    rot = m.get("rot")
    return _r(rotate(x, rot["base"], rot["dims"]) if rot else x, rounding)


def attention(h, t: Dict[str, torch.Tensor], p: str, m: dict, eps: float, rounding=None, kv=None,
              made: list = None):
    """The attention on ``h [T, width]`` with the tensors ``p + name``.  ``kv``: keys and values of
    another layer, used as they are; ``made``: gets this layer's (keys, values)."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = heads_of(h, t, p, "q", H, m, eps, rounding)
    if kv is None:
        kv = (heads_of(h, t, p, "k", G, m, eps, rounding),
              matmul(h, t[p + "v"], rounding).reshape(T, G, m["vdim"]))
    if made is not None:
        made.append(kv)
    k, v = (x.repeat_interleave(H // G, dim=1) for x in kv)
    scores = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    ahead = torch.arange(T)[None, :] > torch.arange(T)[:, None]
    w = plus_one_softmax(scores.masked_fill(ahead, -math.inf))
    ctx = _r(torch.einsum("hij,jhd->ihd", w, v), rounding)
    ctx = _r(ctx * torch.sigmoid(matmul(h, t[p + "g"], rounding))[..., None], rounding)
    return matmul(ctx.reshape(T, H * m["vdim"]), t[p + "o"], rounding)


def short_conv(x, taps, bias):
    """``out[t] = silu(bias + sum_j taps[:, j] x[t - n + 1 + j])``, zeros before the start."""
    n = taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=F64), x])
    out = sum(padded[j:j + x.shape[0]] * taps[:, j].to(F64) for j in range(n))
    return silu(out + bias.to(F64))


def state_space(x, B, C, dt, rate, D):
    """Token by token: ``S <- exp(-rate dt) S + dt B x^T``, ``y = S^T C + D x``.  ``x [T, H, v]``,
    ``B`` and ``C [T, G, N]``, ``dt [T, H]``, ``rate`` and ``D [H]``."""
    T, H, v = x.shape
    B, C = (z.repeat_interleave(H // z.shape[1], dim=1) for z in (B, C))
    S = torch.zeros(H, B.shape[2], v, dtype=F64)
    y = torch.zeros_like(x)
    for i in range(T):
        S = torch.exp(-rate * dt[i])[:, None, None] * S + torch.einsum(
            "hn,hv->hnv", dt[i][:, None] * B[i], x[i])
        y[i] = torch.einsum("hnv,hn->hv", S, C[i]) + D[:, None] * x[i]
    return y


def gated_group_norm(y, z, w, parts: int, eps: float):
    """``y silu(z)`` normed in ``parts`` equal parts of the row, times ``w``."""
    g = (y * silu(z)).reshape(y.shape[0], parts, -1)
    return unit_rms(g, eps).reshape(y.shape) * w.to(F64)


def mamba2(h, t: Dict[str, torch.Tensor], p: str, m: dict, eps: float, rounding=None):
    """The state-space mixer on ``h [T, width]``."""
    T, H, v, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    z, xbc, dt = matmul(h, t[p + "in"], rounding).split([H * v, H * v + 2 * G * N, H], dim=1)
    x, B, C = _r(short_conv(xbc, t[p + "conv"], t[p + "conv.b"]), rounding).split(
        [H * v, G * N, G * N], dim=1)
    dt = torch.nn.functional.softplus(dt + t[p + "dt_bias"].to(F64))
    y = state_space(x.reshape(T, H, v), B.reshape(T, G, N), C.reshape(T, G, N), dt,
                    torch.exp(t[p + "A_log"].to(F64)), t[p + "D"].to(F64))
    y = gated_group_norm(y.reshape(T, H * v), z, t[p + "norm"], m["norm_groups"], eps)
    return matmul(y, t[p + "o"], rounding)


def expert(h, t, p: str, limit: float, rounding=None):
    g = matmul(h, t[p + "gate"], rounding).clamp(max=limit)
    u = matmul(h, t[p + "up"], rounding).clamp(-limit, limit)
    return matmul(g * torch.sigmoid(1.702 * g) * (u + 1.0), t[p + "down"], rounding)


def choose(scores, correction, router: dict):
    """One row's chosen experts, best first: by score plus correction, among the groups whose best
    such value is largest.  Also returns how far the choice stands from another one (the gap at
    the last group kept and at the last expert chosen, whichever is smaller)."""
    c = (scores + correction).tolist()
    allowed, gap = list(range(len(c))), math.inf
    if router.get("groups"):
        n, keep = router["groups"]["count"], router["groups"]["keep"]
        size = len(c) // n
        rank = sorted(((max(c[g * size:(g + 1) * size]), -g) for g in range(n)), reverse=True)
        if keep < n:
            gap = rank[keep - 1][0] - rank[keep][0]
        kept = {-g for _, g in rank[:keep]}
        allowed = [e for e in allowed if e // size in kept]
    order = sorted(allowed, key=lambda e: (-c[e], e))[:router["top"] + 1]
    if router["top"] < len(order):
        gap = min(gap, c[order[-2]] - c[order[-1]])
    return order[:router["top"]], gap


def moe_ff(h, t, p: str, mlp: dict, rounding=None, margins: list = None):
    """``margins``: gets, row by row, how far the choice stands from another one."""
    router = mlp["router"]
    s = torch.softmax(_r(h, rounding) @ t[p + "router"].to(F64).T, dim=-1)
    corr = t[p + "correction"].to(F64)
    picks = [choose(s[i], corr, router) for i in range(h.shape[0])]
    if margins is not None:
        margins.append(torch.tensor([gap for _, gap in picks], dtype=F64))
    out = torch.zeros_like(h)
    for e in range(s.shape[1]):
        rows = torch.tensor([i for i, (order, _) in enumerate(picks) if e in order],
                            dtype=torch.long)
        if not len(rows):
            continue
        x = h[rows]
        if e < router["experts"]:
            y = expert(x, t, f"{p}e{e}.", mlp["expert"]["limit"], rounding)
        else:
            y = _r(x, rounding)
        out[rows] += s[rows, e:e + 1] * y
    if mlp.get("shared"):
        gate = torch.sigmoid(_r(h, rounding) @ t[p + "shared.sg"].to(F64).T)
        out = out + gate * expert(h, t, p + "shared.", mlp["shared"]["limit"], rounding)
    return out


def forward(cfg: dict, t: Dict[str, torch.Tensor], tokens: List[int], rounding=None,
            layers_out: list = None, margins: list = None):
    """Float64 logits [len(tokens), vocab].  ``layers_out``: gets the stream after every layer;
    ``margins``: gets every router's margins (``moe_ff``)."""
    eps = cfg["norm"]["eps"]
    x = t["embed"].to(F64)[torch.tensor(tokens, dtype=torch.long)]
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = one_plus_norm(x, t[p + "norm1"], eps)
        if layer["type"] == "attention":
            made = []
            src = m.get("kv_from")
            h = attention(h, t, p + "mix.", m, eps, rounding,
                          kv=None if src is None else kept[src], made=made)
            kept[i] = made[0]
        elif layer["type"] == "mamba2":
            h = mamba2(h, t, p + "mix.", m, eps, rounding)
        else:
            raise ValueError(f"unknown layer type {layer['type']!r}")
        x = x + one_plus_norm(h, t[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            h = moe_ff(one_plus_norm(x, t[p + "norm2"], eps), t, p + "mlp.", layer["mlp"],
                       rounding, margins)
            x = x + one_plus_norm(h, t[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x)
    return matmul(one_plus_norm(x, t["final.norm"], eps), t["head"], rounding)
