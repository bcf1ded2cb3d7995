"""Tiny Zozezen configurations that differ in every size and option, and helpers that write them
as model folders with random weights and hold results to the plain implementation."""
from __future__ import annotations

import copy
import json

import numpy as np
import torch

from kappai_amd.config import config_from_dict
from kappai_amd.models import build_model
from kappai_amd.weights import random_tensors
from kappai_amd.weights.safetensors_io import write_safetensors


def attention(heads, kv_heads, dim, vdim, scale, rot, mlp, kv_from=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot is not None:
        mixer["rot"] = {"base": rot[0], "dims": rot[1]}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def mamba2(heads, vdim, state, groups, conv, norm_groups, mlp):
    return {"type": "mamba2", "mlp": mlp,
            "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                      "conv": conv, "norm_groups": norm_groups}}


def moe(ff, limit, experts, top, identity=None, groups=None, shared=None):
    router = {"experts": experts, "top": top}
    if identity is not None:
        router["identity"] = identity
    if groups is not None:
        router["groups"] = dict(zip(("count", "keep"), groups))
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}
    if shared is not None:
        out["shared"] = dict(zip(("ff", "limit"), shared))
    return out


def config(vocab, width, eps, layers):
    return {"architecture": "Zozezen", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": layers}


# values wider than keys, half of a head rotated; a state of no multiple of eight; keys read from
# an earlier layer with another scale; a layer without feed-forward; groups across the border
# between experts and those that hand their input on
TINY_A = config(211, 72, 1e-5, [
    attention(6, 2, 16, 24, 0.3, (10000.0, 8), moe(24, 1.5, 7, 2, 2, (3, 2), (40, 0.9))),
    mamba2(6, 12, 20, 3, 3, 2, moe(16, 0.8, 6, 3, 2, (4, 2), (24, 2.5))),
    attention(6, 2, 16, 24, 0.2, (10000.0, 8), None, kv_from=0),
    mamba2(4, 20, 10, 1, 5, 8, moe(32, 2.0, 5, 2, 1, None, None)),
])
INIT_A = dict(seed=61, std=0.15)

# no choice to make in any router (every expert, and one that hands its input on, used by every
# token); nothing rotated; a convolution of one tap; one group for everything; a head of its own
# group; two readers of one layer's keys with another layer of keys in between; a layer that is
# its mixer alone
TINY_B = config(97, 48, 1e-6, [
    attention(3, 1, 16, 8, 0.35, None, moe(56, 1.2, 3, 4, 1, None, (24, 1.0))),
    mamba2(2, 24, 16, 1, 1, 1, None),
    attention(4, 4, 8, 16, 0.6, (500.0, 8), moe(8, 0.7, 4, 4, 0, (2, 2), None)),
    attention(3, 1, 16, 8, 0.4, None, None, kv_from=0),
    mamba2(4, 8, 24, 4, 2, 4, moe(24, 3.0, 2, 3, 1, (3, 3), (16, 0.5))),
    attention(3, 1, 16, 8, 0.25, None, None, kv_from=0),
])
INIT_B = dict(seed=66, std=0.14)

# sizes for the matrix cores everywhere, no choices: the state-space chunks, wide experts
TINY_C = config(160, 64, 1e-5, [
    mamba2(8, 16, 32, 2, 4, 4, moe(32, 1.0, 4, 4, 0, None, (64, 2.0))),
    attention(8, 4, 32, 16, 0.2, (1e6, 32), moe(64, 1.5, 3, 4, 1, None, (32, 1.0))),
    mamba2(4, 72, 40, 1, 4, 1, moe(32, 0.9, 2, 4, 2, (4, 4), None)),
    attention(8, 4, 32, 16, 0.25, (1e6, 32), moe(32, 1.1, 4, 4, 0, None, (32, 0.8)), kv_from=1),
])
INIT_C = dict(seed=63, std=0.12)

TINY_D = config(500, 104, 1e-5, [
    mamba2(6, 64, 128, 3, 4, 3, moe(40, 1.3, 12, 4, 3, (5, 3), (48, 1.7))),
    attention(6, 3, 64, 96, 0.15, (10000.0, 64), moe(64, 2.0, 6, 1, 2, (2, 1), (32, 2.2))),
    mamba2(3, 104, 136, 3, 4, 6, None),
    attention(6, 3, 64, 96, 0.1, (10000.0, 64), moe(24, 1.6, 9, 5, 0, (3, 2), (24, 1.0)),
              kv_from=1),
    attention(1, 1, 96, 32, 0.12, (1000.0, 24), moe(16, 1.0, 8, 2, 8, None, (16, 0.6))),
])
INIT_D = dict(seed=64, std=0.1)

# a width, a vocabulary and head sizes that are multiples of nothing: no kernel takes 16 bytes at
# a time here; groups of one expert
TINY_E = config(131, 54, 1e-5, [
    mamba2(3, 10, 7, 1, 4, 5, moe(10, 1.1, 4, 2, 1, (5, 3), (14, 0.9))),
    attention(3, 1, 10, 14, 0.5, (700.0, 6), moe(34, 1.9, 7, 3, 0, None, (10, 1.3))),
    mamba2(5, 9, 33, 5, 2, 3, moe(22, 0.6, 5, 3, 2, None, None)),
    attention(3, 1, 10, 14, 0.3, (700.0, 6), None, kv_from=1),
])
INIT_E = dict(seed=65, std=0.2)

TINY = {"A": (TINY_A, INIT_A), "B": (TINY_B, INIT_B), "C": (TINY_C, INIT_C),
        "D": (TINY_D, INIT_D), "E": (TINY_E, INIT_E)}


def telling(tensors, seed):
    """Random weights whose special tensors matter: decays from nearly one to nearly none, steps of
    unequal size, norm weights around zero that spread, corrections below zero that decide most
    choices clearly, logits wide enough for the limits to bite."""
    g = torch.Generator().manual_seed(seed)
    for name in sorted(tensors):
        t = tensors[name]
        noise = torch.randn(t.shape, generator=g)
        if name.endswith(".A_log"):
            t = -1.0 + 1.5 * noise
        elif name.endswith(".dt_bias"):
            t = -1.0 + noise
        elif name.endswith(".D"):
            t = 1.0 + 0.5 * noise
        elif name.endswith((".norm1", ".norm2", ".norm1b", ".norm2b", "final.norm")):
            t = 0.2 * noise
        elif name.endswith(".conv"):
            t = 0.5 * noise
        elif name.endswith(".conv.b"):
            t = 0.3 * noise
        elif name.endswith(".correction"):
            t = -0.6 + 0.4 * noise
        elif name.endswith((".router", ".sg", ".g")):
            t = 2.0 * t.float()
        elif name.endswith((".gate", ".up")):
            t = 1.5 * t.float()
        tensors[name] = t.to(torch.bfloat16)
    return tensors


def write_tiny(name: str, folder):
    cfg, init = TINY[name]
    conf = config_from_dict(copy.deepcopy(cfg))
    specs = build_model(conf, "float32").tensor_specs()
    tensors = telling(random_tensors(specs, init["seed"], std=init["std"], norm_jitter=0.2),
                      init["seed"])
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg, indent=2))
    write_safetensors(folder / "model.safetensors", tensors)
    return folder


def read_model_dir(model_dir):
    """(config dictionary, {name: tensor}) of a model folder, for the plain implementation."""
    from kappai_amd.weights.safetensors_io import SafetensorsFile
    cfg = json.loads((model_dir / "config.json").read_text())
    f = SafetensorsFile(model_dir / "model.safetensors")
    tensors = {n: f.read(n) for n in f.names()}
    f.close()
    return cfg, tensors


_plain_cache = {}


def plain_run(model_dir, requests, rounding=None):
    """({id: float64 numpy [len, vocab]}, {id: first close call}) from the plain implementation
    (cached per folder).  A close call: a position at which some router's choice stands less than
    ``CLOSE_CALL`` from another one (the request's length when there is none)."""
    from plain import zozezen as plain
    key = (str(model_dir), json.dumps(requests, sort_keys=True), str(rounding))
    if key not in _plain_cache:
        cfg, t = read_model_dir(model_dir)
        logits, first = {}, {}
        for rid, toks in requests.items():
            margins = []
            logits[rid] = plain.forward(cfg, t, toks, rounding=rounding, margins=margins).numpy()
            first[rid] = len(toks)
            for m in margins:
                close = (m < CLOSE_CALL).nonzero().flatten()
                if close.numel():
                    first[rid] = min(first[rid], int(close[0]))
        _plain_cache[key] = logits, first
    return _plain_cache[key]


def row_errors(got, ref):
    """{(id, pos): error of the row}: root mean square of the difference with its mean taken off,
    over the root mean square of all reference logits."""
    scale = float(np.sqrt(np.mean([np.mean(v * v) for v in ref.values()])))
    out = {}
    for (rid, pos), row in got.items():
        assert np.isfinite(row).all(), f"non-finite logits at {rid} position {pos}"
        d = row.astype(np.float64) - ref[rid][pos]
        d = d - d.mean()
        out[(rid, pos)] = float(np.sqrt((d * d).mean())) / scale
    return out


FP32_TOL = 3e-5
CLOSE_CALL = 0.004      # a router's margin below this may go the other way in bfloat16


def assert_matches_plain(got, model_dir, requests, dtype, what="", min_strict=0.1):
    """float32: every row within FP32_TOL.  bfloat16: against what rounding the same values to
    bfloat16 costs the plain implementation itself: no row over six times its root mean square
    row error and at most one row in fifty over three times (but for rows where the plain
    implementation's own rounding error is that large too), for the rows before a request's first
    close call of a router (at least ``min_strict`` of all rows must be such); the rows behind it
    must stay finite and within twice the logits' own size (another expert may have been chosen,
    rightly)."""
    ref, close = plain_run(model_dir, requests)
    errs = row_errors(got, ref)
    worst = max(errs, key=errs.get)
    if dtype == "float32":
        assert errs[worst] < FP32_TOL, (what, worst, errs[worst])
        return
    rounded, _ = plain_run(model_dir, requests, torch.bfloat16)
    own = row_errors({k: rounded[k[0]][k[1]] for k in got}, ref)
    strict = {k: e for k, e in errs.items() if k[1] < close[k[0]]}
    assert len(strict) >= len(errs) * min_strict, (what, "too few rows before a close call",
                                                   len(strict), len(errs))
    yard = float(np.sqrt(np.mean(np.square([own[k] for k in strict])))) if strict else 0.0
    bad = [k for k, e in strict.items() if e > max(6 * yard, 1.5 * own[k])]
    over = [k for k, e in strict.items() if e > max(3 * yard, 1.5 * own[k])]
    assert not bad, (what, bad[:5], [errs[k] for k in bad[:5]], yard)
    assert len(over) <= max(1, len(strict) // 50), (what, len(over), len(strict), yard, over[:5])
    assert max(errs.values()) < 2.0, (what, max(errs, key=errs.get), max(errs.values()))
