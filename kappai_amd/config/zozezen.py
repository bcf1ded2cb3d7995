"""Configuration of the Zozezen decoder: a list of layers, each a grouped-query attention or a
state-space mixer between two norms and (or not) a mixture of experts between two more.

config.json names the design under ``architecture`` and nests its keys::

    {"architecture": "Zozezen", "vocab": V, "width": D, "norm": {"eps": e},
     "layers": [
       {"type": "attention",
        "mixer": {"heads", "kv_heads", "dim", "vdim", "scale",
                  "rot": {"base", "dims"}, "kv_from": j},
        "mlp": {"kind": "moe", "expert": {"ff": F, "limit": c},
                "router": {"experts": E, "top": k, "identity": n,
                           "groups": {"count": n, "keep": m}},
                "shared": {"ff": F, "limit": c}}},
       {"type": "mamba2",
        "mixer": {"heads", "vdim", "state", "groups", "conv", "norm_groups"},
        "mlp": ...}]}

``kv_from`` (the layer makes keys and values of its own), ``rot`` (nothing turns),
``router.identity`` (none), ``router.groups`` (one group), ``mlp.shared`` (none) and ``mlp`` itself
may be absent or null.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Union

from .base import ConfigError, KeyReader, ModelConfig

ARCHITECTURE = "Zozezen"

MIXER_TYPES = ("attention", "mamba2")


@dataclass
class ZozezenLayer:
    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]]               # None: the layer has no feed-forward


def _sub(r: KeyReader, key: str) -> KeyReader:
    v = r.raw.get(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{r.where}: required key '{key}' must be an object")
    return KeyReader(v, f"{r.where}: {key}")


def _positive(where: str, **values) -> None:
    for name, v in values.items():
        if v <= 0:
            raise ConfigError(f"{where}: {name} must be positive, got {v}")


def _attention(m: KeyReader, where: str) -> Dict[str, Any]:
    out = {"heads": m.int("heads"), "kv_heads": m.int("kv_heads"), "dim": m.int("dim"),
           "vdim": m.int("vdim"), "scale": m.float("scale"), "rot": None,
           "kv_from": m.int("kv_from", None)}
    _positive(where, **{f"mixer.{k}": out[k] for k in ("heads", "kv_heads", "dim", "vdim")})
    if out["heads"] % out["kv_heads"]:
        raise ConfigError(f"{where}: {out['heads']} heads cannot be shared out over "
                          f"{out['kv_heads']} kv heads")
    if m.raw.get("rot") is not None:
        rot = _sub(m, "rot")
        out["rot"] = {"base": rot.float("base"), "dims": rot.int("dims")}
        if out["rot"]["base"] <= 0.0:
            raise ConfigError(f"{where}: mixer.rot.base must be positive")
        if out["rot"]["dims"] % 2 or not 0 <= out["rot"]["dims"] <= out["dim"]:
            raise ConfigError(f"{where}: mixer.rot.dims ({out['rot']['dims']}) must be even and at "
                              f"most mixer.dim ({out['dim']})")
        if out["rot"]["dims"] == 0:
            out["rot"] = None
    return out


def _mamba2(m: KeyReader, where: str) -> Dict[str, Any]:
    out = {k: m.int(k) for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")}
    _positive(where, **{f"mixer.{k}": v for k, v in out.items()})
    if out["heads"] % out["groups"]:
        raise ConfigError(f"{where}: {out['heads']} heads cannot be shared out over "
                          f"{out['groups']} groups")
    if out["heads"] * out["vdim"] % out["norm_groups"]:
        raise ConfigError(f"{where}: {out['heads'] * out['vdim']} values do not form "
                          f"mixer.norm_groups ({out['norm_groups']}) equal parts")
    return out


def _mlp(f: KeyReader, where: str) -> Dict[str, Any]:
    kind = f.raw.get("kind")
    if kind != "moe":
        raise ConfigError(f"{where}: mlp.kind = {kind!r}; known: moe")
    router, expert = _sub(f, "router"), _sub(f, "expert")
    out = {"ff": expert.int("ff"), "limit": expert.float("limit"),
           "experts": router.int("experts"), "top": router.int("top"),
           "identity": router.int("identity", 0) or 0, "groups": 1, "keep_groups": 1,
           "shared_ff": None, "shared_limit": None}
    if router.raw.get("groups") is not None:
        g = _sub(router, "groups")
        out["groups"], out["keep_groups"] = g.int("count"), g.int("keep")
    _positive(where, **{"mlp.expert.ff": out["ff"], "mlp.expert.limit": out["limit"],
                        "mlp.router.experts": out["experts"], "mlp.router.top": out["top"],
                        "mlp.router.groups.count": out["groups"],
                        "mlp.router.groups.keep": out["keep_groups"]})
    if out["identity"] < 0:
        raise ConfigError(f"{where}: mlp.router.identity must not be negative")
    if f.raw.get("shared") is not None:
        shared = _sub(f, "shared")
        out["shared_ff"], out["shared_limit"] = shared.int("ff"), shared.float("limit")
        _positive(where, **{"mlp.shared.ff": out["shared_ff"],
                            "mlp.shared.limit": out["shared_limit"]})
    routed = out["experts"] + out["identity"]
    if routed % out["groups"]:
        raise ConfigError(f"{where}: mlp.router.experts + mlp.router.identity ({routed}) do not form "
                          f"mlp.router.groups.count ({out['groups']}) equal groups")
    if out["keep_groups"] > out["groups"]:
        raise ConfigError(f"{where}: mlp.router.groups.keep ({out['keep_groups']}) exceeds "
                          f"mlp.router.groups.count ({out['groups']})")
    if out["top"] > routed // out["groups"] * out["keep_groups"]:
        raise ConfigError(f"{where}: mlp.router.top ({out['top']}) exceeds the experts that can be "
                          "chosen from")
    return out


def _layer(raw: Any, i: int) -> ZozezenLayer:
    where = f"config.json: layers[{i}]"
    if not isinstance(raw, dict):
        raise ConfigError(f"{where} must be an object")
    r = KeyReader(raw, where)
    kind = raw.get("type")
    if kind not in MIXER_TYPES:
        raise ConfigError(f"{where}: type = {kind!r}; known: {', '.join(MIXER_TYPES)}")
    mixer = (_attention if kind == "attention" else _mamba2)(_sub(r, "mixer"), where)
    mlp = _mlp(_sub(r, "mlp"), where) if raw.get("mlp") is not None else None
    return ZozezenLayer(kind, mixer, mlp)


def _check_shared_keys(layers: List[ZozezenLayer]) -> None:
    for i, layer in enumerate(layers):
        src = layer.mixer.get("kv_from")
        if src is None:
            continue
        where = f"config.json: layers[{i}]: mixer.kv_from"
        if not 0 <= src < i:
            raise ConfigError(f"{where} = {src} names no earlier layer")
        other = layers[src]
        if other.type != "attention" or other.mixer["kv_from"] is not None:
            raise ConfigError(f"{where} = {src}: that layer makes no keys and values of its own")
        for key in ("heads", "kv_heads", "dim", "vdim", "rot"):
            if other.mixer[key] != layer.mixer[key]:
                raise ConfigError(f"{where} = {src}: mixer.{key} differs from that layer's "
                                  f"({layer.mixer[key]} and {other.mixer[key]})")


@dataclass
class ZozezenConfig(ModelConfig):
    vocab_size: int = 0
    width: int = 0
    norm_eps: float = 0.0
    layers: List[ZozezenLayer] = field(default_factory=list)
    max_position_embeddings: int = 0
    eos_token_id: Optional[Union[int, List[int]]] = None
    raw: Dict[str, Any] = field(default_factory=dict, repr=False)

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "ZozezenConfig":
        r = KeyReader(raw)
        cfg = cls(
            architecture=ARCHITECTURE,
            vocab_size=r.int("vocab"),
            width=r.int("width"),
            norm_eps=_sub(r, "norm").float("eps"),
            layers=[_layer(x, i) for i, x in enumerate(r.list("layers"))],
            eos_token_id=r.int_or_ints("eos_token_id", None),
            raw=copy.deepcopy(raw),
        )
        if cfg.vocab_size < 1 or cfg.width < 1:
            raise ConfigError("config.json: vocab and width must be positive")
        if not cfg.layers:
            raise ConfigError("config.json: layers must name at least one layer")
        if cfg.norm_eps <= 0.0:
            raise ConfigError("config.json: norm.eps must be positive")
        _check_shared_keys(cfg.layers)
        return cfg

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.raw)
