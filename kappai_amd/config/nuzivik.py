"""Configuration of the Nuzivik decoder: a list of layers, each an attention between two norms and
(or not) a mixture of experts between two more; the output head is the embedding table.

config.json names the design under ``architecture`` and nests its keys::

    {"architecture": "Nuzivik", "vocab": V, "width": D, "norm": {"eps": e},
     "embedding": {"scale": s},
     "layers": [
       {"type": "attention",
        "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "bias_max",
                  "mask": {"size": window, "keep_first": n}},
        "mlp": {"kind": "moe", "expert": {"ff": F},
                "router": {"experts": E, "top": k, "scale": c,
                           "groups": {"count": n, "keep": m}}}}]}

``mask`` (every earlier key is seen), ``mask.keep_first`` (none), ``router.groups`` (one group),
``router.scale`` (1), ``embedding`` (1) and ``mlp`` itself may be absent or null.  The rows of a
layer's distance-bias table are the tensor's (``adopt_tensor_shapes``); a file for the
random-weights mode states them as ``mixer.buckets``.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Union

from .base import ConfigError, KeyReader, ModelConfig

ARCHITECTURE = "Nuzivik"

MIXER_TYPES = ("attention",)


@dataclass
class NuzivikLayer:
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
        if v < 1:
            raise ConfigError(f"{where}: {name} must be positive, got {v}")


def _attention(m: KeyReader, where: str) -> Dict[str, Any]:
    out = {"heads": m.int("heads"), "kv_heads": m.int("kv_heads"), "dim": m.int("dim"),
           "scale": m.float("scale"), "bias_max": m.float("bias_max"),
           "buckets": m.int("buckets", None), "window": None, "keep_first": 0}
    out["vdim"] = m.int("vdim", None) or out["dim"]
    _positive(where, **{"mixer.heads": out["heads"], "mixer.kv_heads": out["kv_heads"],
                        "mixer.dim": out["dim"]})
    if out["heads"] % out["kv_heads"]:
        raise ConfigError(f"{where}: {out['heads']} heads cannot be shared out over "
                          f"{out['kv_heads']} kv heads")
    if out["vdim"] != out["dim"]:
        raise ConfigError(f"{where}: mixer.vdim ({out['vdim']}) must equal mixer.dim "
                          f"({out['dim']}): the values are the keys")
    if out["bias_max"] <= 1.0:
        raise ConfigError(f"{where}: mixer.bias_max must be larger than 1")
    if m.raw.get("mask") is not None:
        mask = _sub(m, "mask")
        out["window"], out["keep_first"] = mask.int("size"), mask.int("keep_first", 0) or 0
        _positive(where, **{"mixer.mask.size": out["window"]})
        if out["keep_first"] < 0:
            raise ConfigError(f"{where}: mixer.mask.keep_first must not be negative")
    return out


def _mlp(f: KeyReader, where: str) -> Dict[str, Any]:
    kind = f.raw.get("kind")
    if kind != "moe":
        raise ConfigError(f"{where}: mlp.kind = {kind!r}; known: moe")
    router = _sub(f, "router")
    scale = router.float("scale", None)
    out = {"ff": _sub(f, "expert").int("ff"), "experts": router.int("experts"),
           "top": router.int("top"), "scale": 1.0 if scale is None else scale, "groups": 1,
           "keep_groups": 1}
    if router.raw.get("groups") is not None:
        g = _sub(router, "groups")
        out["groups"], out["keep_groups"] = g.int("count"), g.int("keep")
    _positive(where, **{"mlp.expert.ff": out["ff"], "mlp.router.experts": out["experts"],
                        "mlp.router.top": out["top"], "mlp.router.groups.count": out["groups"],
                        "mlp.router.groups.keep": out["keep_groups"]})
    if out["experts"] % out["groups"]:
        raise ConfigError(f"{where}: mlp.router.experts ({out['experts']}) do not form "
                          f"mlp.router.groups.count ({out['groups']}) equal groups")
    if out["keep_groups"] > out["groups"]:
        raise ConfigError(f"{where}: mlp.router.groups.keep ({out['keep_groups']}) exceeds "
                          f"mlp.router.groups.count ({out['groups']})")
    if out["top"] > out["experts"] // out["groups"] * out["keep_groups"]:
        raise ConfigError(f"{where}: mlp.router.top ({out['top']}) exceeds the experts that can be "
                          "chosen from")
    return out


def _layer(raw: Any, i: int) -> NuzivikLayer:
    where = f"config.json: layers[{i}]"
    if not isinstance(raw, dict):
        raise ConfigError(f"{where} must be an object")
    r = KeyReader(raw, where)
    kind = raw.get("type")
    if kind not in MIXER_TYPES:
        raise ConfigError(f"{where}: type = {kind!r}; known: {', '.join(MIXER_TYPES)}")
    mixer = _attention(_sub(r, "mixer"), where)
    mlp = _mlp(_sub(r, "mlp"), where) if raw.get("mlp") is not None else None
    return NuzivikLayer(kind, mixer, mlp)


@dataclass
class NuzivikConfig(ModelConfig):
    vocab_size: int = 0
    width: int = 0
    norm_eps: float = 0.0
    embedding_scale: float = 1.0
    layers: List[NuzivikLayer] = field(default_factory=list)
    max_position_embeddings: int = 0
    eos_token_id: Optional[Union[int, List[int]]] = None
    raw: Dict[str, Any] = field(default_factory=dict, repr=False)

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "NuzivikConfig":
        r = KeyReader(raw)
        scale = None
        if raw.get("embedding") is not None:
            scale = _sub(r, "embedding").float("scale", None)
        cfg = cls(
            architecture=ARCHITECTURE,
            vocab_size=r.int("vocab"),
            width=r.int("width"),
            norm_eps=_sub(r, "norm").float("eps"),
            embedding_scale=1.0 if scale is None else scale,
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
        return cfg

    def adopt_tensor_shapes(self, shapes: Dict[str, tuple]) -> None:
        """The rows of a layer's distance-bias table where the file leaves them to the tensor.  A
        number that config.json states is kept."""
        for i, layer in enumerate(self.layers):
            if layer.mixer.get("buckets") is None:
                name = f"l{i}.mix.rel"
                if name not in shapes or not shapes[name]:
                    raise ConfigError(f"config.json: layers[{i}] mixer.buckets is neither stated "
                                      f"nor given by a tensor '{name}'")
                layer.mixer["buckets"] = int(shapes[name][0])

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.raw)
