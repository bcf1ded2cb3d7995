"""The Zozezen decoder put together from parts.

Every layer is ``block.sandwich_norm`` with RMS norms (weights stored around zero) before and
behind each sublayer, around one of two mixers: ``mixer.scored_attention`` (every q and k head
normed by itself, a rotation over the first places, a sink of score zero, one sigmoid gate a head;
a layer may read the keys and values of an earlier one) or ``mixer.state_space_dual``; and a
mixture of experts with clamped gates whose router takes a softmax over all experts, some of which
hand their input on, with a gated shared expert beside them; or no feed-forward.  Tensor names:
``embed``, ``final.norm``, ``head`` and per layer ``l<i>.norm1|norm1b|norm2|norm2b``, ``l<i>.mix.*``,
``l<i>.mlp.*``; no name ends in ``.weight``.
"""
from __future__ import annotations

import torch

from ..config.base import register_architecture
from ..config.zozezen import ARCHITECTURE, ZozezenConfig
from ..kernels import ops
from ..parts.base import make_part
from ..parts.embedding import OutputHead, TokenEmbedding
from .base import LayerCall, Model


def _mixer(kind: str, m: dict, p: str, width: int, eps: float, dtype):
    if kind == "attention":
        position = None
        if m["rot"]:
            position = make_part("position_encoding", "rotary", head_dim=m["dim"],
                                 theta=m["rot"]["base"], rot_dim=m["rot"]["dims"], pairing="half")
        return make_part(
            "mixer", "scored_attention", prefix=p, width=width, num_heads=m["heads"],
            num_kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=m["scale"],
            dtype=dtype, norm_eps=eps, head_qk_norm=True, sink_value=0.0, head_gate=True,
            position=position, own_keys=m["kv_from"] is None, weight_suffix="")
    return make_part(
        "mixer", "state_space_dual", prefix=p, width=width, num_heads=m["heads"],
        vdim=m["vdim"], state=m["state"], groups=m["groups"], taps=m["conv"],
        norm_groups=m["norm_groups"], norm_eps=eps, dtype=dtype, weight_suffix="",
        bias_suffix=".b")


def _feed_forward(mlp: dict, p: str, width: int, dtype):
    shared = mlp["shared_ff"] is not None
    return make_part("feed_forward", "moe", prefix=p, width=width, hidden=mlp["ff"],
                     experts=mlp["experts"], top=mlp["top"], dtype=dtype, weight_suffix="",
                     activation="clamped", clamp=ops.ClampedGate(mlp["limit"]),
                     scoring="softmax_all", correction=True, groups=mlp["groups"],
                     keep_groups=mlp["keep_groups"], group_best=1, identity=mlp["identity"],
                     shared_hidden=mlp["shared_ff"], shared_gate=shared,
                     shared_clamp=ops.ClampedGate(mlp["shared_limit"]) if shared else None)


def build_zozezen(config: ZozezenConfig, dtype: torch.dtype) -> Model:
    width, eps = config.width, config.norm_eps

    def norm(name):
        return make_part("norm", "rmsnorm", name=name, width=width, eps=eps, dtype=dtype,
                         suffix="", weight_offset=1.0)

    layers, unused, schedule = [], [], []
    for i, layer in enumerate(config.layers):
        p = f"l{i}."
        feed_forward = ffn_norm = ffn_out_norm = None
        if layer.mlp is not None:
            feed_forward = _feed_forward(layer.mlp, p + "mlp.", width, dtype)
            ffn_norm, ffn_out_norm = norm(p + "norm2"), norm(p + "norm2b")
        else:
            unused += [p + "norm2", p + "norm2b"]
        layers.append(make_part(
            "block", "sandwich_norm", mixer_norm=norm(p + "norm1"),
            mixer=_mixer(layer.type, layer.mixer, p + "mix.", width, eps, dtype),
            mixer_out_norm=norm(p + "norm1b"), ffn_norm=ffn_norm, feed_forward=feed_forward,
            ffn_out_norm=ffn_out_norm))
        schedule.append(LayerCall(i, reads_cache_of=layer.mixer.get("kv_from")))
    embedding = TokenEmbedding("embed", config.vocab_size, width, suffix="")
    head = OutputHead("head", config.vocab_size, width, tied_to=None, suffix="")
    model = Model(config, dtype, embedding, layers, norm("final.norm"), head, schedule=schedule)
    model.unused_tensor_names = unused
    return model


register_architecture(ARCHITECTURE, ZozezenConfig, build_zozezen)
