"""The Nuzivik decoder put together from parts.

Every layer is ``block.sandwich_norm`` with saturating norms (``norm.tanh_norm``) before and behind
each sublayer: ``mixer.scored_attention`` (q and k heads divided by their root mean square, values
that are the keys as projected, a learned bias by distance, a sliding window beside the first
positions of the sequence, a learned sink a head, no rotation) and a mixture of SiLU-gated experts
whose router squashes its logits, chooses with a correction within the best groups and weighs
without it; or no feed-forward.  The embedded rows are scaled; the output head is the table without
the scale.  Tensor names: ``embed``, ``final.norm`` and per layer ``l<i>.norm1|norm1b|norm2|norm2b``
(each with ``.alpha`` and ``.b``), ``l<i>.mix.*``, ``l<i>.mlp.*``; no name ends in ``.weight``.
"""
from __future__ import annotations

import torch

from ..config.base import register_architecture
from ..config.nuzivik import ARCHITECTURE, NuzivikConfig
from ..parts.base import make_part
from ..parts.embedding import OutputHead, TokenEmbedding
from .base import Model


def _mixer(m: dict, p: str, width: int, eps: float, dtype):
    if m["buckets"] is None:
        raise ValueError("config.json does not state mixer.buckets, and no tensor shapes were "
                         "read that could give it")
    return make_part(
        "mixer", "scored_attention", prefix=p, width=width, num_heads=m["heads"],
        num_kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=m["scale"], dtype=dtype,
        norm_eps=eps, head_qk_norm=True, head_norm_weight=False, values_from_keys=True,
        bias_buckets=m["buckets"], bias_far=m["bias_max"], sink=True, window=m["window"],
        keep_first=m["keep_first"], weight_suffix="")


def _feed_forward(mlp: dict, p: str, width: int, dtype):
    return make_part("feed_forward", "moe", prefix=p, width=width, hidden=mlp["ff"],
                     experts=mlp["experts"], top=mlp["top"], dtype=dtype, weight_suffix="",
                     activation="silu_gated", scoring="sigmoid", correction=True,
                     groups=mlp["groups"], keep_groups=mlp["keep_groups"],
                     weight_scale=mlp["scale"])


def build_nuzivik(config: NuzivikConfig, dtype: torch.dtype) -> Model:
    width, eps = config.width, config.norm_eps

    def norm(name):
        return make_part("norm", "tanh_norm", name=name, width=width, dtype=dtype)

    layers, unused = [], []
    for i, layer in enumerate(config.layers):
        p = f"l{i}."
        feed_forward = ffn_norm = ffn_out_norm = None
        if layer.mlp is not None:
            feed_forward = _feed_forward(layer.mlp, p + "mlp.", width, dtype)
            ffn_norm, ffn_out_norm = norm(p + "norm2"), norm(p + "norm2b")
        else:
            unused += [s.name for n in ("norm2", "norm2b") for s in norm(p + n).tensor_specs()]
        layers.append(make_part(
            "block", "sandwich_norm", mixer_norm=norm(p + "norm1"),
            mixer=_mixer(layer.mixer, p + "mix.", width, eps, dtype),
            mixer_out_norm=norm(p + "norm1b"), ffn_norm=ffn_norm, feed_forward=feed_forward,
            ffn_out_norm=ffn_out_norm))
    embedding = TokenEmbedding("embed", config.vocab_size, width, suffix="",
                               scale=config.embedding_scale)
    head = OutputHead("embed", config.vocab_size, width, tied_to=embedding, suffix="")
    model = Model(config, dtype, embedding, layers, norm("final.norm"), head)
    model.unused_tensor_names = unused
    return model


register_architecture(ARCHITECTURE, NuzivikConfig, build_nuzivik)
