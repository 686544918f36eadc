"""Lugitar: a decoder whose layers mix latent attention (own or shared latents, sliding window,
YaRN rotary positions) and lightning attention, with a layer norm before and after every sublayer
and a scaled residual sum:

    x <- x + m * norm1b(mixer(norm1(x)));   x <- x + m * norm2b(mlp(norm2(x)))

The residual stream is fp32 in both model dtypes; the norm after a sublayer, the residual sum and
the norm before the next sublayer are one kernel, so a layer is its matrix products, its mixer's
kernels, two of these and (for the feed-forward) the gate product.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch
import torch.nn as nn
from torch import Tensor

from astrai_amd.extension import _mix
from astrai_amd.model.cache import MixerCache
from astrai_amd.model.mixers import (Fp32Vector, GatedMLP, LatentAttention, LightningAttention, MixerLM, Rotation,
                                     assign_checked)


@dataclass
class LugitarConfig:
    """config.json of a Lugitar model. ``layers`` stays a list of plain dicts: ``type``, ``mixer``
    (its sizes and constants) and ``mlp`` (or None)."""

    vocab: int
    width: int
    layers: List[dict]
    norm: dict
    residual_mult: float
    architecture: str = "Lugitar"

    @staticmethod
    def from_dict(d: dict) -> "LugitarConfig":
        return LugitarConfig(int(d["vocab"]), int(d["width"]), list(d["layers"]), dict(d["norm"]),
                             float(d["residual_mult"]))

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])


def _latent_attention(cfg: LugitarConfig, i: int) -> LatentAttention:
    m = cfg.layers[i]["mixer"]
    source = m.get("kv_from")
    if source is not None:
        if not 0 <= source < i or cfg.layers[source]["type"] != "latent_attention":
            raise ValueError(f"layer {i}: kv_from {source} is not an earlier latent-attention layer")
        src = cfg.layers[source]["mixer"]
        if src.get("kv_from") is not None:
            raise ValueError(f"layer {i}: kv_from {source} has no latents of its own")
        m = {**{key: src[key] for key in ("kv_rank", "rot_dim", "rot")}, **m}
        for key in ("kv_rank", "rot_dim", "rot"):
            if src[key] != m[key]:
                raise ValueError(f"layer {i}: {key} differs from layer {source}, whose latents it reads")
    window = (m.get("mask") or {}).get("size")
    return LatentAttention(cfg.width, int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]),
                           int(m["kv_rank"]), Rotation.from_dict(m["rot"]), float(m["scale"]),
                           None if window is None else int(window), cfg.eps, i, source)


def _lightning(cfg: LugitarConfig, i: int) -> LightningAttention:
    m = cfg.layers[i]["mixer"]
    return LightningAttention(cfg.width, int(m["heads"]), int(m["dim"]), int(m["vdim"]), [float(d) for d in m["decay"]],
                              cfg.eps, i)


_MIXERS = {"latent_attention": _latent_attention, "lightning": _lightning}


class LugitarLayer(nn.Module):
    def __init__(self, cfg: LugitarConfig, i: int):
        super().__init__()
        spec = cfg.layers[i]
        if spec["type"] not in _MIXERS:
            raise ValueError(f"layer {i}: unknown mixer {spec['type']!r}")
        self.norm1, self.norm1b = Fp32Vector(cfg.width), Fp32Vector(cfg.width)
        self.mix = _MIXERS[spec["type"]](cfg, i)
        mlp = spec.get("mlp")
        if mlp is None:
            self.norm2 = self.norm2b = self.mlp = None
            return
        if mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
        self.norm2, self.norm2b = Fp32Vector(cfg.width), Fp32Vector(cfg.width)
        self.mlp = GatedMLP(cfg.width, int(mlp["ff"]))

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        for name in ("norm1", "norm1b", "norm2", "norm2b"):
            norm = getattr(self, name)
            if norm is not None:
                norm.assign(assign_checked("layer", {name: (norm.dim,)}, tensors, prefix)[name])
        self.mix.load(tensors, prefix + "mix.")
        if self.mlp is not None:
            self.mlp.load(tensors, prefix + "mlp.")


class LugitarLM(MixerLM):
    def __init__(self, config: LugitarConfig):
        super().__init__(config, [LugitarLayer(config, i) for i in range(len(config.layers))])
        self.reset()

    @torch.no_grad()
    def forward(self, input_ids: Tensor, kv_cache: Optional[MixerCache] = None, positions: Optional[Tensor] = None,
                logits_at: Optional[Tensor] = None) -> Dict[str, Tensor]:
        """See ``MixerLM.begin``; ``logits_at``: indices into the block; only these tokens' logits are formed."""
        ctx = self.begin(input_ids, kv_cache, positions)
        eps, mult = self.config.eps, self.config.residual_mult
        pre = [layer.norm1.weight for layer in self.layers] + [self.final_norm.weight]
        x, h = _mix.embed_norm(self.embed.weight, input_ids.reshape(-1).contiguous(), pre[0], eps)
        for i, layer in enumerate(self.layers):
            y = layer.mix(h, ctx)
            if layer.mlp is None:
                h = _mix.residual_norm(y, x, layer.norm1b.weight, pre[i + 1], mult, eps)
            else:
                h = _mix.residual_norm(y, x, layer.norm1b.weight, layer.norm2.weight, mult, eps)
                h = _mix.residual_norm(layer.mlp(h), x, layer.norm2b.weight, pre[i + 1], mult, eps)
        return self.finish(h, x, ctx, logits_at)
