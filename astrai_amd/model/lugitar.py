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
from astrai_amd.model.decoder import Embedding, Linear
from astrai_amd.model.mixers import (Fp32Vector, GatedMLP, LatentAttention, LightningAttention, Rotation,
                                     StepContext, assign_checked)


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


class LugitarLM(nn.Module):
    """Same calling convention as ``AutoRegressiveLM``: ``model(ids, cache, positions)["logits"]``."""

    def __init__(self, config: LugitarConfig):
        super().__init__()
        self.config = config
        self.embed = Embedding(config.vocab, config.width)
        self.layers = nn.ModuleList([LugitarLayer(config, i) for i in range(len(config.layers))])
        self.final_norm = Fp32Vector(config.width)
        self.head = Linear(config.width, config.vocab)
        self.apply(lambda m: m.reset_parameters() if hasattr(m, "reset_parameters") else None)
        self._ready = False

    @property
    def dtype(self) -> torch.dtype:
        return self.embed.weight.dtype

    @torch.no_grad()
    def load_tensors(self, tensors: Dict[str, Tensor]) -> "LugitarLM":
        """Take every weight from ``tensors`` (stored names); a missing, unknown or misshapen one raises."""
        left = dict(tensors)
        cfg = self.config
        top = assign_checked("model", {"embed": (cfg.vocab, cfg.width), "final.norm": (cfg.width,),
                                       "head": (cfg.vocab, cfg.width)}, left, "")
        self.embed.weight.copy_(top["embed"])
        self.head.weight.copy_(top["head"])
        self.final_norm.assign(top["final.norm"])
        for i, layer in enumerate(self.layers):
            layer.load(left, f"l{i}.")
        if left:
            raise ValueError(f"checkpoint does not match the model: unexpected {sorted(left)[:8]}")
        self._ready = False
        return self

    def _apply(self, fn, recurse=True):
        self._ready = False
        return super()._apply(fn, recurse)

    def finalize(self) -> "LugitarLM":
        """Derive the weight layouts the kernels read; called by the first forward after loading or
        moving the model."""
        for layer in self.layers:
            layer.mix.finalize()
        self._ready = True
        return self

    def new_cache(self, batch: int, max_len: int) -> MixerCache:
        cache = MixerCache(batch, max_len, self.embed.weight.device, self.dtype)
        for layer in self.layers:
            layer.mix.add_to_cache(cache)
        return cache

    @torch.no_grad()
    def forward(self, input_ids: Tensor, kv_cache: Optional[MixerCache] = None, positions: Optional[Tensor] = None,
                logits_at: Optional[Tensor] = None) -> Dict[str, Tensor]:
        """``input_ids [batch, seq]``: the tokens after those the cache holds, ``kv_cache.tokens`` of them
        (``positions``, if given, is those tokens' positions on the device; the caller advances the
        cache). Without a cache: a sequence of its own. ``logits_at``: indices into the block; only
        these tokens' logits are formed."""
        if input_ids.ndim != 2:
            raise ValueError("input_ids must be [batch, seq_len]")
        b, s = input_ids.shape
        if not self._ready:
            self.finalize()
        if kv_cache is None:
            kv_cache = self.new_cache(b, s)
        if kv_cache.batch != b:
            raise ValueError(f"{b} sequences with a cache for {kv_cache.batch}")
        if positions is None:
            positions = kv_cache.next_positions(s)
        elif kv_cache.tokens + s > kv_cache.max_len:
            raise ValueError(f"{s} tokens after {kv_cache.tokens} do not fit a cache of {kv_cache.max_len}")
        ctx = StepContext(kv_cache, positions, kv_cache.tokens, b, s)
        cfg, eps, mult = self.config, self.config.eps, self.config.residual_mult
        n = len(self.layers)
        pre = [layer.norm1.weight for layer in self.layers] + [self.final_norm.weight]
        x, h = _mix.embed_norm(self.embed.weight, input_ids.reshape(-1).contiguous(), pre[0], eps)
        for i, layer in enumerate(self.layers):
            y = layer.mix(h, ctx)
            if layer.mlp is None:
                h = _mix.residual_norm(y, x, layer.norm1b.weight, pre[i + 1], mult, eps)
            else:
                h = _mix.residual_norm(y, x, layer.norm1b.weight, layer.norm2.weight, mult, eps)
                h = _mix.residual_norm(layer.mlp(h), x, layer.norm2b.weight, pre[i + 1], mult, eps)
        hidden = h.reshape(b, s, cfg.width)
        if logits_at is not None:
            hidden = hidden.index_select(1, logits_at)
        return {"logits": self.head(hidden), "hidden_states": hidden, "residual": x.reshape(b, s, cfg.width)}
