"""Sarulix: a decoder whose layers mix grouped-query attention with a sink, a real-gated linear recurrent
unit and a gated delta rule with a decay per key channel, pre-norm, some layers without a feed-forward:

    x <- x + mixer(norm1(x));   x <- x + mlp(norm2(x))

A run of layers may be passed through several times with the same weights, each pass with its own caches.
A pass begins with x <- W_in [x; x0] + step_t, x0 the embedding output. W_in is kept as its two halves, so that
W_b x0 is formed once per forward, and together with W_a x0 where a forward begins with a pass.

The residual stream is fp32 in both model dtypes; a sublayer's residual sum (or a pass's new stream) and the
norm before the next sublayer are one kernel.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn
from torch import Tensor

from astrai_amd.extension import _mix
from astrai_amd.model.cache import MixerCache
from astrai_amd.model.mixers import (ChannelDelta, Fp32Vector, GatedMLP, GatedRecurrence, GroupedAttention, MixerLM,
                                     PackedLinear, Rotation, Rows, assign_checked, columns_of, linear_f32)

NO_LOOP = (0, 0, 0)


@dataclass
class SarulixConfig:
    """config.json of a Sarulix model. ``layers`` stays a list of plain dicts: ``type``, ``mixer`` (its sizes and
    constants) and ``mlp`` (or None); ``loop`` is (start, stop, times): layers ``start .. stop - 1`` run ``times``
    times in a row. ``ranks[i]`` are the inner sizes of a delta-rule layer's decay and gate projections, which only
    the stored weights tell (``with_tensors``)."""

    vocab: int
    width: int
    layers: List[dict]
    norm: dict
    embedding_scale: float
    logit_scale: float
    loop: Tuple[int, int, int] = NO_LOOP
    ranks: Optional[Dict[int, Tuple[int, int]]] = None
    architecture: str = "Sarulix"

    @staticmethod
    def from_dict(d: dict) -> "SarulixConfig":
        loop = d.get("loop")
        loop = NO_LOOP if loop is None else (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
        if loop != NO_LOOP and not (0 <= loop[0] < loop[1] <= len(d["layers"]) and loop[2] >= 1):
            raise ValueError(f"loop {loop} over {len(d['layers'])} layers")
        return SarulixConfig(int(d["vocab"]), int(d["width"]), list(d["layers"]), dict(d["norm"]),
                             float(d["embedding"]["scale"]), float(d["logit_scale"]), loop)

    def with_tensors(self, tensors: Dict[str, Tensor]) -> "SarulixConfig":
        """Fill in the sizes that config.json leaves to the tensors' shapes."""
        self.ranks = {}
        for i, layer in enumerate(self.layers):
            if layer["type"] == "channel_delta":
                names = [f"l{i}.mix.a1", f"l{i}.mix.g1"]
                for name in names:
                    if name not in tensors:
                        raise ValueError(f"delta rule: tensor {name} is missing")
                self.ranks[i] = tuple(tensors[name].size(0) for name in names)
        return self

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])

    def order(self) -> List[Tuple[int, int, bool]]:
        """The layers in the order they run: (layer, pass, whether it begins a pass)."""
        start, stop, times = self.loop
        once = [(i, 0, False) for i in range(len(self.layers))]
        passes = [(i, t, i == start) for t in range(times) for i in range(start, stop)]
        return once[:start] + passes + once[stop:]


def _attention(cfg: SarulixConfig, i: int) -> GroupedAttention:
    m = cfg.layers[i]["mixer"]
    return GroupedAttention(cfg.width, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                            Rotation.from_dict(m["rot"]), float(m["scale"]), float(m["softcap"]), cfg.eps, i)


def _rglru(cfg: SarulixConfig, i: int) -> GatedRecurrence:
    m = cfg.layers[i]["mixer"]
    return GatedRecurrence(cfg.width, int(m["width"]), int(m["blocks"]), int(m["conv"]), i)


def _channel_delta(cfg: SarulixConfig, i: int) -> ChannelDelta:
    m = cfg.layers[i]["mixer"]
    # (random weights without a checkpoint: both ranks the value size)
    rank, gate_rank = (cfg.ranks or {}).get(i, (int(m["vdim"]), int(m["vdim"])))
    return ChannelDelta(cfg.width, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), int(m["conv"]),
                        rank, gate_rank, cfg.eps, i)


_MIXERS = {"attention": _attention, "rglru": _rglru, "channel_delta": _channel_delta}


class OnePlusVector(Fp32Vector):
    """A norm's weight that is stored around zero."""

    def assign(self, t: Tensor) -> None:
        super().assign(1.0 + t.float())


class SarulixLayer(nn.Module):
    def __init__(self, cfg: SarulixConfig, i: int):
        super().__init__()
        spec = cfg.layers[i]
        if spec["type"] not in _MIXERS:
            raise ValueError(f"layer {i}: unknown mixer {spec['type']!r}")
        self.norm1 = OnePlusVector(cfg.width)
        self.mix = _MIXERS[spec["type"]](cfg, i)
        mlp = spec.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
        self.norm2 = None if mlp is None else OnePlusVector(cfg.width)
        self.mlp = None if mlp is None else GatedMLP(cfg.width, int(mlp["ff"]), "gelu_tanh")

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        for name in ("norm1", "norm2"):
            norm = getattr(self, name)
            if norm is not None:
                norm.assign(assign_checked("layer", {name: (norm.dim,)}, tensors, prefix)[name])
        self.mix.load(tensors, prefix + "mix.")
        if self.mlp is not None:
            self.mlp.load(tensors, prefix + "mlp.")


class SarulixLM(MixerLM):
    def __init__(self, config: SarulixConfig):
        super().__init__(config, [SarulixLayer(config, i) for i in range(len(config.layers))])
        w = config.width
        self.final_norm = OnePlusVector(w)
        self.final_norm.weight.mul_(config.logit_scale)
        # W_in: W_a (on x), then W_b (on x0)
        self.loop_in = self.loop_step = None
        if config.loop != NO_LOOP:
            self.loop_in = PackedLinear(Rows("x", 1, ((w, w),)), [columns_of("a", w), columns_of("b", w)])
            self.loop_step = nn.ModuleList([Fp32Vector(w) for _ in range(config.loop[2])])
        self.reset()

    def load_rest(self, tensors: Dict[str, Tensor]) -> None:
        self.final_norm.weight.mul_(self.config.logit_scale)   # the head is linear: its scale rides on the norm's
        if self.loop_in is None:
            return
        w, times = self.config.width, self.config.loop[2]
        t = assign_checked("loop", {"loop.in": (w, 2 * w), "loop.step": (times, w)}, tensors, "")
        self.loop_in.assign("a", t["loop.in"][:, :w])
        self.loop_in.assign("b", t["loop.in"][:, w:])
        for i, step in enumerate(self.loop_step):
            step.assign(t["loop.step"][i])

    def new_cache(self, batch: int, max_len: int) -> MixerCache:
        cache = MixerCache(batch, max_len, self.embed.weight.device, self.dtype)
        for i, run, _ in self.config.order():
            self.layers[i].mix.add_to_cache(cache, run)
        return cache

    @torch.no_grad()
    def forward(self, input_ids: Tensor, kv_cache: Optional[MixerCache] = None, positions: Optional[Tensor] = None,
                logits_at: Optional[Tensor] = None, residuals: Optional[list] = None) -> Dict[str, Tensor]:
        """See ``MixerLM.begin``; ``logits_at``: indices into the block; only these tokens' logits are formed;
        ``residuals``: takes a copy of the residual after every layer that runs."""
        ctx = self.begin(input_ids, kv_cache, positions)
        cfg, eps, dtype, w = self.config, self.config.eps, self.dtype, self.config.width
        order = cfg.order()
        # the norm after step k's residual sum; None where a pass begins: its input projection reads x itself
        pre = [None if begins else self.layers[i].norm1.weight for i, _, begins in order] + [self.final_norm.weight]
        x, h = _mix.sum_norm(self.embed.weight, pre[0], dtype, eps, tokens=input_ids.reshape(-1).contiguous(),
                             mult=cfg.embedding_scale)
        u = None
        if self.loop_in is not None:
            b = self.loop_in.offset["b"]
            if not order[0][2]:
                u = linear_f32(x.to(dtype), self.loop_in.weight[b:])[:, :w]
        for k, (i, ctx.run, begins) in enumerate(order):
            layer = self.layers[i]
            if begins:
                if u is None:
                    both = linear_f32(h, self.loop_in.weight)
                    y, u = both[:, :w], both[:, b:b + w]
                else:
                    y = linear_f32(h, self.loop_in.weight[:b])[:, :w]
                _, h = _mix.sum_norm(y, layer.norm1.weight, dtype, eps, u=u, vec=self.loop_step[ctx.run].weight, out=x)
            y = layer.mix(h, ctx)
            if layer.mlp is not None:
                _, h = _mix.sum_norm(y, layer.norm2.weight, dtype, eps, x=x, out=x)
                y = layer.mlp(h)
            _, h = _mix.sum_norm(y, pre[k + 1], dtype, eps, x=x, out=x)
            if residuals is not None:
                residuals.append(x.reshape(ctx.batch, ctx.seq, w).clone())
        return self.finish(h, x, ctx, logits_at)
