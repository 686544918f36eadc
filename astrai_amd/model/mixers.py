"""Building blocks of decoders whose layers differ in their sequence mixer and keep an fp32
residual stream, on the kernels of ``astrai_amd.extension._mix``:

  ``PackedLinear``        several projections of one input stored and run as one matrix, each head's
                          rows padded to what the kernels take
  ``LatentAttention``     sliding-window attention over cached latents, own or another layer's
  ``LightningAttention``  linear attention with a constant decay per head
  ``GatedMLP``            ``down(silu(gate(h)) * up(h))``

All constants are constructor arguments. A mixer maps the normed input ``h [batch * seq, width]``
to its output of the same shape and reads and writes its layer's part of a ``MixerCache``.
Padded rows and columns of weights are zero, so padded activations are zero everywhere.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Dict, Optional, Sequence, Tuple

import torch
import torch.nn as nn
import torch.nn.functional as F
from torch import Tensor

from astrai_amd.extension import _mix
from astrai_amd.extension._mix import LatentShape, pad_to
from astrai_amd.model.cache import MixerCache
from astrai_amd.model.decoder import Linear, rotary_table, yarn_frequencies

# a block of at most this many tokens attends in the latent space, longer ones form keys and values
LATENT_ROWS_MAX = 16
# a block of at most this many tokens runs the recurrence token by token
LIGHTNING_STEP_MAX = 8


@dataclass
class StepContext:
    """One forward: ``seq`` new tokens of each of ``batch`` sequences, at positions ``start ..`` (also
    on the device)."""

    cache: MixerCache
    positions: Tensor
    start: int
    batch: int
    seq: int


@dataclass(frozen=True)
class Rows:
    """Output rows of one projection: ``groups`` blocks (heads), each a run of parts ``(size, padded)``."""

    name: str
    groups: int
    parts: Tuple[Tuple[int, int], ...]

    @property
    def size(self) -> int:
        return self.groups * sum(s for s, _ in self.parts)

    @property
    def padded(self) -> int:
        return self.groups * sum(p for _, p in self.parts)

    def pack(self, t: Tensor) -> Tensor:
        """``[size, ...]`` -> ``[padded, ...]`` with zero rows."""
        t = t.reshape(self.groups, -1, *t.shape[1:])
        out = t.new_zeros((self.groups, sum(p for _, p in self.parts), *t.shape[2:]))
        src = dst = 0
        for size, padded in self.parts:
            out[:, dst:dst + size] = t[:, src:src + size]
            src, dst = src + size, dst + padded
        return out.reshape(self.padded, *t.shape[2:])


def heads_of(name: str, heads: int, *dims: int) -> Rows:
    return Rows(name, heads, tuple((d, pad_to(d)) for d in dims))


def columns_of(name: str, n: int, q: int = 8) -> Rows:
    return Rows(name, 1, ((n, pad_to(n, q)),))


class PackedLinear(Linear):
    """``F.linear`` with one weight ``[sum of padded rows, padded input columns]`` that holds several
    projections; ``offset[name]`` is the first output column of each. ``inputs`` describes how the
    input columns are packed (a ``Rows`` over them)."""

    def __init__(self, inputs: Rows, rows: Sequence[Rows]):
        super().__init__(inputs.padded, sum(r.padded for r in rows))
        self.inputs, self.rows = inputs, list(rows)
        self.offset: Dict[str, int] = {}
        at = 0
        for r in self.rows:
            self.offset[r.name] = at
            at += r.padded
        self.out_cols = at

    def expected(self) -> Dict[str, Tuple[int, ...]]:
        return {r.name: (r.size, self.inputs.size) for r in self.rows}

    def reset_parameters(self):
        std = self.inputs.size ** -0.5
        for r in self.rows:
            self.assign(r.name, torch.randn(r.size, self.inputs.size, device=self.weight.device) * std)

    @torch.no_grad()
    def assign(self, name: str, t: Tensor) -> None:
        r = next(r for r in self.rows if r.name == name)
        t = t.to(device=self.weight.device, dtype=self.weight.dtype)
        packed = self.inputs.pack(r.pack(t).t().contiguous()).t()
        self.weight[self.offset[name]:self.offset[name] + r.padded] = packed


def assign_checked(owner: str, expected: Dict[str, Tuple[int, ...]], tensors: Dict[str, Tensor], prefix: str) -> Dict[str, Tensor]:
    """The tensors ``prefix + name`` of ``expected``, taken out of ``tensors`` after a shape check."""
    out = {}
    for name, shape in expected.items():
        t = tensors.pop(prefix + name, None)
        if t is None:
            raise ValueError(f"{owner}: tensor {prefix + name} is missing")
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"{owner}: tensor {prefix + name} has shape {tuple(t.shape)}, expected {tuple(shape)}")
        out[name] = t
    return out


class Fp32Vector(nn.Module):
    """A vector that kernels read in fp32 whatever the model's dtype is: a norm's weight, a table of
    decay powers."""

    def __init__(self, dim: int, rows: Optional[Rows] = None):
        super().__init__()
        self.dim, self.rows = dim, rows
        self.register_buffer("weight", torch.ones(dim) if rows is None else rows.pack(torch.ones(dim)))

    def _apply(self, fn, recurse=True):
        # follows the module's device but not its dtype
        self.weight = self.weight.to(fn(self.weight).device)
        return self

    @torch.no_grad()
    def assign(self, t: Tensor) -> None:
        t = t.float()
        self.weight.copy_(t if self.rows is None else self.rows.pack(t))


@dataclass(frozen=True)
class Rotation:
    """Rotary positions: ``dims`` rotated dimensions in the rotate-half pairing, frequencies
    ``base^(-2i/dims)``, optionally under YaRN scaling."""

    dims: int
    base: float
    yarn: Optional[Tuple[float, float, float, float]] = None   # factor, original, fast, slow

    @staticmethod
    def from_dict(d: dict) -> "Rotation":
        s = d.get("scaling")
        yarn = None if s is None else (float(s["factor"]), float(s["original"]), float(s["fast"]), float(s["slow"]))
        return Rotation(int(d["dims"]), float(d["base"]), yarn)

    def table(self, max_len: int, device="cpu") -> Tensor:
        """``[max_len, dims / 2, 2]`` fp32 (cos, sin) on ``device``, YaRN's magnitude included."""
        if self.yarn is None:
            freqs = self.base ** (-torch.arange(0, self.dims, 2, dtype=torch.float64) / self.dims)
            return rotary_table(freqs.to(device), max_len)
        factor, original, fast, slow = self.yarn
        freqs = yarn_frequencies(self.dims, self.base, factor, original, fast, slow)
        return rotary_table(freqs.to(device), max_len, 0.1 * math.log(factor) + 1.0)


class LatentAttention(nn.Module):
    """Per head, keys and values are projections ``uk``, ``uv`` of a latent that is cached in their place,
    next to one rotated key part shared by all heads. A query sees itself and the ``window - 1`` tokens
    before it (``window`` None: all of them); each head's output is gated by a sigmoid of its own
    projection of the input. With ``kv_from`` the layer reads that layer's latents."""

    def __init__(self, width: int, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, rotation: Rotation,
                 scale: float, window: Optional[int], eps: float, layer: int, kv_from: Optional[int] = None):
        super().__init__()
        if rotation.dims > rot_dim or rotation.dims % 2:
            raise ValueError(f"layer {layer}: rotation over {rotation.dims} of {rot_dim} dimensions")
        self.layer, self.kv_layer = layer, layer if kv_from is None else kv_from
        self.owns_latent = kv_from is None
        self.rotation, self.eps = rotation, eps
        self.shape = LatentShape(heads, pad_to(dim), pad_to(rot_dim), pad_to(kv_rank), pad_to(vdim), kv_rank,
                                 _mix.UNBOUNDED if window is None else window, scale)
        rows = [heads_of("q", heads, dim, rot_dim)]
        if self.owns_latent:
            rows.append(heads_of("dkv", 1, kv_rank, rot_dim))
        rows.append(columns_of("g", heads))
        self.in_proj = PackedLinear(Rows("h", 1, ((width, width),)), rows)
        latent = heads_of("c", 1, kv_rank)
        self.uk = PackedLinear(latent, [heads_of("uk", heads, dim)])
        self.uv = PackedLinear(latent, [heads_of("uv", heads, vdim)])
        self.o = PackedLinear(heads_of("h", heads, vdim), [Rows("o", 1, ((width, width),))])
        self.latent_norm = Fp32Vector(kv_rank, latent) if self.owns_latent else None
        self.w_ukv: Optional[Tensor] = None   # set by finalize
        self.w_uk_t: Optional[Tensor] = None

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        linears = [self.in_proj, self.uk, self.uv, self.o]
        for lin in linears:
            for name, t in assign_checked("latent attention", lin.expected(), tensors, prefix).items():
                lin.assign(name, t)
        if self.latent_norm is not None:
            t = assign_checked("latent attention", {"dkv.norm": (self.latent_norm.dim,)}, tensors, prefix)
            self.latent_norm.assign(t["dkv.norm"])

    @torch.no_grad()
    def finalize(self) -> None:
        """The layouts the kernels read: key and value rows interleaved per head, and (bf16) the key
        rows transposed for the absorbed query."""
        s = self.shape
        uk = self.uk.weight.reshape(s.heads, s.dn, s.rp)
        self.w_ukv = torch.cat([uk, self.uv.weight.reshape(s.heads, s.vp, s.rp)], dim=1).reshape(-1, s.rp).contiguous()
        self.w_uk_t = uk.transpose(1, 2).contiguous() if uk.dtype == torch.bfloat16 else None

    def add_to_cache(self, cache: MixerCache) -> None:
        if self.owns_latent:
            cache.add_latent(self.layer, self.shape.cache_cols)
        cache.add_rotary(self.rotation, self.rotation.table)

    def forward(self, h: Tensor, ctx: StepContext) -> Tensor:
        s, cache = self.shape, ctx.cache
        latent = cache.latent[self.kv_layer]
        proj = self.in_proj(h)
        g_off = self.in_proj.offset["g"]
        rows = ctx.seq <= LATENT_ROWS_MAX or proj.dtype != torch.bfloat16 or not _mix.latent_prefill_supported(s)
        absorb = rows and self.w_uk_t is not None and _mix.latent_rows_supported(s, cache.max_len)
        q_abs = _mix.latent_append(proj, s, self.in_proj.offset.get("dkv", -1), cache.rotary[self.rotation],
                                   ctx.positions, self.latent_norm.weight if self.owns_latent else None, latent,
                                   self.eps, self.w_uk_t if absorb else None)
        if rows:
            out = _mix.latent_rows(proj, s, g_off, self.w_ukv, latent, ctx.positions, q_abs)
        else:
            first = max(ctx.start - s.window + 1, 0)
            c = latent[:, first:ctx.start + ctx.seq, :s.rp]
            # (a plain 2-D product: a strided 3-D operand would go to a batched one)
            kv = F.linear(c[0] if ctx.batch == 1 else c.reshape(-1, s.rp), self.w_ukv)
            kv = kv.reshape(ctx.batch, -1, kv.size(-1))
            out = _mix.latent_prefill(proj, s, g_off, kv, latent, ctx.start, first)
        return self.o(out)


class LightningAttention(nn.Module):
    """``S <- decay_h S + k v^T``, ``o = S^T q`` per head on silu of the projections; the concatenated
    heads are RMS-normed together, gated by a sigmoid of a projection of the input, and projected."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, decay: Sequence[float], eps: float, layer: int):
        super().__init__()
        if len(decay) != heads:
            raise ValueError(f"layer {layer}: {len(decay)} decays for {heads} heads")
        self.layer, self.eps, self.heads = layer, eps, heads
        self.dp, self.vp, self.count = pad_to(dim), pad_to(vdim), heads * vdim
        values = heads_of("v", heads, vdim)
        self.in_proj = PackedLinear(Rows("h", 1, ((width, width),)), [
            heads_of("q", heads, dim), heads_of("k", heads, dim), values, heads_of("g", heads, vdim)])
        self.o = PackedLinear(values, [Rows("o", 1, ((width, width),))])
        self.norm = Fp32Vector(self.count, values)
        self.decay = Fp32Vector(heads * (_mix.LIGHTNING_CHUNK + 1))
        self.decay.assign(_mix.decay_powers(decay).reshape(-1))

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        for lin in (self.in_proj, self.o):
            for name, t in assign_checked("lightning attention", lin.expected(), tensors, prefix).items():
                lin.assign(name, t)
        self.norm.assign(assign_checked("lightning attention", {"norm": (self.count,)}, tensors, prefix)["norm"])

    def finalize(self) -> None:
        pass

    def add_to_cache(self, cache: MixerCache) -> None:
        cache.add_state(self.layer, self.heads, self.dp, self.vp)

    def forward(self, h: Tensor, ctx: StepContext) -> Tensor:
        proj, off = self.in_proj(h), self.in_proj.offset
        step = ctx.seq <= LIGHTNING_STEP_MAX or proj.dtype != torch.bfloat16 or not _mix.lightning_chunk_supported(self.dp)
        o = _mix.lightning(proj, off["q"], off["k"], off["v"], self.decay.weight.view(self.heads, -1),
                           ctx.cache.state[self.layer], step)
        return self.o(_mix.gated_rms_norm(o, proj, off["g"], self.norm.weight, self.count, self.eps))


class GatedMLP(nn.Module):
    def __init__(self, width: int, ff: int):
        super().__init__()
        hidden = columns_of("up", ff)
        self.gate_up = PackedLinear(Rows("h", 1, ((width, width),)), [columns_of("gate", ff), hidden])
        self.down = PackedLinear(hidden, [Rows("down", 1, ((width, width),))])

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        for lin in (self.gate_up, self.down):
            for name, t in assign_checked("feed-forward", lin.expected(), tensors, prefix).items():
                lin.assign(name, t)

    def forward(self, h: Tensor) -> Tensor:
        return self.down(_mix.silu_mul(self.gate_up(h)))
