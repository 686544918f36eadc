"""Building blocks of decoders whose layers differ in their sequence mixer and keep an fp32
residual stream, on the kernels of ``astrai_amd.extension._mix``:

  ``PackedLinear``        several projections of one input stored and run as one matrix, each head's
                          rows padded to what the kernels take
  ``LatentAttention``     sliding-window attention over cached latents, own or another layer's
  ``LightningAttention``  linear attention with a constant decay per head
  ``GroupedAttention``    grouped-query attention: normed and rotated queries and keys, soft-capped scores,
                          a sink, an output gate per element
  ``GatedRecurrence``     real-gated linear recurrent unit behind a short convolution
  ``ChannelDelta``        gated delta rule with a decay per key channel, behind short convolutions
  ``GatedMLP``            ``down(act(gate(h)) * up(h))``
  ``MixerLM``             what decoders made of these share: weights by stored name, caches, a forward's context

All constants are constructor arguments. A mixer maps the normed input ``h [batch * seq, width]``
to its output of the same shape and reads and writes its layer's part of a ``MixerCache``.
Padded rows and columns of weights are zero, so padded activations are zero everywhere.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence, Tuple

import torch
import torch.nn as nn
import torch.nn.functional as F
from torch import Tensor

from astrai_amd.extension import _mix
from astrai_amd.extension._mix import RING_STEPS, DeltaShape, GqaShape, LatentShape, pad_to
from astrai_amd.model.cache import MixerCache
from astrai_amd.model.decoder import Embedding, Linear, rotary_table, yarn_frequencies

# a block of at most this many tokens attends in the latent space, longer ones form keys and values
LATENT_ROWS_MAX = 16
# a block of at most this many tokens attends with the split-context kernel
GQA_ROWS_MAX = 16
# a block of at most this many tokens runs the recurrence token by token
LIGHTNING_STEP_MAX = 8


@dataclass
class StepContext:
    """One forward: ``seq`` new tokens of each of ``batch`` sequences, at positions ``start ..`` (also
    on the device). ``run``: the pass that layers are in, if they run several times."""

    cache: MixerCache
    positions: Tensor
    start: int
    batch: int
    seq: int
    run: int = 0


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
    input columns are packed (a ``Rows`` over them). The projections named in ``biased`` have a bias,
    stored as ``<name>.b``."""

    def __init__(self, inputs: Rows, rows: Sequence[Rows], biased: Sequence[str] = ()):
        super().__init__(inputs.padded, sum(r.padded for r in rows), bias=bool(biased))
        self.inputs, self.rows, self.biased = inputs, list(rows), list(biased)
        self.offset: Dict[str, int] = {}
        at = 0
        for r in self.rows:
            self.offset[r.name] = at
            at += r.padded
        self.out_cols = at

    def expected(self) -> Dict[str, Tuple[int, ...]]:
        out = {r.name: (r.size, self.inputs.size) for r in self.rows}
        out.update({r.name + ".b": (r.size,) for r in self.rows if r.name in self.biased})
        return out

    def reset_parameters(self):
        std = self.inputs.size ** -0.5
        for r in self.rows:
            self.assign(r.name, torch.randn(r.size, self.inputs.size, device=self.weight.device) * std)

    @torch.no_grad()
    def assign(self, name: str, t: Tensor) -> None:
        r = next(r for r in self.rows if name in (r.name, r.name + ".b"))
        t = t.to(device=self.weight.device, dtype=self.weight.dtype)
        if name != r.name:
            self.bias[self.offset[r.name]:self.offset[r.name] + r.padded] = r.pack(t)
            return
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


def linear_f32(x: Tensor, weight: Tensor) -> Tensor:
    """``x W^T`` in fp32: bf16 operands keep their fp32 accumulators' digits."""
    if x.dtype == torch.float32:
        return F.linear(x, weight)
    return torch.mm(x, weight.t(), out_dtype=torch.float32)


class BlockDiagonal(nn.Module):
    """``blocks`` square matrices ``[out, in]`` with a bias each, padded to ``blocks x [bp, bp]``."""

    def __init__(self, part: Rows):
        super().__init__()
        self.part = part
        self.blocks, self.size, self.bp = part.groups, part.size // part.groups, part.padded // part.groups
        self.weight = nn.Parameter(torch.zeros(self.blocks, self.bp, self.bp))
        self.bias = Fp32Vector(part.size, part)
        self.transposed: Optional[Tensor] = None   # set by finalize

    def reset_parameters(self):
        with torch.no_grad():
            self.weight.zero_()
            n = self.size
            self.weight[:, :n, :n] = torch.randn(self.blocks, n, n, device=self.weight.device) * n ** -0.5
            self.bias.weight.zero_()

    @torch.no_grad()
    def assign(self, weight: Tensor, bias: Tensor) -> None:
        self.weight.zero_()
        self.weight[:, :self.size, :self.size] = weight.to(self.weight)
        self.bias.assign(bias.reshape(-1))

    @torch.no_grad()
    def finalize(self, transposed: bool) -> None:
        self.transposed = self.weight.transpose(1, 2).contiguous() if transposed else None


class ShortConv(nn.Module):
    """Taps (and a bias) of a causal convolution over the padded columns of the projections ``rows``, fp32
    ``[taps, columns]``, the last row on the current token."""

    def __init__(self, rows: Sequence[Rows], taps: int, bias: bool = False):
        super().__init__()
        self.rows, self.taps = list(rows), taps
        self.cols = sum(r.padded for r in rows)
        self.table = Fp32Vector(taps * self.cols)
        self.table.assign(torch.full((taps * self.cols,), 1.0 / taps))
        self.bias = Fp32Vector(self.cols) if bias else None
        if bias:
            self.bias.assign(torch.zeros(self.cols))

    @property
    def weight(self) -> Tensor:
        return self.table.weight.view(self.taps, self.cols)

    @torch.no_grad()
    def assign(self, taps: Sequence[Tensor], bias: Optional[Tensor] = None) -> None:
        """``taps[i] [channels, taps]`` of ``rows[i]``; the bias of the only projection."""
        self.table.assign(torch.cat([r.pack(t.float()) for r, t in zip(self.rows, taps)]).t().reshape(-1))
        if bias is not None:
            self.bias.assign(self.rows[0].pack(bias.float()))


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
            cache.add_rows(self.layer, self.shape.cache_cols)
        cache.add_rotary(self.rotation, self.rotation.table)

    def forward(self, h: Tensor, ctx: StepContext) -> Tensor:
        s, cache = self.shape, ctx.cache
        latent = cache.rows[self.kv_layer]
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


class GroupedAttention(nn.Module):
    """Causal softmax attention of ``heads`` query heads over ``kv_heads`` cached key / value heads. Queries and keys
    are RMS-normed per head (plain weights) and rotated; scores are ``softcap * tanh(q . k * scale / softcap)``; the
    softmax denominator has one more term ``exp(0)``; the heads are multiplied by a sigmoid of their own projection
    of the input before the output projection. q, k, v and the output projection have biases."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, rotation: Rotation, scale: float,
                 softcap: float, eps: float, layer: int):
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"layer {layer}: {heads} heads do not share {kv_heads} key/value heads evenly")
        if rotation.dims > dim or rotation.dims % 2:
            raise ValueError(f"layer {layer}: rotation over {rotation.dims} of {dim} dimensions")
        self.layer, self.rotation, self.eps = layer, rotation, eps
        self.shape = GqaShape(heads, kv_heads, pad_to(dim), pad_to(vdim), dim, scale, softcap, True)
        key = heads_of("k", 1, dim)
        values = heads_of("h", heads, vdim)
        self.in_proj = PackedLinear(Rows("h", 1, ((width, width),)), [
            heads_of("q", heads, dim), heads_of("k", kv_heads, dim), heads_of("v", kv_heads, vdim),
            heads_of("g", heads, vdim)], biased=("q", "k", "v"))
        self.o = PackedLinear(values, [Rows("o", 1, ((width, width),))], biased=("o",))
        self.q_norm, self.k_norm = Fp32Vector(dim, key), Fp32Vector(dim, key)

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        for lin in (self.in_proj, self.o):
            for name, t in assign_checked("attention", lin.expected(), tensors, prefix).items():
                lin.assign(name, t)
        for name, norm in (("q.norm", self.q_norm), ("k.norm", self.k_norm)):
            norm.assign(assign_checked("attention", {name: (norm.dim,)}, tensors, prefix)[name])

    def finalize(self) -> None:
        pass

    def add_to_cache(self, cache: MixerCache, run: int = 0) -> None:
        cache.add_rows((self.layer, run), self.shape.cache_cols)
        cache.add_rotary(self.rotation, self.rotation.table)

    def forward(self, h: Tensor, ctx: StepContext) -> Tensor:
        s, off, kv = self.shape, self.in_proj.offset, ctx.cache.rows[self.layer, ctx.run]
        proj = self.in_proj(h)
        _mix.gqa_append(proj, s, off["k"], off["v"], ctx.cache.rotary[self.rotation], ctx.positions,
                        self.q_norm.weight, self.k_norm.weight, kv, self.eps)
        bf16 = proj.dtype == torch.bfloat16
        if ctx.seq > GQA_ROWS_MAX and bf16 and _mix.gqa_prefill_supported(s):
            out = _mix.gqa_prefill(proj, s, off["g"], kv, ctx.start)
        else:
            out = _mix.gqa_rows(proj, s, off["g"], kv, ctx.positions,
                                matrix=bf16 and _mix.gqa_rows_supported(s, ctx.cache.max_len))
        return self.o(out)


class GatedRecurrence(nn.Module):
    """Griffin's recurrent block: ``y = gelu(W_y h + b)`` beside ``u = conv(W_x h + b)``; per channel
    ``S <- a S + sqrt(1 - a^2) i u`` with ``log a = -8 r softplus(lam)``, r and i sigmoids of block-diagonal
    projections of u; output ``W_o (S * y)``."""

    def __init__(self, width: int, channels: int, blocks: int, taps: int, layer: int):
        super().__init__()
        if channels % blocks:
            raise ValueError(f"layer {layer}: {channels} channels do not make {blocks} equal blocks")
        self.layer, self.channels = layer, channels
        part = heads_of("u", blocks, channels // blocks)
        self.in_proj = PackedLinear(Rows("h", 1, ((width, width),)), [
            Rows("y", part.groups, part.parts), Rows("x", part.groups, part.parts)], biased=("y", "x"))
        self.conv = ShortConv([part], taps, bias=True)
        self.r, self.i = BlockDiagonal(part), BlockDiagonal(part)
        self.coef = Fp32Vector(channels, part)
        self.set_lam(torch.full((channels,), -2.0))
        self.o = PackedLinear(part, [Rows("o", 1, ((width, width),))])

    def set_lam(self, lam: Tensor) -> None:
        self.coef.assign(-8.0 * F.softplus(lam.double()))

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        for lin in (self.in_proj, self.o):
            for name, t in assign_checked("recurrence", lin.expected(), tensors, prefix).items():
                lin.assign(name, t)
        n, b, c = self.r.size, self.r.blocks, self.channels
        t = assign_checked("recurrence", {"conv": (c, self.conv.taps), "conv.b": (c,), "ra": (b, n, n), "ra.b": (b, n),
                                          "ri": (b, n, n), "ri.b": (b, n), "lam": (c,)}, tensors, prefix)
        self.conv.assign([t["conv"]], t["conv.b"])
        self.r.assign(t["ra"], t["ra.b"])
        self.i.assign(t["ri"], t["ri.b"])
        self.set_lam(t["lam"])

    def _matrix(self) -> bool:
        return self.r.weight.dtype == torch.bfloat16 and _mix.rglru_chunk_supported(self.r.bp)

    def finalize(self) -> None:
        for m in (self.r, self.i):
            m.finalize(not self._matrix())

    def add_to_cache(self, cache: MixerCache, run: int = 0) -> None:
        cache.add_state((self.layer, run), self.conv.cols)
        cache.add_ring((self.layer, run), _mix.ring_rows(self.conv.taps), self.conv.cols)

    def forward(self, h: Tensor, ctx: StepContext) -> Tensor:
        proj, off, slot = self.in_proj(h), self.in_proj.offset, (self.layer, ctx.run)
        state, ring, matrix = ctx.cache.state[slot], ctx.cache.ring[slot], self._matrix()
        gates = (self.r.bias.weight, self.i.bias.weight, self.coef.weight, state)
        if ctx.seq <= RING_STEPS and proj.dtype == torch.bfloat16:
            out = _mix.rglru_step(proj, off["y"], off["x"], self.conv.weight, self.conv.bias.weight, ring, ctx.positions,
                                  self.r.weight, self.i.weight, *gates)
        else:
            u = _mix.conv(proj, off["x"], self.conv.weight, self.conv.bias.weight, ring, ctx.positions, silu=False)
            w = [m.weight if matrix else m.transposed for m in (self.r, self.i)]
            out = _mix.rglru(u, proj, off["y"], *w, *gates, matrix=matrix)
        return self.o(out)


class ChannelDelta(nn.Module):
    """Gated delta rule: per head ``S <- g * S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q`` with one decay
    ``g = exp(-exp(A_log) softplus(a2 a1 h + dt_bias))`` per head and key channel. q, k (``kv_heads``, shared by groups
    of heads) and v pass a short convolution and silu, q and k become unit vectors; each head's output is
    RMS-normed (plain weight) and gated by ``sigmoid(g2 g1 h)``."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, rank: int, gate_rank: int,
                 eps: float, layer: int):
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"layer {layer}: {heads} heads do not share {kv_heads} query/key heads evenly")
        self.layer, self.eps = layer, eps
        self.shape = DeltaShape(heads, kv_heads, pad_to(dim), pad_to(vdim), vdim, dim ** -0.5)
        qkv = [heads_of("q", kv_heads, dim), heads_of("k", kv_heads, dim), heads_of("v", heads, vdim)]
        a1, g1 = columns_of("a1", rank), columns_of("g1", gate_rank)
        values = heads_of("h", heads, vdim)
        self.in_proj = PackedLinear(Rows("h", 1, ((width, width),)), [*qkv, columns_of("b", heads), a1, g1])
        self.conv = ShortConv(qkv, taps)
        self.channels = heads_of("a2", heads, dim)
        self.a2 = PackedLinear(a1, [self.channels])
        self.g2 = PackedLinear(g1, [heads_of("g2", heads, vdim)])
        self.o = PackedLinear(values, [Rows("o", 1, ((width, width),))])
        self.dt_bias = Fp32Vector(heads * dim, self.channels)
        self.dt_bias.assign(torch.full((heads * dim,), -4.0))
        self.decay = Fp32Vector(heads)
        self.norm = Fp32Vector(vdim, heads_of("norm", 1, vdim))

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        for lin in (self.in_proj, self.a2, self.g2, self.o):
            for name, t in assign_checked("delta rule", lin.expected(), tensors, prefix).items():
                lin.assign(name, t)
        t = assign_checked("delta rule", {**{r.name + ".conv": (r.size, self.conv.taps) for r in self.conv.rows},
                                          "A_log": (self.shape.heads,), "dt_bias": (self.channels.size,),
                                          "norm": (self.norm.dim,)}, tensors, prefix)
        self.conv.assign([t[r.name + ".conv"] for r in self.conv.rows])
        self.decay.assign(t["A_log"].double().exp())
        self.dt_bias.assign(t["dt_bias"])
        self.norm.assign(t["norm"])

    def finalize(self) -> None:
        pass

    def add_to_cache(self, cache: MixerCache, run: int = 0) -> None:
        s, slot = self.shape, (self.layer, run)
        cache.add_state(slot, s.heads, s.dp, s.vp)
        cache.add_ring(slot, _mix.ring_rows(self.conv.taps), self.conv.cols)

    def forward(self, h: Tensor, ctx: StepContext) -> Tensor:
        proj, off, s, slot = self.in_proj(h), self.in_proj.offset, self.shape, (self.layer, ctx.run)
        state, ring = ctx.cache.state[slot], ctx.cache.ring[slot]
        z = linear_f32(proj[:, off["a1"]:off["a1"] + self.a2.inputs.padded], self.a2.weight)
        gate = self.g2(proj[:, off["g1"]:off["g1"] + self.g2.inputs.padded])
        rule = (s, off["b"], z, self.dt_bias.weight, self.decay.weight)
        bf16 = proj.dtype == torch.bfloat16
        if ctx.seq <= RING_STEPS and bf16 and _mix.delta_step_supported(s):
            out = _mix.delta_step(proj, *rule, gate, self.norm.weight, state, self.eps, x_off=off["q"],
                                  conv_w=self.conv.weight, ring=ring, positions=ctx.positions)
        else:
            qkv = _mix.conv(proj, off["q"], self.conv.weight, None, ring, ctx.positions, silu=True)
            if bf16 and _mix.delta_chunk_supported(s):
                o = _mix.delta_chunk(qkv, proj, *rule, state)
                out = _mix.head_gated_rms_norm(o, gate, self.norm.weight, s.vdim, self.eps)
            else:
                out = _mix.delta_step(proj, *rule, gate, self.norm.weight, state, self.eps, qkv=qkv)
        return self.o(out)


class GatedMLP(nn.Module):
    def __init__(self, width: int, ff: int, act: str = "silu"):
        super().__init__()
        self.act = act
        hidden = columns_of("up", ff)
        self.gate_up = PackedLinear(Rows("h", 1, ((width, width),)), [columns_of("gate", ff), hidden])
        self.down = PackedLinear(hidden, [Rows("down", 1, ((width, width),))])

    def load(self, tensors: Dict[str, Tensor], prefix: str) -> None:
        for lin in (self.gate_up, self.down):
            for name, t in assign_checked("feed-forward", lin.expected(), tensors, prefix).items():
                lin.assign(name, t)

    def forward(self, h: Tensor) -> Tensor:
        return self.down(_mix.act_mul(self.gate_up(h), self.act))


class MixerLM(nn.Module):
    """Embedding, layers (each with a ``mix``), final norm and head. Same calling convention as
    ``AutoRegressiveLM``: ``model(ids, cache, positions)["logits"]``."""

    def __init__(self, config, layers: List[nn.Module]):
        super().__init__()
        self.config = config
        self.embed = Embedding(config.vocab, config.width)
        self.layers = nn.ModuleList(layers)
        self.final_norm = Fp32Vector(config.width)
        self.head = Linear(config.width, config.vocab)
        self._ready = False

    def reset(self) -> None:
        """Random weights; called at the end of a subclass's constructor."""
        self.apply(lambda m: m.reset_parameters() if hasattr(m, "reset_parameters") else None)

    @property
    def dtype(self) -> torch.dtype:
        return self.embed.weight.dtype

    @torch.no_grad()
    def load_tensors(self, tensors: Dict[str, Tensor]) -> "MixerLM":
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
        self.load_rest(left)
        if left:
            raise ValueError(f"checkpoint does not match the model: unexpected {sorted(left)[:8]}")
        self._ready = False
        return self

    def load_rest(self, tensors: Dict[str, Tensor]) -> None:
        """Take the tensors that belong to no layer out of ``tensors``."""

    def _apply(self, fn, recurse=True):
        self._ready = False
        return super()._apply(fn, recurse)

    def finalize(self) -> "MixerLM":
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

    def begin(self, input_ids: Tensor, kv_cache: Optional[MixerCache], positions: Optional[Tensor]) -> StepContext:
        """``input_ids [batch, seq]``: the tokens after those the cache holds, ``kv_cache.tokens`` of them
        (``positions``, if given, is those tokens' positions on the device; the caller advances the
        cache). Without a cache: a sequence of its own."""
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
        return StepContext(kv_cache, positions, kv_cache.tokens, b, s)

    def finish(self, h: Tensor, x: Tensor, ctx: StepContext, logits_at: Optional[Tensor]) -> Dict[str, Tensor]:
        """Logits of the normed rows ``h``, of all tokens or of the places ``logits_at`` in the block."""
        hidden = h.reshape(ctx.batch, ctx.seq, -1)
        if logits_at is not None:
            hidden = hidden.index_select(1, logits_at)
        return {"logits": self.head(hidden), "hidden_states": hidden, "residual": x.reshape(ctx.batch, ctx.seq, -1)}
