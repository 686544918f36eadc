"""ctypes binding of ``lib/libastrai_mix.so`` (the C ABI in include/astrai_mix.h): latent, lightning
and grouped-query attention, the real-gated linear recurrent unit, the gated delta rule and the
row operations of decoders with an fp32 residual stream, as functions on tensors. As in ``_cabi``: shapes and devices are checked here, outputs and scratch
come from torch's allocator, the launch goes to torch's current stream, a failing status raises,
and without the HIP library every call raises (no CPU or PyTorch fallback).
"""

from __future__ import annotations

import ctypes
import os
from dataclasses import dataclass
from typing import Optional

import torch  # imported before the CDLL so the library binds to torch's HIP runtime

from astrai_amd.extension._cabi import _LIB_DIR, _on_device, _stream

LIB_PATH = os.path.join(_LIB_DIR, "libastrai_mix.so")

ABI_VERSION = 2
LIGHTNING_CHUNK = 64
MAX_SPLIT = 64
RING_STEPS = 8    # most tokens of a step that reads and writes a convolution's ring in one launch
DELTA_CHUNK = 16
HEAD_PAD = 32     # head sizes are padded to multiples of this
UNBOUNDED = 1 << 30   # window of a layer that sees every earlier token

_P = ctypes.c_void_p
_I64 = ctypes.c_int64
_INT = ctypes.c_int
_F32 = ctypes.c_float

# name -> argtypes, exactly the prototypes of include/astrai_mix.h
PROTOTYPES = {
    "astrai_mix_abi_version": ([], _INT),
    "astrai_mix_last_error": ([], ctypes.c_char_p),
    "astrai_mix_residual_norm": ([_P] * 6 + [_I64, _I64, _F32, _F32, _INT, _P], _INT),
    "astrai_mix_embed_norm": ([_P] * 5 + [_I64, _I64, _I64, _F32, _INT, _P], _INT),
    "astrai_mix_sum_norm": (
        [_P, _I64, _P, _I64, _F32, _P, _P, _I64] + [_P] * 4 + [_I64, _I64, _F32, _INT, _INT, _P], _INT),
    "astrai_mix_act_mul": ([_P, _P, _I64, _I64, _INT, _INT, _P], _INT),
    "astrai_mix_head_gated_rms_norm": ([_P, _P, _I64, _P, _P] + [_I64] * 4 + [_F32, _INT, _P], _INT),
    "astrai_mix_gated_rms_norm": ([_P, _P, _I64, _P, _P, _I64, _I64, _I64, _F32, _INT, _P], _INT),
    "astrai_mix_latent_append": (
        [_P, _I64, _I64, _P, _I64, _I64] + [_P] * 5 + [_I64] * 8 + [_F32, _INT, _P], _INT),
    "astrai_mix_latent_prefill": ([_P, _I64, _I64, _P, _P, _P] + [_I64] * 12 + [_F32, _P], _INT),
    "astrai_mix_latent_rows_workspace_floats": ([_I64] * 4, _I64),
    "astrai_mix_latent_rows": (
        [_P, _I64, _I64] + [_P] * 6 + [_I64] * 9 + [_F32, _I64, _P], _INT),
    "astrai_mix_latent_rows_general": ([_P, _I64, _I64, _P, _P, _P, _P] + [_I64] * 9 + [_F32, _INT, _P], _INT),
    "astrai_mix_lightning_chunk": ([_P] + [_I64] * 4 + [_P] * 4 + [_I64] * 6 + [_P], _INT),
    "astrai_mix_lightning_step": ([_P] + [_I64] * 4 + [_P] * 3 + [_I64] * 5 + [_INT, _P], _INT),
    "astrai_mix_gqa_append": ([_P, _I64, _I64, _I64, _P, _I64, _I64] + [_P] * 4 + [_I64] * 8 + [_F32, _INT, _P], _INT),
    "astrai_mix_gqa_prefill": ([_P, _I64, _I64, _P, _P] + [_I64] * 9 + [_F32, _F32, _INT, _P], _INT),
    "astrai_mix_gqa_rows_workspace_floats": ([_I64] * 4, _I64),
    "astrai_mix_gqa_rows": ([_P, _I64, _I64] + [_P] * 4 + [_I64] * 8 + [_F32, _F32, _INT, _I64, _P], _INT),
    "astrai_mix_gqa_rows_general": ([_P, _I64, _I64] + [_P] * 3 + [_I64] * 8 + [_F32, _F32, _INT, _INT, _P], _INT),
    "astrai_mix_conv": ([_P] + [_I64] * 3 + [_P, _P, _I64] + [_P] * 3 + [_I64, _I64] + [_INT] * 3 + [_P], _INT),
    "astrai_mix_rglru_chunk": ([_P, _P, _I64, _I64] + [_P] * 8 + [_I64] * 5 + [_P], _INT),
    "astrai_mix_rglru_general": ([_P, _P, _I64, _I64] + [_P] * 8 + [_I64] * 4 + [_INT, _P], _INT),
    "astrai_mix_rglru_step": ([_P] + [_I64] * 3 + [_P, _P, _I64] + [_P] * 9 + [_I64] * 4 + [_P], _INT),
    "astrai_mix_delta_step": (
        [_P, _P] + [_I64] * 3 + [_P, _I64] + [_P] * 6 + [_I64] + [_P] * 3 + [_I64] * 7 + [_F32, _F32, _INT, _P], _INT),
    "astrai_mix_delta_image_bytes": ([_I64], _I64),
    "astrai_mix_delta_chunk": ([_P, _P, _I64, _I64] + [_P] * 6 + [_I64] * 6 + [_F32, _P], _INT),
}

_lib: Optional[ctypes.CDLL] = None
_load_error: Optional[str] = None


def load() -> Optional[ctypes.CDLL]:
    """Load the library once; ``None`` (with the reason kept) if it is absent or of another ABI."""
    global _lib, _load_error
    if _lib is not None or _load_error is not None:
        return _lib
    if not os.path.exists(LIB_PATH):
        _load_error = f"{LIB_PATH} not built"
        return None
    try:
        lib = ctypes.CDLL(LIB_PATH)
        for name, (argtypes, restype) in PROTOTYPES.items():
            fn = getattr(lib, name)
            fn.argtypes = argtypes
            fn.restype = restype
        got = lib.astrai_mix_abi_version()
        if got != ABI_VERSION:
            raise OSError(f"ABI version {got}, expected {ABI_VERSION}")
    except (OSError, AttributeError) as e:
        _load_error = f"{type(e).__name__}: {e}"
        return None
    _lib = lib
    return _lib


def load_error() -> Optional[str]:
    return _load_error


def _require() -> ctypes.CDLL:
    lib = load()
    if lib is None:
        raise RuntimeError(f"HIP library libastrai_mix.so is not available ({_load_error}). "
                           "Build it with `make -C astrai_amd/csrc mix`.")
    return lib


def _check(rc: int, lib: ctypes.CDLL) -> None:
    if rc != 0:
        raise RuntimeError(f"astrai_mix error {rc}: {lib.astrai_mix_last_error().decode('utf-8', 'replace')}")


_DTYPES = {torch.bfloat16: 0, torch.float32: 1}


def _dtype(t: torch.Tensor, what: str) -> int:
    if t.dtype not in _DTYPES:
        raise RuntimeError(f"{what}: bf16 or float32 required, got {t.dtype}")
    return _DTYPES[t.dtype]


def _dense(what: str, dtype, *tensors: torch.Tensor) -> None:
    """Contiguous tensors of one dtype on one GPU."""
    dev = tensors[0].device
    for t in tensors:
        if not t.is_cuda or t.device != dev:
            raise RuntimeError(f"{what}: CUDA tensors on one device required")
        if t.dtype != dtype:
            raise RuntimeError(f"{what}: expected {dtype}, got {t.dtype}")
        if not t.is_contiguous():
            raise RuntimeError(f"{what}: contiguous tensors required")


def _shape(what: str, t: torch.Tensor, *shape: int) -> None:
    if tuple(t.shape) != shape:
        raise RuntimeError(f"{what}: expected shape {shape}, got {tuple(t.shape)}")


def pad_to(n: int, q: int = HEAD_PAD) -> int:
    return -(-n // q) * q


# ---------------------------------------------------------------------------
# Row operations
# ---------------------------------------------------------------------------


def residual_norm(y: torch.Tensor, x: torch.Tensor, w_post: torch.Tensor, w_pre: torch.Tensor, mult: float,
                  eps: float) -> torch.Tensor:
    """``x += mult * LN(y) * w_post`` (in place, fp32) and ``LN(x) * w_pre`` in ``y``'s dtype, returned."""
    lib = _require()
    n, width = y.shape
    code = _dtype(y, "residual_norm")
    _dense("residual_norm", y.dtype, y)
    _dense("residual_norm", torch.float32, x, w_post, w_pre)
    _shape("residual_norm", x, n, width)
    _shape("residual_norm", w_post, width)
    _shape("residual_norm", w_pre, width)
    with _on_device(y.device):
        h = torch.empty_like(y)
        _check(lib.astrai_mix_residual_norm(y.data_ptr(), x.data_ptr(), x.data_ptr(), w_post.data_ptr(),
                                            w_pre.data_ptr(), h.data_ptr(), n, width, mult, eps, code, _stream(y)), lib)
    return h


def embed_norm(table: torch.Tensor, tokens: torch.Tensor, w_pre: torch.Tensor, eps: float):
    """``x = table[tokens]`` as the fp32 residual and ``LN(x) * w_pre`` in the table's dtype."""
    lib = _require()
    vocab, width = table.shape
    code = _dtype(table, "embed_norm")
    _dense("embed_norm", table.dtype, table)
    _dense("embed_norm", torch.int64, tokens)
    _dense("embed_norm", torch.float32, w_pre)
    _shape("embed_norm", w_pre, width)
    if tokens.device != table.device:
        raise RuntimeError("embed_norm: tokens and table must be on one device")
    n = tokens.numel()
    with _on_device(table.device):
        x = torch.empty((n, width), device=table.device, dtype=torch.float32)
        h = torch.empty((n, width), device=table.device, dtype=table.dtype)
        _check(lib.astrai_mix_embed_norm(table.data_ptr(), tokens.data_ptr(), x.data_ptr(), w_pre.data_ptr(),
                                         h.data_ptr(), n, width, vocab, eps, code, _stream(table)), lib)
    return x, h


def sum_norm(y: torch.Tensor, w: Optional[torch.Tensor], dtype: torch.dtype, eps: float,
             x: Optional[torch.Tensor] = None, u: Optional[torch.Tensor] = None, vec: Optional[torch.Tensor] = None,
             tokens: Optional[torch.Tensor] = None, mult: float = 1.0, out: Optional[torch.Tensor] = None):
    """The residual ``mult * y + x + u + vec`` in fp32 (every term but the first optional; ``y`` the table whose rows
    ``tokens`` are taken, if given) and its RMS norm times ``w`` in ``dtype`` (without ``w``: the residual itself).
    ``y [n, width]`` and ``u`` may be rows of a wider matrix and have one type, ``dtype`` or float32. The residual
    goes to ``out`` (which may be ``x``) or a new tensor. Returns (residual, normed)."""
    lib = _require()
    width = y.size(1)
    n = y.size(0) if tokens is None else tokens.numel()
    code = _DTYPES[dtype]
    for t in (y, u):
        if t is None:
            continue
        if not t.is_cuda or t.dim() != 2 or t.stride(1) != 1 or t.stride(0) < width or t.size(1) != width:
            raise RuntimeError(f"sum_norm: rows of {width} on the GPU required")
        if t.dtype != y.dtype or t.dtype not in (dtype, torch.float32):
            raise RuntimeError(f"sum_norm: {t.dtype} terms with {y.dtype} and {dtype}")
    if tokens is not None:
        _dense("sum_norm", torch.int64, tokens)
    if u is not None:
        _shape("sum_norm", u, n, width)
    for t, shape in ((x, (n, width)), (out, (n, width)), (vec, (width,)), (w, (width,))):
        if t is not None:
            _dense("sum_norm", torch.float32, t)
            _shape("sum_norm", t, *shape)
    if any(t is not None and t.device != y.device for t in (x, u, vec, tokens, out, w)):
        raise RuntimeError("sum_norm: tensors on one device required")

    def ptr(t):
        return None if t is None else t.data_ptr()

    with _on_device(y.device):
        if out is None:
            out = torch.empty((n, width), device=y.device, dtype=torch.float32)
        h = torch.empty((n, width), device=y.device, dtype=dtype)
        _check(lib.astrai_mix_sum_norm(y.data_ptr(), y.stride(0), ptr(tokens), y.size(0), mult, ptr(x), ptr(u),
                                       0 if u is None else u.stride(0), ptr(vec), out.data_ptr(), ptr(w), h.data_ptr(),
                                       n, width, eps, int(y.dtype == torch.float32), code, _stream(y)), lib)
    return out, h


ACTIVATIONS = {"silu": 0, "gelu_tanh": 1}


def act_mul(gu: torch.Tensor, act: str) -> torch.Tensor:
    """``act(gate) * up`` of ``gu [n, 2 ff]`` (gate columns, then up)."""
    lib = _require()
    code = _dtype(gu, "act_mul")
    _dense("act_mul", gu.dtype, gu)
    n, ff = gu.size(0), gu.size(1) // 2
    with _on_device(gu.device):
        h = torch.empty((n, ff), device=gu.device, dtype=gu.dtype)
        _check(lib.astrai_mix_act_mul(gu.data_ptr(), h.data_ptr(), n, ff, ACTIVATIONS[act], code, _stream(gu)), lib)
    return h


def silu_mul(gu: torch.Tensor) -> torch.Tensor:
    return act_mul(gu, "silu")


def head_gated_rms_norm(o: torch.Tensor, g: torch.Tensor, weight: torch.Tensor, count: int, eps: float) -> torch.Tensor:
    """:func:`gated_rms_norm` of each head: ``o [n, heads * vp]``, gate logits ``g`` (rows of a wider matrix allowed),
    ``weight [vp]``; ``count`` of a head's columns are real."""
    lib = _require()
    n, width = o.shape
    vp = weight.numel()
    _dense("head_gated_rms_norm", o.dtype, o)
    _dense("head_gated_rms_norm", torch.float32, weight)
    if g.shape != o.shape or g.dtype != o.dtype or g.device != o.device or g.stride(1) != 1 or width % vp:
        raise RuntimeError("head_gated_rms_norm: gate and heads do not fit")
    with _on_device(o.device):
        out = torch.empty_like(o)
        _check(lib.astrai_mix_head_gated_rms_norm(o.data_ptr(), g.data_ptr(), g.stride(0), weight.data_ptr(), out.data_ptr(),
                                                  n, width // vp, vp, count, eps, _dtype(o, "head_gated_rms_norm"),
                                                  _stream(o)), lib)
    return out


def gated_rms_norm(o: torch.Tensor, proj: torch.Tensor, g_off: int, weight: torch.Tensor, count: int,
                   eps: float) -> torch.Tensor:
    """``o / sqrt(mean(o^2) + eps) * weight * sigmoid(g)`` with ``g`` the columns of ``proj`` from ``g_off``;
    ``count`` of the columns are real, the rest padding."""
    lib = _require()
    n, width = o.shape
    code = _dtype(o, "gated_rms_norm")
    _dense("gated_rms_norm", o.dtype, o, proj)
    _dense("gated_rms_norm", torch.float32, weight)
    _shape("gated_rms_norm", weight, width)
    if proj.size(0) != n or g_off < 0 or g_off + width > proj.size(1):
        raise RuntimeError("gated_rms_norm: gate columns outside the projection")
    with _on_device(o.device):
        out = torch.empty_like(o)
        _check(lib.astrai_mix_gated_rms_norm(o.data_ptr(), proj.data_ptr() + g_off * proj.element_size(),
                                             proj.size(1), weight.data_ptr(), out.data_ptr(), n, width, count, eps,
                                             code, _stream(o)), lib)
    return out


# ---------------------------------------------------------------------------
# Latent attention
# ---------------------------------------------------------------------------


@dataclass(frozen=True)
class LatentShape:
    """Padded head sizes of a latent-attention layer: ``dn`` unrotated and ``dr`` rotated query / key
    dimensions, ``rp`` latent columns (``kv_rank`` of them real), ``vp`` value columns."""

    heads: int
    dn: int
    dr: int
    rp: int
    vp: int
    kv_rank: int
    window: int
    scale: float

    @property
    def q_cols(self) -> int:
        return self.heads * (self.dn + self.dr)

    @property
    def cache_cols(self) -> int:
        return self.rp + self.dr


def _latent_block(what: str, s: LatentShape, proj, cache, positions):
    """Checks shared by the latent entries; returns (batch, seq, max_len)."""
    _dense(what, proj.dtype, proj, cache)
    batch, max_len, cols = cache.shape
    if cols != s.cache_cols:
        raise RuntimeError(f"{what}: cache rows of {cols}, expected {s.cache_cols}")
    if proj.dim() != 2 or proj.size(0) % batch or proj.size(0) == 0:
        raise RuntimeError(f"{what}: projection rows {tuple(proj.shape)} do not fit batch {batch}")
    seq = proj.size(0) // batch
    if positions is not None:
        _dense(what, torch.int64, positions)
        _shape(what, positions, seq)
        if positions.device != proj.device:
            raise RuntimeError(f"{what}: positions must be on the input device")
    return batch, seq, max_len


def latent_append(proj: torch.Tensor, s: LatentShape, dkv_off: int, rot: torch.Tensor, positions: torch.Tensor,
                  norm_w: Optional[torch.Tensor], cache: torch.Tensor, eps: float,
                  w_uk_t: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """Rotate the queries of ``proj [batch * seq, ld]`` in place and, with ``dkv_off >= 0``, write the
    normed latents and rotated key parts into ``cache [batch, max_len, rp + dr]`` at ``positions``. With
    ``w_uk_t [heads, rp, dn]`` (bf16) the absorbed queries ``[batch * seq, heads, rp]`` are returned."""
    lib = _require()
    batch, seq, max_len = _latent_block("latent_append", s, proj, cache, positions)
    _dense("latent_append", torch.float32, rot)
    if rot.dim() != 3 or rot.size(2) != 2 or rot.size(0) < max_len:
        raise RuntimeError(f"latent_append: rotary table {tuple(rot.shape)} does not cover {max_len} positions")
    if dkv_off >= 0:
        _dense("latent_append", torch.float32, norm_w)
        _shape("latent_append", norm_w, s.rp)
    q_abs = None
    if w_uk_t is not None:
        _dense("latent_append", torch.bfloat16, proj, w_uk_t)
        _shape("latent_append", w_uk_t, s.heads, s.rp, s.dn)
    with _on_device(proj.device):
        if w_uk_t is not None:
            q_abs = torch.empty((proj.size(0), s.heads, s.rp), device=proj.device, dtype=proj.dtype)
        _check(lib.astrai_mix_latent_append(
            proj.data_ptr(), proj.size(1), dkv_off, rot.data_ptr(), rot.size(0), rot.size(1), positions.data_ptr(),
            norm_w.data_ptr() if dkv_off >= 0 else None, cache.data_ptr(), None if w_uk_t is None else w_uk_t.data_ptr(),
            None if q_abs is None else q_abs.data_ptr(), batch, seq, max_len, s.heads, s.dn, s.dr,
            s.rp, s.kv_rank, eps, _dtype(proj, "latent_append"), _stream(proj)), lib)
    return q_abs


def latent_prefill_supported(s: LatentShape) -> bool:
    """Sizes the matrix-core prompt kernel takes (the limits its entry point checks)."""
    return (s.dn <= 128 and s.dr <= 64 and s.vp <= 128 and 1e-4 <= s.scale <= 1e4
            and 128 * s.heads * (s.dn + s.vp) < 1 << 30)


def latent_prefill(proj: torch.Tensor, s: LatentShape, g_off: int, kv: torch.Tensor, cache: torch.Tensor,
                   start: int, key_base: int) -> torch.Tensor:
    """Windowed attention of the tokens at positions ``start ..`` over per-head keys and values
    ``kv [batch, n_keys, heads * (dn + vp)]`` of the positions from ``key_base``; bf16. Returns
    ``[batch * seq, heads * vp]``."""
    lib = _require()
    batch, seq, max_len = _latent_block("latent_prefill", s, proj, cache, None)
    _dense("latent_prefill", torch.bfloat16, proj, kv)
    if kv.dim() != 3 or kv.size(0) != batch or kv.size(2) != s.heads * (s.dn + s.vp):
        raise RuntimeError(f"latent_prefill: keys and values {tuple(kv.shape)} do not fit")
    with _on_device(proj.device):
        out = torch.empty((batch * seq, s.heads * s.vp), device=proj.device, dtype=proj.dtype)
        _check(lib.astrai_mix_latent_prefill(
            proj.data_ptr(), proj.size(1), g_off, kv.data_ptr(), cache.data_ptr(), out.data_ptr(), batch, seq, max_len,
            start, key_base, kv.size(1), s.heads, s.dn, s.dr, s.rp, s.vp, s.window, s.scale, _stream(proj)), lib)
    return out


def latent_rows_supported(s: LatentShape, max_len: int) -> bool:
    """Sizes the matrix-core kernels of :func:`latent_rows` take (the limits its entry point checks)."""
    return s.rp <= 1024 and s.dr <= 64 and max_len * s.cache_cols * 2 < 0x7fffffff


def latent_rows_nsplit(s: LatentShape, batch: int, seq: int, max_len: int) -> int:
    """How many workgroups share a context: enough for two per CU, each with four 32-key tiles or
    more of the longest key range the rows can have."""
    groups = batch * -(-seq * s.heads // 16)
    tiles = -(-min(s.window + seq, max_len) // 32)
    return max(1, min(-(-512 // groups), tiles // 4, MAX_SPLIT))


def latent_rows(proj: torch.Tensor, s: LatentShape, g_off: int, w_ukv: torch.Tensor, cache: torch.Tensor,
                positions: torch.Tensor, q_abs: Optional[torch.Tensor] = None, nsplit: int = 0) -> torch.Tensor:
    """The same attention computed in the latent space, for a few new tokens (positions on the
    device). ``w_ukv [heads * (dn + vp), rp]``. With the absorbed queries ``q_abs`` of
    :func:`latent_append` (overwritten here) on the matrix cores, ``nsplit`` 0 picking a split count;
    without them on the general kernel, bf16 or float."""
    lib = _require()
    batch, seq, max_len = _latent_block("latent_rows", s, proj, cache, positions)
    _dense("latent_rows", proj.dtype, proj, w_ukv)
    _shape("latent_rows", w_ukv, s.heads * (s.dn + s.vp), s.rp)
    n, dev = proj.size(0), proj.device
    with _on_device(dev):
        out = torch.empty((n, s.heads * s.vp), device=dev, dtype=proj.dtype)
        if q_abs is not None:
            _dense("latent_rows", torch.bfloat16, proj, q_abs)
            _shape("latent_rows", q_abs, n, s.heads, s.rp)
            nsplit = nsplit or latent_rows_nsplit(s, batch, seq, max_len)
            ws = torch.empty(lib.astrai_mix_latent_rows_workspace_floats(n, s.heads, s.rp, nsplit), device=dev,
                             dtype=torch.float32)
            _check(lib.astrai_mix_latent_rows(
                proj.data_ptr(), proj.size(1), g_off, w_ukv.data_ptr(), cache.data_ptr(), positions.data_ptr(),
                q_abs.data_ptr(), ws.data_ptr(), out.data_ptr(), batch, seq, max_len, s.heads, s.dn, s.dr, s.rp, s.vp,
                s.window, s.scale, nsplit, _stream(proj)), lib)
        else:
            _check(lib.astrai_mix_latent_rows_general(
                proj.data_ptr(), proj.size(1), g_off, w_ukv.data_ptr(), cache.data_ptr(), positions.data_ptr(),
                out.data_ptr(), batch, seq, max_len, s.heads, s.dn, s.dr, s.rp, s.vp, s.window, s.scale,
                _dtype(proj, "latent_rows"), _stream(proj)), lib)
    return out


# ---------------------------------------------------------------------------
# Lightning attention
# ---------------------------------------------------------------------------


def decay_powers(decay) -> torch.Tensor:
    """``[heads, LIGHTNING_CHUNK + 1]`` fp32: ``decay_h ** n``, formed in fp64."""
    d = torch.tensor(list(decay), dtype=torch.float64)
    return (d[:, None] ** torch.arange(LIGHTNING_CHUNK + 1, dtype=torch.float64)[None, :]).float()


def lightning_chunk_supported(dp: int) -> bool:
    return dp <= 256


def lightning_nseg(batch: int, heads: int, vp: int, seq: int) -> int:
    """Segments of a sequence that run side by side: enough workgroups for two per CU, no segment
    shorter than four chunks."""
    groups = batch * heads * -(-vp // 64)
    chunks = -(-seq // LIGHTNING_CHUNK)
    return max(1, min(-(-512 // groups), chunks // 4))


def lightning(proj: torch.Tensor, q_off: int, k_off: int, v_off: int, decay_pow: torch.Tensor, state: torch.Tensor,
              step: bool, nseg: Optional[int] = None) -> torch.Tensor:
    """``S <- decay S + k v^T``, ``o = S^T q`` on silu of the projected columns of ``proj [batch * seq, ld]``;
    ``state [batch, heads, dp, vp]`` fp32 is read and written. ``step``: the token-by-token kernel,
    else the chunked one (bf16). Returns ``[batch * seq, heads * vp]``."""
    lib = _require()
    batch, heads, dp, vp = state.shape
    _dense("lightning", proj.dtype, proj)
    _dense("lightning", torch.float32, decay_pow, state)
    _shape("lightning", decay_pow, heads, LIGHTNING_CHUNK + 1)
    n, ld, dev = proj.size(0), proj.size(1), proj.device
    if state.device != dev or n % batch or n == 0:
        raise RuntimeError("lightning: projection rows and state do not fit")
    seq = n // batch
    with _on_device(dev):
        out = torch.empty((n, heads * vp), device=dev, dtype=proj.dtype)
        if step:
            _check(lib.astrai_mix_lightning_step(proj.data_ptr(), ld, q_off, k_off, v_off, decay_pow.data_ptr(),
                                                 state.data_ptr(), out.data_ptr(), batch, seq, heads, dp, vp,
                                                 _dtype(proj, "lightning"), _stream(proj)), lib)
        else:
            _dense("lightning", torch.bfloat16, proj)
            if nseg is None:
                nseg = lightning_nseg(batch, heads, vp, seq)
            seg = torch.empty((batch, heads, nseg, dp, vp), device=dev, dtype=torch.float32) if nseg > 1 else None
            _check(lib.astrai_mix_lightning_chunk(proj.data_ptr(), ld, q_off, k_off, v_off, decay_pow.data_ptr(),
                                                  state.data_ptr(), None if seg is None else seg.data_ptr(),
                                                  out.data_ptr(), batch, seq, heads, dp, vp, nseg, _stream(proj)), lib)
    return out


# ---------------------------------------------------------------------------
# Grouped-query attention
# ---------------------------------------------------------------------------


@dataclass(frozen=True)
class GqaShape:
    """Padded head sizes (``dk``, ``vp``; ``dim`` key columns are real) and the constants of a layer's attention:
    ``softcap`` 0 means none, ``sink`` one more term exp(0) in the softmax denominator."""

    heads: int
    kv_heads: int
    dk: int
    vp: int
    dim: int
    scale: float
    softcap: float = 0.0
    sink: bool = False
    window: int = UNBOUNDED

    @property
    def cache_cols(self) -> int:
        return self.kv_heads * (self.dk + self.vp)


def _gqa_block(what: str, s: GqaShape, proj, cache, positions):
    _dense(what, proj.dtype, proj, cache)
    batch, max_len, cols = cache.shape
    if cols != s.cache_cols:
        raise RuntimeError(f"{what}: cache rows of {cols}, expected {s.cache_cols}")
    return batch, _rows_of_batch(what, proj, batch, positions), max_len


def _rows_of_batch(what: str, proj: torch.Tensor, batch: int, positions: Optional[torch.Tensor]) -> int:
    """Tokens per sequence of a projection's rows, checked against the positions."""
    if proj.dim() != 2 or proj.size(0) % batch or proj.size(0) == 0:
        raise RuntimeError(f"{what}: projection rows {tuple(proj.shape)} do not fit batch {batch}")
    seq = proj.size(0) // batch
    if positions is not None:
        _dense(what, torch.int64, positions)
        _shape(what, positions, seq)
        if positions.device != proj.device:
            raise RuntimeError(f"{what}: positions must be on the input device")
    return seq


def gqa_append(proj: torch.Tensor, s: GqaShape, k_off: int, v_off: int, rot: Optional[torch.Tensor],
               positions: torch.Tensor, q_norm: Optional[torch.Tensor], k_norm: Optional[torch.Tensor],
               cache: torch.Tensor, eps: float) -> None:
    """Norm and rotate the queries of ``proj [batch * seq, ld]`` in place (columns from 0), and the keys into ``cache
    [batch, max_len, kv_heads * (dk + vp)]`` at ``positions``, next to their values. ``rot`` None: no rotation;
    norm weights None: no norm."""
    lib = _require()
    batch, seq, max_len = _gqa_block("gqa_append", s, proj, cache, positions)
    half = 0
    if rot is not None:
        _dense("gqa_append", torch.float32, rot)
        if rot.dim() != 3 or rot.size(2) != 2 or rot.size(0) < max_len:
            raise RuntimeError(f"gqa_append: rotary table {tuple(rot.shape)} does not cover {max_len} positions")
        half = rot.size(1)
    for w in (q_norm, k_norm):
        if w is not None:
            _dense("gqa_append", torch.float32, w)
            _shape("gqa_append", w, s.dk)
    with _on_device(proj.device):
        _check(lib.astrai_mix_gqa_append(
            proj.data_ptr(), proj.size(1), k_off, v_off, None if rot is None else rot.data_ptr(),
            0 if rot is None else rot.size(0), half, positions.data_ptr(), None if q_norm is None else q_norm.data_ptr(),
            None if k_norm is None else k_norm.data_ptr(), cache.data_ptr(), batch, seq, max_len, s.heads, s.kv_heads,
            s.dk, s.vp, s.dim, eps, _dtype(proj, "gqa_append"), _stream(proj)), lib)


def gqa_prefill_supported(s: GqaShape) -> bool:
    """Sizes the matrix-core prompt kernel takes (the limits its entry point checks)."""
    return s.dk <= 128 and s.vp <= 128 and 1e-4 <= s.scale <= 1e4 and 128 * s.heads * (s.dk + s.vp) < 1 << 30


def gqa_prefill(proj: torch.Tensor, s: GqaShape, g_off: int, cache: torch.Tensor, start: int) -> torch.Tensor:
    """Attention of the tokens at positions ``start ..`` (appended to the cache already), bf16; ``g_off`` the gate
    columns or -1. Returns ``[batch * seq, heads * vp]``."""
    lib = _require()
    batch, seq, max_len = _gqa_block("gqa_prefill", s, proj, cache, None)
    _dense("gqa_prefill", torch.bfloat16, proj)
    with _on_device(proj.device):
        out = torch.empty((batch * seq, s.heads * s.vp), device=proj.device, dtype=proj.dtype)
        _check(lib.astrai_mix_gqa_prefill(
            proj.data_ptr(), proj.size(1), g_off, cache.data_ptr(), out.data_ptr(), batch, seq, max_len, start, s.heads,
            s.kv_heads, s.dk, s.vp, s.window, s.scale, s.softcap, int(s.sink), _stream(proj)), lib)
    return out


def gqa_rows_supported(s: GqaShape, max_len: int) -> bool:
    """Sizes the matrix-core form of :func:`gqa_rows` takes (the limits its entry point checks)."""
    return s.dk <= 256 and s.vp <= 128 and (max_len + 64) * s.cache_cols * 2 < 0x7fffffff


def gqa_rows_nsplit(s: GqaShape, batch: int, seq: int, max_len: int) -> int:
    """How many workgroups share a context: enough for two per CU, each with two rounds of four 32-key
    tiles or more of the longest key range the rows can have."""
    groups = batch * s.kv_heads * -(-seq * (s.heads // s.kv_heads) // 16)
    tiles = -(-min(s.window + seq, max_len) // 32)
    return max(1, min(-(-512 // groups), tiles // 8, MAX_SPLIT))


def gqa_rows(proj: torch.Tensor, s: GqaShape, g_off: int, cache: torch.Tensor, positions: torch.Tensor,
             matrix: bool, nsplit: int = 0) -> torch.Tensor:
    """The same for a few new tokens (positions on the device): ``matrix``: on the matrix cores (bf16), ``nsplit`` 0
    picking a split count; else the general kernel, bf16 or float, any number of tokens."""
    lib = _require()
    batch, seq, max_len = _gqa_block("gqa_rows", s, proj, cache, positions)
    n, dev = proj.size(0), proj.device
    with _on_device(dev):
        out = torch.empty((n, s.heads * s.vp), device=dev, dtype=proj.dtype)
        if matrix:
            _dense("gqa_rows", torch.bfloat16, proj)
            nsplit = nsplit or gqa_rows_nsplit(s, batch, seq, max_len)
            ws = torch.empty(lib.astrai_mix_gqa_rows_workspace_floats(n, s.heads, s.vp, nsplit), device=dev,
                             dtype=torch.float32)
            _check(lib.astrai_mix_gqa_rows(
                proj.data_ptr(), proj.size(1), g_off, cache.data_ptr(), positions.data_ptr(), ws.data_ptr(),
                out.data_ptr(), batch, seq, max_len, s.heads, s.kv_heads, s.dk, s.vp, s.window, s.scale, s.softcap,
                int(s.sink), nsplit, _stream(proj)), lib)
        else:
            _check(lib.astrai_mix_gqa_rows_general(
                proj.data_ptr(), proj.size(1), g_off, cache.data_ptr(), positions.data_ptr(), out.data_ptr(), batch, seq,
                max_len, s.heads, s.kv_heads, s.dk, s.vp, s.window, s.scale, s.softcap, int(s.sink),
                _dtype(proj, "gqa_rows"), _stream(proj)), lib)
    return out


# ---------------------------------------------------------------------------
# Short convolution with a ring of earlier inputs
# ---------------------------------------------------------------------------


def ring_rows(taps: int) -> int:
    return taps - 1 + RING_STEPS


def _conv_checks(what: str, proj, off, w, bias, ring, positions):
    taps, cols = w.shape
    _dense(what, proj.dtype, proj, ring)
    _dense(what, torch.float32, w)
    if bias is not None:
        _dense(what, torch.float32, bias)
        _shape(what, bias, cols)
    if ring.dim() != 3 or tuple(ring.shape[1:]) != (ring_rows(taps), cols):
        raise RuntimeError(f"{what}: ring {tuple(ring.shape)}, expected [batch, {ring_rows(taps)}, {cols}]")
    if off < 0 or off + cols > proj.size(1) or w.device != proj.device:
        raise RuntimeError(f"{what}: columns {off} .. + {cols} of {proj.size(1)}")
    return ring.size(0), _rows_of_batch(what, proj, ring.size(0), positions), taps, cols


def conv(proj: torch.Tensor, off: int, w: torch.Tensor, bias: Optional[torch.Tensor], ring: torch.Tensor,
         positions: torch.Tensor, silu: bool) -> torch.Tensor:
    """Causal convolution per channel of the columns of ``proj [batch * seq, ld]`` from ``off``: ``w [taps, cols]``, the
    last row on the current token; ``ring [batch, ring_rows(taps), cols]`` holds earlier inputs (the one of position p
    in row p mod rows) and takes this block's last ``taps - 1``. Returns ``[batch * seq, cols]``."""
    lib = _require()
    batch, seq, taps, cols = _conv_checks("conv", proj, off, w, bias, ring, positions)
    with _on_device(proj.device):
        out = torch.empty((proj.size(0), cols), device=proj.device, dtype=proj.dtype)
        _check(lib.astrai_mix_conv(proj.data_ptr(), proj.size(1), off, cols, w.data_ptr(),
                                   None if bias is None else bias.data_ptr(), taps, ring.data_ptr(), positions.data_ptr(),
                                   out.data_ptr(), batch, seq, int(silu), 1, _dtype(proj, "conv"), _stream(proj)), lib)
    return out


# ---------------------------------------------------------------------------
# Real-gated linear recurrent unit
# ---------------------------------------------------------------------------


def rglru_chunk_supported(bp: int) -> bool:
    return bp <= 1024


def rglru_nseg(batch: int, blocks: int, bp: int, seq: int) -> int:
    """Segments of a sequence that run side by side: enough workgroups for one per CU, no segment shorter
    than two tiles."""
    groups = batch * blocks * -(-bp // 64)
    tiles = -(-seq // 64)
    return max(1, min(-(-256 // groups), tiles // 2))


def _rglru_checks(what: str, proj, y_off, w_r, w_i, b_r, b_i, coef, state, *rows):
    blocks, bp = w_r.size(0), w_r.size(1)
    cols = blocks * bp
    _dense(what, proj.dtype, proj, w_r, w_i, *rows)
    _dense(what, torch.float32, b_r, b_i, coef, state)
    for w in (w_r, w_i):
        _shape(what, w, blocks, bp, bp)
    for v in (b_r, b_i, coef):
        _shape(what, v, cols)
    if state.dim() != 2 or state.size(1) != cols or proj.size(0) % state.size(0) or state.device != proj.device or \
            y_off < 0 or y_off + cols > proj.size(1):
        raise RuntimeError(f"{what}: state {tuple(state.shape)} or columns do not fit")
    for t in rows:
        _shape(what, t, proj.size(0), cols)
    return state.size(0), proj.size(0) // state.size(0), blocks, bp


def rglru(u: torch.Tensor, proj: torch.Tensor, y_off: int, w_r: torch.Tensor, w_i: torch.Tensor, b_r: torch.Tensor,
          b_i: torch.Tensor, coef: torch.Tensor, state: torch.Tensor, matrix: bool,
          nseg: Optional[int] = None) -> torch.Tensor:
    """``r, i = sigmoid(W u + b)`` per block of channels, ``a = exp(coef r)``, ``S <- a S + sqrt(1 - a^2) i u``; returns
    ``S gelu(y)``, ``[batch * seq, blocks * bp]``. ``state [batch, blocks * bp]`` fp32 is read and written. ``matrix``:
    the chunked kernel (bf16), ``w_r, w_i [blocks, out, in]``; else the general one, weights ``[blocks, in, out]``."""
    lib = _require()
    batch, seq, blocks, bp = _rglru_checks("rglru", proj, y_off, w_r, w_i, b_r, b_i, coef, state, u)
    dev = proj.device
    with _on_device(dev):
        out = torch.empty_like(u)
        args = [u.data_ptr(), proj.data_ptr(), proj.size(1), y_off, w_r.data_ptr(), w_i.data_ptr(), b_r.data_ptr(),
                b_i.data_ptr(), coef.data_ptr(), state.data_ptr()]
        if matrix:
            _dense("rglru", torch.bfloat16, proj)
            if nseg is None:
                nseg = rglru_nseg(batch, blocks, bp, seq)
            scratch = torch.empty((batch, nseg, 2, blocks * bp), device=dev, dtype=torch.float32) if nseg > 1 else None
            _check(lib.astrai_mix_rglru_chunk(*args, None if scratch is None else scratch.data_ptr(), out.data_ptr(),
                                              batch, seq, blocks, bp, nseg, _stream(proj)), lib)
        else:
            scratch = torch.empty((2, batch * seq, blocks * bp), device=dev, dtype=torch.float32)
            _check(lib.astrai_mix_rglru_general(*args, scratch.data_ptr(), out.data_ptr(), batch, seq, blocks, bp,
                                                _dtype(proj, "rglru"), _stream(proj)), lib)
    return out


def rglru_step(proj: torch.Tensor, y_off: int, x_off: int, conv_w: torch.Tensor, conv_b: Optional[torch.Tensor],
               ring: torch.Tensor, positions: torch.Tensor, w_r: torch.Tensor, w_i: torch.Tensor, b_r: torch.Tensor,
               b_i: torch.Tensor, coef: torch.Tensor, state: torch.Tensor) -> torch.Tensor:
    """:func:`conv` of the columns from ``x_off`` and :func:`rglru` of the result in one launch, for at most
    ``RING_STEPS`` tokens; bf16, ``w_r, w_i [blocks, out, in]``."""
    lib = _require()
    _dense("rglru_step", torch.bfloat16, proj)
    batch, seq, blocks, bp = _rglru_checks("rglru_step", proj, y_off, w_r, w_i, b_r, b_i, coef, state)
    cb, cs, taps, cols = _conv_checks("rglru_step", proj, x_off, conv_w, conv_b, ring, positions)
    if (cb, cs, cols) != (batch, seq, blocks * bp):
        raise RuntimeError("rglru_step: convolution and state do not fit")
    with _on_device(proj.device):
        out = torch.empty((proj.size(0), cols), device=proj.device, dtype=proj.dtype)
        _check(lib.astrai_mix_rglru_step(
            proj.data_ptr(), proj.size(1), y_off, x_off, conv_w.data_ptr(), None if conv_b is None else conv_b.data_ptr(),
            taps, ring.data_ptr(), positions.data_ptr(), w_r.data_ptr(), w_i.data_ptr(), b_r.data_ptr(), b_i.data_ptr(),
            coef.data_ptr(), state.data_ptr(), out.data_ptr(), batch, seq, blocks, bp, _stream(proj)), lib)
    return out


# ---------------------------------------------------------------------------
# Gated delta rule with a decay per key channel
# ---------------------------------------------------------------------------


@dataclass(frozen=True)
class DeltaShape:
    """Padded head sizes (``dp`` key, ``vp`` value; ``vdim`` value columns are real); queries are unit vectors times
    ``q_scale``."""

    heads: int
    kv_heads: int
    dp: int
    vp: int
    vdim: int
    q_scale: float

    @property
    def qkv_cols(self) -> int:
        return 2 * self.kv_heads * self.dp + self.heads * self.vp


def delta_step_supported(s: DeltaShape) -> bool:
    lanes = 8
    while lanes * 4 < s.vp:
        lanes *= 2
    return s.vp <= 256 and s.dp <= 1024 and s.dp * lanes <= 16384


def delta_chunk_supported(s: DeltaShape) -> bool:
    return s.dp <= 256


def _delta_checks(what: str, s: DeltaShape, proj, b_off, z, dt_bias, decay, state):
    n = proj.size(0)
    _dense(what, proj.dtype, proj)
    _dense(what, torch.float32, z, dt_bias, decay, state)
    _shape(what, z, n, s.heads * s.dp)
    _shape(what, dt_bias, s.heads * s.dp)
    _shape(what, decay, s.heads)
    if state.dim() != 4 or tuple(state.shape[1:]) != (s.heads, s.dp, s.vp) or n % state.size(0) or n == 0 or \
            state.device != proj.device or b_off < 0 or b_off + s.heads > proj.size(1):
        raise RuntimeError(f"{what}: state {tuple(state.shape)} or columns do not fit")
    return state.size(0), n // state.size(0)


def delta_step(proj: torch.Tensor, s: DeltaShape, b_off: int, z: torch.Tensor, dt_bias: torch.Tensor,
               decay: torch.Tensor, gate: torch.Tensor, norm_w: torch.Tensor, state: torch.Tensor, eps: float,
               qkv: Optional[torch.Tensor] = None, x_off: int = 0, conv_w: Optional[torch.Tensor] = None,
               ring: Optional[torch.Tensor] = None, positions: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Token by token: ``S <- diag(g) S``, ``u = beta (v - S^T k)``, ``S <- S + k u^T``, ``o = S^T q``; returns the RMS norm
    of each head's ``o`` times ``norm_w`` times ``sigmoid(gate)``, ``[batch * seq, heads * vp]``. ``qkv``: the convolved
    q | k | v; without it they are convolved here (as :func:`conv` with silu) from the columns at ``x_off``, for at most
    ``RING_STEPS`` tokens. ``z [batch * seq, heads * dp]`` fp32, ``g = exp(-decay softplus(z + dt_bias))``; ``state``
    fp32 ``[batch, heads, dp, vp]``; the step size is the sigmoid of column ``b_off + head``."""
    lib = _require()
    batch, seq = _delta_checks("delta_step", s, proj, b_off, z, dt_bias, decay, state)
    _dense("delta_step", torch.float32, norm_w)
    _shape("delta_step", norm_w, s.vp)
    if gate.dtype != proj.dtype or gate.device != proj.device or gate.stride(1) != 1 or \
            tuple(gate.shape) != (proj.size(0), s.heads * s.vp):
        raise RuntimeError("delta_step: gate does not fit")
    taps = 1
    if qkv is not None:
        _dense("delta_step", proj.dtype, proj, qkv)
        _shape("delta_step", qkv, proj.size(0), s.qkv_cols)
    else:
        cb, cs, taps, cols = _conv_checks("delta_step", proj, x_off, conv_w, None, ring, positions)
        if (cb, cs, cols) != (batch, seq, s.qkv_cols):
            raise RuntimeError("delta_step: convolution and state do not fit")

    def ptr(t):
        return None if t is None else t.data_ptr()

    with _on_device(proj.device):
        out = torch.empty((proj.size(0), s.heads * s.vp), device=proj.device, dtype=proj.dtype)
        _check(lib.astrai_mix_delta_step(
            ptr(qkv), proj.data_ptr(), proj.size(1), x_off, b_off, ptr(conv_w), taps, ptr(ring), ptr(positions), z.data_ptr(),
            dt_bias.data_ptr(), decay.data_ptr(), gate.data_ptr(), gate.stride(0), norm_w.data_ptr(), state.data_ptr(),
            out.data_ptr(), batch, seq, s.heads, s.kv_heads, s.dp, s.vp, s.vdim, s.q_scale, eps,
            _dtype(proj, "delta_step"), _stream(proj)), lib)
    return out


def delta_chunk(qkv: torch.Tensor, proj: torch.Tensor, s: DeltaShape, b_off: int, z: torch.Tensor,
                dt_bias: torch.Tensor, decay: torch.Tensor, state: torch.Tensor) -> torch.Tensor:
    """The same recurrence in chunks on the matrix cores (bf16); returns ``o``, neither normed nor gated."""
    lib = _require()
    batch, seq = _delta_checks("delta_chunk", s, proj, b_off, z, dt_bias, decay, state)
    _dense("delta_chunk", torch.bfloat16, proj, qkv)
    _shape("delta_chunk", qkv, proj.size(0), s.qkv_cols)
    with _on_device(proj.device):
        out = torch.empty((proj.size(0), s.heads * s.vp), device=proj.device, dtype=proj.dtype)
        size = lib.astrai_mix_delta_image_bytes(s.dp) * batch * s.heads * -(-seq // DELTA_CHUNK)
        image = torch.empty(size, device=proj.device, dtype=torch.uint8)
        _check(lib.astrai_mix_delta_chunk(
            qkv.data_ptr(), proj.data_ptr(), proj.size(1), b_off, z.data_ptr(), dt_bias.data_ptr(), decay.data_ptr(),
            state.data_ptr(), image.data_ptr(), out.data_ptr(), batch, seq, s.heads, s.kv_heads, s.dp, s.vp, s.q_scale,
            _stream(proj)), lib)
    return out
