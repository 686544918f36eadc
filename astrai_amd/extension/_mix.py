"""ctypes binding of ``lib/libastrai_mix.so`` (the C ABI in include/astrai_mix.h): latent and
lightning attention and the row operations of decoders with an fp32 residual stream, as
functions on tensors. As in ``_cabi``: shapes and devices are checked here, outputs and scratch
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

ABI_VERSION = 1
LIGHTNING_CHUNK = 64
MAX_SPLIT = 64
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
    "astrai_mix_silu_mul": ([_P, _P, _I64, _I64, _INT, _P], _INT),
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


def silu_mul(gu: torch.Tensor) -> torch.Tensor:
    """``silu(gate) * up`` of ``gu [n, 2 ff]`` (gate columns, then up)."""
    lib = _require()
    code = _dtype(gu, "silu_mul")
    _dense("silu_mul", gu.dtype, gu)
    n, ff = gu.size(0), gu.size(1) // 2
    with _on_device(gu.device):
        h = torch.empty((n, ff), device=gu.device, dtype=gu.dtype)
        _check(lib.astrai_mix_silu_mul(gu.data_ptr(), h.data_ptr(), n, ff, code, _stream(gu)), lib)
    return h


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
