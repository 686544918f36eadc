"""Plain CPU restatement of the Lugitar decoder: latent attention with a sliding window
and shared latents, lightning (decayed linear) attention, sandwich layer norms.
TEST INFRASTRUCTURE ONLY (see oracle/__init__.py): one function per mechanism, no cache,
no batch, no shared code with the product.

Every function takes the tokens of ONE sequence as rows ``[tokens, width]`` and the whole
sequence at once, in the dtype of its inputs (float64 for the checks). Weights are a plain
``name -> tensor`` dict, the configuration the plain dict of config.json.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1 + torch.exp(-z))


def layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """Layer norm with a weight and no bias: centred, divided by the root of the mean squared
    deviation plus eps, times ``w``."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotary_frequencies(dims: int, base: float, scaling: Optional[dict]) -> List[float]:
    """Angle per position of each of the ``dims / 2`` pairs: ``base^(-2i/dims)``, under YaRN
    scaling blended with its ``1/factor`` along a ramp between the two pair indices that turn
    ``fast`` and ``slow`` times over the original context."""
    freqs = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return freqs

    def pair_of(turns):
        return dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(pair_of(scaling["fast"])), 0)
    hi = min(math.ceil(pair_of(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / scaling["factor"] * ramp + f * (1.0 - ramp))
    return out


def rotary_magnitude(scaling: Optional[dict]) -> float:
    """What cos and sin are multiplied by (YaRN's attention temperature)."""
    return 1.0 if scaling is None else 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_half(x: torch.Tensor, positions: torch.Tensor, rot: dict) -> torch.Tensor:
    """Rotate the first ``rot.dims`` entries of the last axis of ``x [tokens, ..., d]``: entry i
    and entry i + dims/2 form a pair."""
    dims, scaling = rot["dims"], rot.get("scaling")
    f = torch.tensor(rotary_frequencies(dims, rot["base"], scaling), dtype=torch.float64)
    ang = positions.double()[:, None] * f[None, :]
    mag = rotary_magnitude(scaling)
    shape = (x.size(0),) + (1,) * (x.dim() - 2) + (dims // 2,)
    cos, sin = (torch.cos(ang) * mag).reshape(shape), (torch.sin(ang) * mag).reshape(shape)
    cos, sin = cos.to(x.dtype), sin.to(x.dtype)
    u, v, rest = x[..., : dims // 2], x[..., dims // 2: dims], x[..., dims:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


def window_mask(n: int, size: Optional[int]) -> torch.Tensor:
    """``[n, n]`` bool: query i sees key j iff ``0 <= i - j < size`` (no upper limit for None)."""
    d = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    seen = d >= 0
    return seen if size is None else seen & (d < size)


def latent_of(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mix: dict, eps: float):
    """What a latent-attention layer keeps of each token: the normed latent ``c [n, kv_rank]`` and
    the rotated key part ``[n, rot_dim]`` that all heads share."""
    r = mix["kv_rank"]
    y = h @ w[p + "dkv"].T
    c = rms_norm(y[:, :r], w[p + "dkv.norm"], eps)
    return c, rotate_half(y[:, r:], torch.arange(h.size(0)), mix["rot"])


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mix: dict, latent) -> torch.Tensor:
    """Softmax attention whose per-head keys and values are projections of the latent."""
    n, heads, dim, rd, vd = h.size(0), mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"]
    c, kr = latent
    q = (h @ w[p + "q"].T).reshape(n, heads, dim + rd)
    qn, qr = q[..., :dim], rotate_half(q[..., dim:], torch.arange(n), mix["rot"])
    k = (c @ w[p + "uk"].T).reshape(n, heads, dim)
    v = (c @ w[p + "uv"].T).reshape(n, heads, vd)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    seen = window_mask(n, (mix.get("mask") or {}).get("size"))
    out = torch.empty(n, heads, vd, dtype=h.dtype)
    for a in range(heads):
        s = (qn[:, a] @ k[:, a].T + qr[:, a] @ kr.T) * mix["scale"]
        s = s.masked_fill(~seen, float("-inf"))
        out[:, a] = torch.softmax(s, dim=-1) @ v[:, a] * gate[:, a, None]
    return out.reshape(n, heads * vd) @ w[p + "o"].T


def lightning_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay, state=None):
    """Token by token per head: ``S <- decay_h S + k v^T``, ``o = S^T q``. ``q, k [n, heads, dim]``,
    ``v [n, heads, vdim]``; returns the outputs and the last state ``[heads, dim, vdim]``."""
    n, heads, dim = q.shape
    s = torch.zeros(heads, dim, v.size(-1), dtype=q.dtype) if state is None else state.clone()
    lam = torch.tensor(decay, dtype=torch.float64).to(q.dtype).reshape(heads, 1, 1)
    out = torch.empty(n, heads, v.size(-1), dtype=q.dtype)
    for t in range(n):
        s = lam * s + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (s * q[t][:, :, None]).sum(1)
    return out, s


def lightning(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mix: dict, eps: float) -> torch.Tensor:
    n, heads, dim, vd = h.size(0), mix["heads"], mix["dim"], mix["vdim"]
    q = silu(h @ w[p + "q"].T).reshape(n, heads, dim)
    k = silu(h @ w[p + "k"].T).reshape(n, heads, dim)
    v = silu(h @ w[p + "v"].T).reshape(n, heads, vd)
    o, _ = lightning_scan(q, k, v, mix["decay"])
    o = rms_norm(o.reshape(n, heads * vd), w[p + "norm"], eps)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def dense_mlp(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens, dtype=torch.float64,
            layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[tokens, vocab]`` of one sequence; the residual after every layer is appended to
    ``layers_out`` if given."""
    w = {k: t.to(dtype) for k, t in weights.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    latents: Dict[int, tuple] = {}
    for i, layer in enumerate(cfg["layers"]):
        p, mix = f"l{i}.", layer["mixer"]
        h = layer_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "latent_attention":
            j = mix.get("kv_from")
            latents[i] = latent_of(h, w, p + "mix.", mix, eps) if j is None else latents[j]
            y = latent_attention(h, w, p + "mix.", mix, latents[i])
        elif layer["type"] == "lightning":
            y = lightning(h, w, p + "mix.", mix, eps)
        else:
            raise ValueError(layer["type"])
        x = x + m * layer_norm(y, w[p + "norm1b"], eps)
        if layer["mlp"] is not None:
            y = dense_mlp(layer_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
            x = x + m * layer_norm(y, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T
