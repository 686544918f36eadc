"""Plain CPU restatement of the Sarulix decoder: softmax attention with normed queries and keys,
soft-capped scores, a sink and an output gate; a real-gated linear recurrent unit behind a short
convolution; a gated delta rule with one decay per key channel; layers that run several times.
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


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1 / (1 + torch.exp(-z))


def softplus(z: torch.Tensor) -> torch.Tensor:
    """log(1 + e^z), the larger part taken out of the logarithm."""
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-torch.abs(z)))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return z / 2 * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z * z * z)))


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def rotate_half(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """Rotate the first ``dims`` entries of the last axis of ``x [tokens, heads, d]``: entry i and
    entry i + dims/2 form a pair that turns by ``position * base^(-2i/dims)``."""
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    ang = (positions.double()[:, None] * f[None, :])[:, None, :]
    cos, sin = torch.cos(ang).to(x.dtype), torch.sin(ang).to(x.dtype)
    u, v, rest = x[..., : dims // 2], x[..., dims // 2: dims], x[..., dims:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


def softmax_with_sink(s: torch.Tensor) -> torch.Tensor:
    """exp(s_j) / (1 + sum exp(s_j)) over the last axis; -inf hides a key."""
    m = torch.clamp(s.amax(-1, keepdim=True), min=0)   # (the sink's score is 0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attention_core(q, k, v, scale: float, softcap: float) -> torch.Tensor:
    """``q [n, H, d]``, ``k [n, G, d]``, ``v [n, G, vd]`` -> ``[n, H, vd]``, causal."""
    n, heads, _ = q.shape
    rep = heads // k.size(1)
    hidden = torch.arange(n)[None, :] > torch.arange(n)[:, None]
    out = torch.empty(n, heads, v.size(-1), dtype=q.dtype)
    for h in range(heads):
        s = q[:, h] @ k[:, h // rep].T * scale
        s = softcap * torch.tanh(s / softcap)
        out[:, h] = softmax_with_sink(s.masked_fill(hidden, float("-inf"))) @ v[:, h // rep]
    return out


def attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mix: dict, eps: float) -> torch.Tensor:
    n, heads, groups, dim, vdim = h.size(0), mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"]
    pos, rot = torch.arange(n), mix["rot"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(n, heads, dim)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(n, groups, dim)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(n, groups, vdim)
    q = rotate_half(rms(q, eps) * w[p + "q.norm"], pos, rot["dims"], rot["base"])
    k = rotate_half(rms(k, eps) * w[p + "k.norm"], pos, rot["dims"], rot["base"])
    o = attention_core(q, k, v, mix["scale"], mix["softcap"]).reshape(n, heads * vdim)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T + w[p + "o.b"]


def short_conv(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """Causal convolution per channel: ``x [n, c]``, ``taps [c, t]``, the last tap on the current token."""
    n, t = x.size(0), taps.size(1)
    out = torch.zeros_like(x)
    for j in range(t):
        back = t - 1 - j
        if back < n:
            out[back:] += x[:n - back] * taps[:, j]
    return out


def linear_unit_scan(u: torch.Tensor, r: torch.Tensor, i: torch.Tensor, lam: torch.Tensor, state=None):
    """``S <- a S + sqrt(1 - a^2) i u`` per channel with ``a = exp(-8 r softplus(lam))``; all
    ``[n, c]``. Returns every token's state and the last one."""
    s = torch.zeros_like(u[0]) if state is None else state.clone()
    out = torch.empty_like(u)
    sp = softplus(lam)
    for t in range(u.size(0)):
        log_a = -8 * r[t] * sp
        s = torch.exp(log_a) * s + torch.sqrt(-torch.expm1(2 * log_a)) * i[t] * u[t]
        out[t] = s
    return out, s


def rglru(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mix: dict) -> torch.Tensor:
    n, width, blocks = h.size(0), mix["width"], mix["blocks"]
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = short_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"]) + w[p + "conv.b"]
    part = u.reshape(n, blocks, width // blocks)
    r, i = torch.empty_like(part), torch.empty_like(part)
    for b in range(blocks):
        r[:, b] = sigmoid(part[:, b] @ w[p + "ra"][b].T + w[p + "ra.b"][b])
        i[:, b] = sigmoid(part[:, b] @ w[p + "ri"][b].T + w[p + "ri.b"][b])
    s, _ = linear_unit_scan(u, r.reshape(n, width), i.reshape(n, width), w[p + "lam"])
    return (s * y) @ w[p + "o"].T


def delta_scan(q, k, v, g, beta, state=None):
    """Token by token per head: ``S <- diag(g) S``, ``u = beta (v - S^T k)``, ``S <- S + k u^T``,
    ``o = S^T q``. ``q, k, g [n, heads, dim]``, ``v [n, heads, vdim]``, ``beta [n, heads]``; returns
    the outputs and the last state ``[heads, dim, vdim]``."""
    n, heads, dim = q.shape
    s = torch.zeros(heads, dim, v.size(-1), dtype=q.dtype) if state is None else state.clone()
    out = torch.empty(n, heads, v.size(-1), dtype=q.dtype)
    for t in range(n):
        s = s * g[t][:, :, None]
        u = beta[t][:, None] * (v[t] - (s * k[t][:, :, None]).sum(1))
        s = s + k[t][:, :, None] * u[:, None, :]
        out[t] = (s * q[t][:, :, None]).sum(1)
    return out, s


def channel_delta(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mix: dict, eps: float) -> torch.Tensor:
    n, heads, groups, dim, vdim = h.size(0), mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"]

    def conv_silu(name):
        z = short_conv(h @ w[p + name].T, w[p + name + ".conv"])
        return z * sigmoid(z)

    rep = heads // groups
    q = unit(conv_silu("q").reshape(n, groups, dim)) * dim ** -0.5
    k = unit(conv_silu("k").reshape(n, groups, dim))
    v = conv_silu("v").reshape(n, heads, vdim)
    beta = sigmoid(h @ w[p + "b"].T)
    step = softplus(h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "dt_bias"]).reshape(n, heads, dim)
    g = torch.exp(-torch.exp(w[p + "A_log"])[:, None] * step)
    o, _ = delta_scan(q.repeat_interleave(rep, 1), k.repeat_interleave(rep, 1), v, g, beta)
    gate = sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T).reshape(n, heads, vdim)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(n, heads * vdim) @ w[p + "o"].T


def dense_mlp(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def layer_order(cfg: dict) -> List[tuple]:
    """(layer, pass number if the layer opens a pass, else None) in the order they run."""
    loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 0}
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], len(cfg["layers"]))]


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens, dtype=torch.float64,
            layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[tokens, vocab]`` of one sequence; the residual after every layer that ran is
    appended to ``layers_out`` if given."""
    w = {k: t.to(dtype) for k, t in weights.items()}
    eps = cfg["norm"]["eps"]
    x = x0 = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    for i, opens in layer_order(cfg):
        p, layer = f"l{i}.", cfg["layers"][i]
        mix = layer["mixer"]
        if opens is not None:
            x = torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][opens]
        h = rms(x, eps) * (1 + w[p + "norm1"])
        if layer["type"] == "attention":
            x = x + attention(h, w, p + "mix.", mix, eps)
        elif layer["type"] == "rglru":
            x = x + rglru(h, w, p + "mix.", mix)
        elif layer["type"] == "channel_delta":
            x = x + channel_delta(h, w, p + "mix.", mix, eps)
        else:
            raise ValueError(layer["type"])
        if layer["mlp"] is not None:
            x = x + dense_mlp(rms(x, eps) * (1 + w[p + "norm2"]), w, p + "mlp.")
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms(x, eps) * (1 + w["final.norm"]) @ w["head"].T * cfg["logit_scale"]
