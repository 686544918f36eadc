"""Small random Lugitar models for the tests: a configuration from a list of layer descriptions, and
its tensors by stored name."""

import torch


def rotation(dims, base=500.0, scaling=None):
    rot = {"dims": dims, "base": base}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return rot


YARN = (4.0, 64, 8.0, 1.0)


def latent(heads=3, dim=24, rot_dim=8, vdim=40, kv_rank=56, window=11, scale=None, ff=72, kv_from=None, rot=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
             "rot": rot or rotation(rot_dim, scaling=YARN), "scale": scale or (dim + rot_dim) ** -0.5}
    if window is not None:
        mixer["mask"] = {"size": window}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mixer, "mlp": ff and {"kind": "dense", "ff": ff}}


def lightning(heads=3, dim=40, vdim=24, decay=(0.5, 0.93, 0.9995), ff=72):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)},
            "mlp": ff and {"kind": "dense", "ff": ff}}


def config(layers, width=88, vocab=101, eps=1e-5, mult=0.4):
    layers = [dict(l, mlp=l["mlp"] or None) for l in layers]
    return {"architecture": "Lugitar", "layers": layers, "norm": {"eps": eps}, "residual_mult": mult,
            "vocab": vocab, "width": width}


def mixed(**kw):
    """Both mixers, own and shared latents, different sizes and windows per layer, a layer without feed-forward."""
    return config([
        latent(window=11),
        lightning(),
        latent(heads=2, dim=32, vdim=16, window=29, kv_from=0, ff=None),
        latent(heads=1, dim=8, rot_dim=16, vdim=72, kv_rank=40, window=1, ff=40, rot=rotation(16, 100.0)),
        lightning(heads=1, dim=16, vdim=72, decay=(0.97,), ff=50),
        latent(heads=5, dim=16, vdim=8, window=None, kv_from=0),
    ], **kw)


def tensors(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)

    def r(*size, std=1.0):
        return (torch.randn(*size, generator=g) * std).to(dtype)

    def norm(n):
        return (1.0 + 0.3 * torch.randn(n, generator=g)).to(dtype)

    w, out = cfg["width"], {}
    out["embed"] = r(cfg["vocab"], w)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"], out[p + "norm1b"] = norm(w), norm(w)
        h, d, v = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "latent_attention":
            rank, rd = m["kv_rank"], m["rot_dim"]
            out[p + "mix.q"] = r(h * (d + rd), w, std=2 * w ** -0.5)
            if "kv_from" not in m:
                out[p + "mix.dkv"] = r(rank + rd, w, std=w ** -0.5)
                out[p + "mix.dkv.norm"] = norm(rank)
            out[p + "mix.uk"], out[p + "mix.uv"] = r(h * d, rank, std=rank ** -0.5), r(h * v, rank, std=rank ** -0.5)
            out[p + "mix.g"] = r(h, w, std=w ** -0.5)
        else:
            for name, n in (("q", h * d), ("k", h * d), ("v", h * v), ("g", h * v)):
                out[p + "mix." + name] = r(n, w, std=w ** -0.5)
            out[p + "mix.norm"] = norm(h * v)
        out[p + "mix.o"] = r(w, h * v, std=(h * v) ** -0.5)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out[p + "norm2"], out[p + "norm2b"] = norm(w), norm(w)
            out[p + "mlp.gate"], out[p + "mlp.up"] = r(ff, w, std=w ** -0.5), r(ff, w, std=w ** -0.5)
            out[p + "mlp.down"] = r(w, ff, std=ff ** -0.5)
    out["final.norm"] = norm(w)
    out["head"] = r(cfg["vocab"], w, std=w ** -0.5)
    return out


def relative_rms(got, want):
    """rms(got - want) / rms(want) of each row's difference, the worst row."""
    got, want = got.double().cpu(), want.double().cpu()
    scale = want.pow(2).mean().sqrt()
    return ((got - want).pow(2).mean(-1).sqrt() / scale).max().item()
