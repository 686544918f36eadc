"""Small random Sarulix models for the tests: a configuration from a list of layer descriptions, and
its tensors by stored name."""

import torch

from lugitar_helpers import relative_rms  # noqa: F401


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def attention(heads=6, kv_heads=3, dim=24, vdim=40, rot=12, base=700.0, scale=None, softcap=9.0, ff=72):
    return _layer("attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                "rot": {"dims": rot, "base": base}, "scale": scale or dim ** -0.5, "softcap": softcap}, ff)


def rglru(width=90, blocks=3, conv=4, ff=None):
    return _layer("rglru", {"width": width, "blocks": blocks, "conv": conv}, ff)


def delta(heads=4, kv_heads=2, dim=40, vdim=24, conv=3, ff=None):
    return _layer("channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, ff)


# (eps is large on purpose: a head whose read-out nearly cancels would turn bf16 rounding into an error of its
# own size under a small one, and an eps in the wrong place shows)
def config(layers, width=88, vocab=101, eps=1e-2, scale=2.5, logit_scale=0.4, loop=(0, 0, 0)):
    out = {"architecture": "Sarulix", "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "logit_scale": logit_scale, "vocab": vocab, "width": width}
    if loop[2]:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def mixed(**kw):
    """All mixers, different sizes per layer, feed-forwards behind some, the middle run three times."""
    kw.setdefault("loop", (1, 4, 3))
    return config([
        delta(),
        rglru(ff=40),
        attention(),
        delta(heads=3, kv_heads=1, dim=16, vdim=72, conv=2, ff=50),
        attention(heads=2, kv_heads=2, dim=64, vdim=16, rot=64, softcap=30.0, ff=None),
        rglru(width=64, blocks=1, conv=2),
    ], **kw)


def tensors(cfg, seed=0, dtype=torch.bfloat16, ranks=(12, 20)):
    g = torch.Generator().manual_seed(seed)

    def r(*size, std=1.0, mean=0.0):
        return (torch.randn(*size, generator=g) * std + mean).to(dtype)

    def uniform(lo, hi, *size):
        return (torch.rand(*size, generator=g) * (hi - lo) + lo).to(dtype)

    w, out = cfg["width"], {}
    out["embed"] = r(cfg["vocab"], w, std=1 / cfg["embedding"]["scale"])
    if "loop" in cfg:
        out["loop.in"] = r(w, 2 * w, std=(2 * w) ** -0.5)
        out["loop.step"] = r(cfg["loop"]["times"], w, std=0.4)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        out[f"l{i}.norm1"] = r(w, std=0.3)

        def lin(name, rows, cols=w, bias=False, std=1.0):
            out[p + name] = r(rows, cols, std=std * cols ** -0.5)
            if bias:
                out[p + name + ".b"] = r(rows, std=0.3)

        def conv(name, rows):
            out[p + name] = r(rows, m["conv"], std=m["conv"] ** -0.5)

        if layer["type"] == "attention":
            h, kh, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            lin("q", h * d, bias=True)
            lin("k", kh * d, bias=True)
            lin("v", kh * v, bias=True)
            lin("g", h * v)
            lin("o", w, h * v, bias=True)
            out[p + "q.norm"], out[p + "k.norm"] = r(d, std=0.3, mean=1.4), r(d, std=0.3, mean=1.4)
        elif layer["type"] == "rglru":
            c, b = m["width"], m["blocks"]
            lin("y", c, bias=True)
            lin("x", c, bias=True)
            conv("conv", c)
            out[p + "conv.b"] = r(c, std=0.2)
            for name in ("ra", "ri"):
                out[p + name] = r(b, c // b, c // b, std=(c // b) ** -0.5)
            out[p + "ra.b"], out[p + "ri.b"] = uniform(-6, 2, b, c // b), r(b, c // b)
            out[p + "lam"] = uniform(-5, 1, c)
            lin("o", w, c)
        else:
            h, kh, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for name, n in (("q", kh * d), ("k", kh * d), ("v", h * v)):
                lin(name, n)
                conv(name + ".conv", n)
            lin("b", h)
            out[p + "A_log"], out[p + "dt_bias"] = uniform(-4, 1.5, h), uniform(-5, 1, h * d)
            lin("a1", ranks[0])
            lin("a2", h * d, ranks[0])
            lin("g1", ranks[1])
            lin("g2", h * v, ranks[1])
            out[p + "norm"] = r(v, std=0.3, mean=1.0)
            lin("o", w, h * v)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out[f"l{i}.norm2"] = r(w, std=0.3)
            out[f"l{i}.mlp.gate"], out[f"l{i}.mlp.up"] = r(ff, w, std=w ** -0.5), r(ff, w, std=w ** -0.5)
            out[f"l{i}.mlp.down"] = r(w, ff, std=ff ** -0.5)
    out["final.norm"] = r(w, std=0.3)
    out["head"] = r(cfg["vocab"], w, std=w ** -0.5)
    return out
