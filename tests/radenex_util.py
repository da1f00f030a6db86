"""Small Radenex models for tests: configurations and random weights on disk.
Driving, comparing and writing is shared with the other hybrid designs."""

from __future__ import annotations

import torch

from tefezen_util import (error, errors, feed, rounding_limits,  # noqa: F401
                          tokens, write)


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def window(heads=4, kv_heads=2, dim=16, vdim=24, size=13, keep=2, scale=0.5,
           rot=8, base=500.0, factor=2.5, mlp=()):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "scale": scale,
                      "mask": {"size": size, "keep_first": keep},
                      "rot": {"dims": rot, "base": base,
                              "scaling": {"factor": factor}}},
            "mlp": dense() if mlp == () else mlp}


def latent(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=32, scale=0.3,
           base=5000.0, factor=4.0, original=64, fast=8.0, slow=0.5, mlp=()):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim,
                      "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "rot": {"dims": rot_dim, "base": base,
                              "scaling": {"factor": factor, "fast": fast,
                                          "original": original,
                                          "slow": slow}}},
            "mlp": dense() if mlp == () else mlp}


def config(layers, width=56, vocab=272, eps=1e-4, loop=(0, 0, 1)):
    return {"architecture": "Radenex", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "layers": layers,
            "loop": dict(zip(("start", "stop", "times"), loop))}


def standard():
    """Both mixers in unlike sizes, several windows, layers without a
    feed-forward, and three of them run three times."""
    return config([
        latent(heads=2, dim=24, rot_dim=16, vdim=16, kv_rank=40,
               mlp=dense(72)),
        window(heads=6, kv_heads=2, dim=24, vdim=16, size=21, keep=5, rot=16),
        latent(heads=5, dim=8, rot_dim=8, vdim=40, kv_rank=24, factor=16.0,
               mlp=None),
        window(heads=3, kv_heads=3, dim=8, vdim=32, size=37, keep=1, rot=8,
               scale=0.8, factor=1.5),
        window(heads=4, kv_heads=1, dim=16, vdim=8, size=5, keep=17, rot=4,
               mlp=None)], loop=(1, 4, 3))


def shapes(cfg):
    w, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, w), "head": (v, w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        x, h, d, e = p + "mix.", m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = (w,)
        out[x + "o"] = (w, h * e)
        if layer["type"] == "attention":
            g = m["kv_heads"]
            out.update({x + "q": (h * d, w), x + "k": (g * d, w),
                        x + "v": (g * e, w)})
        else:
            r, t = m["kv_rank"], m["rot_dim"]
            out.update({x + "q": (h * (d + t), w), x + "dkv": (r + t, w),
                        x + "dkv.norm": (r,), x + "uk": (h * d, r),
                        x + "uv": (h * e, r), x + "sink": (h,),
                        x + "g": (h, w)})
        if f is not None:
            out.update({p + "mlp.up": (f["ff"], w),
                        p + "mlp.down": (w, f["ff"])})
    return out


def weights(cfg, seed=0):
    """bf16 weights under which every part shows: single keys stand out, sinks
    take a good share, gates open and close."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        x = torch.randn(shape, generator=gen)
        last = name.rsplit(".", 1)[-1]
        if "norm" in last:
            x = 1.0 + 0.4 * x
        elif last == "sink":
            x = 2.0 + x
        elif name != "embed":
            x = x / shape[-1] ** 0.5
            if last in ("g", "uk") or name.endswith("mix.q"):
                x = 2.0 * x
            elif last == "down":
                x = 0.5 * x
        out[name] = x.to(torch.bfloat16)
    return out
