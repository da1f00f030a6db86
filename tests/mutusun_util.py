"""Small Mutusun models for tests: configurations and random weights on disk.
Driving, comparing and writing is shared with the other hybrid designs."""

from __future__ import annotations

import copy

import torch

from tefezen_util import (error, errors, feed, rounding_limits,  # noqa: F401
                          tokens, write)


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, identity=2, top=3, ff=24, limit=0.7):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "identity": identity, "top": top}}


def layer(heads=4, kv_heads=2, dim=16, vdim=24, chunk=13, scale=0.5,
          softcap=9.0, mlp=()):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "mask": {"size": chunk}, "scale": scale,
                      "softcap": softcap},
            "mlp": moe() if mlp == () else mlp}


def again(layers, j):
    """Another run of layer j's tensors."""
    return {**copy.deepcopy(layers[j]), "weights_of": j}


def config(layers, width=56, vocab=272, eps=1e-4, taps=4):
    return {"architecture": "Mutusun", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "canon": {"taps": taps}, "layers": layers}


def standard():
    """Dense, expert and no feed-forward, several chunk lengths, layers that
    run with the tensors of an earlier and of a later one."""
    own = [layer(heads=6, kv_heads=2, dim=24, vdim=16, chunk=21,
                 mlp=dense(72)),
           layer(heads=3, kv_heads=3, dim=8, vdim=32, chunk=37, softcap=4.0),
           layer(heads=4, kv_heads=1, dim=16, vdim=8, chunk=50, scale=0.3,
                 mlp=None),
           layer(chunk=5, mlp=moe(4, 0, 2, 40, 1.5))]
    return config([own[0], own[1], {**copy.deepcopy(own[2]), "weights_of": 4},
                   again(own, 1), own[2], own[3], again(own, 0)])


def shapes(cfg):
    w, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, w), "head": (v, w), "final.norm": (w,)}
    for i, x in enumerate(cfg["layers"]):
        if "weights_of" in x:
            continue
        p, m, f = f"l{i}.", x["mixer"], x["mlp"]
        h, g, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n in ("1", "2")[:1 if f is None else 2]:
            out.update({f"{p}norm{n}": (w,), f"{p}norm{n}b": (w,),
                        f"{p}canon{n}": (w, cfg["canon"]["taps"])})
        out.update({p + "mix.q": (h * d, w), p + "mix.k": (g * d, w),
                    p + "mix.v": (g * e, w), p + "mix.o": (w, h * e),
                    p + "mix.q.norm": (d,), p + "mix.k.norm": (d,),
                    p + "mix.pb": (h,)})
        if f is None:
            continue
        if f["kind"] == "dense":
            out.update({p + "mlp.up": (f["ff"], w),
                        p + "mlp.down": (w, f["ff"])})
            continue
        r, k = f["router"], f["expert"]["ff"]
        n = r["experts"] + r["identity"]
        out.update({p + "mlp.router": (n, w), p + "mlp.correction": (n,)})
        for j in range(r["experts"]):
            out.update({f"{p}mlp.e{j}.gate": (k, w), f"{p}mlp.e{j}.up": (k, w),
                        f"{p}mlp.e{j}.down": (w, k)})
    return out


def weights(cfg, seed=0):
    """bf16 weights under which every part shows: scores spread over the
    cap's bend, gates reach their limits, corrections change choices."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        x = torch.randn(shape, generator=gen)
        last = name.rsplit(".", 1)[-1]
        if name.endswith(("q.norm", "k.norm")):
            x = 1.0 + 0.5 * x
        elif "norm" in last:
            x = 0.5 * x                       # stored around zero
        elif last.startswith("canon"):
            x = 0.5 * x
        elif last == "correction":
            x = 0.1 * x
        elif last == "pb":
            x = x - 1.0
        elif name == "embed":
            x = 0.3 * x
        else:
            x = x / shape[-1] ** 0.5
        out[name] = x.to(torch.bfloat16)
    return out
