"""Small Tefezen models for tests: configurations and random weights on disk.
Driving and comparing is shared with the other hybrid design's helpers."""

from __future__ import annotations

import json
import os

import torch

from sumosun_util import error, feed, tokens  # noqa: F401


def moe(experts=5, top=2, ff=24, shared=40):
    m = {"kind": "moe", "expert": {"ff": ff},
         "router": {"experts": experts, "top": top}}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def latent(heads=2, dim=16, rot_dim=8, vdim=24, kv_rank=32, window=9,
           base=1000.0, scale=None, kv_from=None, mlp=()):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
         "kv_rank": kv_rank, "mask": {"size": window},
         "rot": {"base": base, "dims": rot_dim},
         "scale": scale or (dim + rot_dim) ** -0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m,
            "mlp": moe() if mlp == () else mlp}


def lightning(heads=2, dim=16, vdim=24, decay=None, mlp=()):
    decay = decay or [1.0 - 0.3 / 4 ** i for i in range(heads)]
    return {"type": "lightning",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                      "decay": decay},
            "mlp": moe() if mlp == () else mlp}


def config(layers, width=56, vocab=272, eps=1e-5, scale=2.0, side=8):
    return {"architecture": "Tefezen", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "embedding": {"scale": scale},
            "token_side": {"dim": side}, "layers": layers}


def standard():
    """Both mixers, latents of an earlier layer under other heads, sizes and
    window, a layer without feed-forward, one without shared expert."""
    return config([
        latent(heads=3, dim=24, rot_dim=8, vdim=16, kv_rank=40, window=21),
        lightning(heads=3, dim=24, vdim=16, mlp=moe(7, 3, 16, None)),
        latent(heads=5, dim=8, rot_dim=8, vdim=40, kv_rank=40, window=37,
               kv_from=0, mlp=None),
        lightning(heads=2, dim=16, vdim=48, decay=[0.97, 0.5]),
        latent(heads=2, dim=16, rot_dim=16, vdim=24, kv_rank=24, window=5,
               base=300.0)])


def shapes(cfg):
    w, v, n = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"]
    out = {"embed": (v, w), "head": (v, w), "final.norm": (w,),
           "side.embed": (v, n * len(cfg["layers"]))}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h, d, e = m["heads"], m["dim"], m["vdim"]
        x = p + "mix."
        out[p + "norm1"] = (w,)
        out[x + "o"] = (w, h * e)
        if layer["type"] == "latent_attention":
            r, t = m["kv_rank"], m["rot_dim"]
            out.update({x + "q": (h * (d + t), w), x + "uk": (h * d, r),
                        x + "uv": (h * e, r)})
            if "kv_from" not in m:
                out.update({x + "dkv": (r + t, w), x + "dkv.norm": (r,)})
        else:
            out.update({x + "q": (h * d, w), x + "k": (h * d, w),
                        x + "v": (h * e, w), x + "g": (h * e, w),
                        x + "norm": (h * e,)})
        f = layer["mlp"]
        if f is not None:
            out[p + "norm2"] = (w,)
            out[p + "mlp.router"] = (f["router"]["experts"], w)
            sizes = {f"e{j}": f["expert"]["ff"]
                     for j in range(f["router"]["experts"])}
            if "shared" in f:
                sizes["shared"] = f["shared"]["ff"]
                out[p + "mlp.shared.sg"] = (1, w)
            for j, k in sizes.items():
                out.update({f"{p}mlp.{j}.gate": (k, w),
                            f"{p}mlp.{j}.up": (k, w),
                            f"{p}mlp.{j}.down": (w, k)})
        out.update({p + "side.gate": (n, w), p + "side.proj": (w, n),
                    p + "side.norm": (w,)})
    return out


def weights(cfg, seed=0, sharp=2.0):
    """bf16 weights under which single keys stand out: queries and latents
    are scaled up (`sharp`), and the residual does not just follow the
    token.  Rounding grows with `sharp` as well."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        x = torch.randn(shape, generator=gen)
        if name.endswith(("norm1", "norm2", "final.norm")):
            x = 0.6 * x                       # stored around zero
        elif name.endswith("norm"):
            x = 1.0 + 0.5 * x
        elif name == "embed":
            x = 0.15 * x
        elif name == "head":
            x = x / shape[1] ** 0.5
        elif name != "side.embed":
            x = x / shape[1] ** 0.5
            if name.endswith(("mix.q", "mix.uk", "router")):
                x = sharp * x
        out[name] = x.to(torch.bfloat16)
    return out


def errors(got, want):
    """Per-position RMS difference (mean removed), relative to the RMS of all
    wanted logits."""
    d = got.double() - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def rounding_limits(forward, cfg, w, toks, times=3.0):
    """What 16-bit rounding may cost at every position: a multiple of the
    plain implementation's answer to noise of that size on all weights (some
    positions of a small random model amplify it a hundredfold)."""
    want, worst = forward(cfg, w, toks)[0], 0.0
    for seed in range(8):
        g = torch.Generator().manual_seed(seed)
        noisy = {n: t.double() * (1 + 2 ** -8.5 * torch.randn(
            t.shape, generator=g, dtype=torch.float64)) for n, t in w.items()}
        e = errors(forward(cfg, noisy, toks)[0], want)
        worst = torch.maximum(e, torch.as_tensor(worst, dtype=e.dtype))
    return times * worst.clamp_min(float(worst.mean()))


def write(folder, cfg, w):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({n: t.contiguous() for n, t in w.items()},
              os.path.join(folder, "model.safetensors"))
    return str(folder)
