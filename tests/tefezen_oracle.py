"""Plain, slow implementation of the Tefezen design, one function per
mechanism, in float64 on the CPU.

It shares no code with the framework: whole sequences only, no cache, no
batching, loops over heads and tokens.  Elementwise functions, the interleaved
rotation and the windowed softmax are those of the other plain
implementation.  Weights are a dict name -> tensor, the configuration is the
parsed config.json.
"""

from __future__ import annotations

import torch

from sumosun_oracle import (F64, gelu_tanh, read_safetensors,  # noqa: F401
                            rms, rotate_pairs, silu,
                            window_softmax_attention)


# -------------------------------------------------------- latent attention

def latents(h, w, m, eps):
    """Normed latent c [T, rank] and rotated shared key part [T, rot]."""
    both = h @ w["dkv"].T
    c = rms(both[:, :m["kv_rank"]], eps) * w["dkv.norm"]
    pos = torch.arange(h.shape[0])
    return c, rotate_pairs(both[:, m["kv_rank"]:], pos, m["rot"]["dims"],
                           m["rot"]["base"])


def latent_attention(h, w, m, c, kr):
    """Attention over latents (c, kr), this layer's or another one's."""
    T, H = h.shape[0], m["heads"]
    D, R, E = m["dim"], m["rot_dim"], m["vdim"]
    pos = torch.arange(T)
    q = (h @ w["q"].T).view(T, H, D + R)
    k = (c @ w["uk"].T).view(T, H, D)
    v = (c @ w["uv"].T).view(T, H, E)
    heads = []
    for n in range(H):
        qr = rotate_pairs(q[:, n, D:], pos, m["rot"]["dims"],
                          m["rot"]["base"])
        heads.append(window_softmax_attention(
            torch.cat([q[:, n, :D], qr], -1), torch.cat([k[:, n], kr], -1),
            v[:, n], m["scale"], m["mask"]["size"]))
    return torch.cat(heads, -1) @ w["o"].T


# ----------------------------------------------------- lightning attention

def decayed_recurrence(q, k, v, decay):
    """One head: q, k [T, D], v [T, E], a constant decay -> o [T, E]."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=F64)
    out = []
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out.append(S.T @ q[t])
    return torch.stack(out)


def lightning(h, w, m, eps):
    T, H = h.shape[0], m["heads"]
    q = silu(h @ w["q"].T).view(T, H, m["dim"])
    k = silu(h @ w["k"].T).view(T, H, m["dim"])
    v = silu(h @ w["v"].T).view(T, H, m["vdim"])
    o = torch.cat([decayed_recurrence(q[:, n], k[:, n], v[:, n],
                                      m["decay"][n]) for n in range(H)], -1)
    return (rms(o, eps) * w["norm"] * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ----------------------------------------------------------------- experts

def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, top):
    """Router logits [T, experts] -> chosen experts and weights [T, top]."""
    ids = torch.argsort(z, -1, descending=True)[:, :top]
    s = torch.exp(torch.gather(z, 1, ids) - z.max(-1, keepdim=True).values)
    return ids, s / s.sum(-1, keepdim=True)


def mixture(h, w, m):
    ids, weight = route(h @ w["router"].T, m["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(ids.shape[1]):
            out[t] += weight[t, j] * expert(h[t], w, f"e{int(ids[t, j])}.")
    if m.get("shared") is None:
        return out
    return out + (torch.sigmoid(h @ w["shared.sg"].T)
                  * expert(h, w, "shared."))


# --------------------------------------------------------------- the model

def token_side(x, e, w, eps):
    """Gate of the residual times the token's entry, projected and normed."""
    y = (gelu_tanh(x @ w["gate"].T) * e) @ w["proj"].T
    return rms(y, eps) * w["norm"]


def local(weights, prefix):
    return {n[len(prefix):]: t.to(F64) for n, t in weights.items()
            if n.startswith(prefix)}


def offset_norm(weights, name, x, eps):
    return rms(x, eps) * (1.0 + weights[name].to(F64))


def forward(config, weights, tokens):
    """All logits [T, vocab] and the residual after every layer."""
    eps = config["norm"]["eps"]
    ids = torch.as_tensor(tokens)
    x = weights["embed"].to(F64)[ids] * config["embedding"]["scale"]
    side = weights["side.embed"].to(F64)[ids]
    n = config["token_side"]["dim"]
    trail, kept = [], {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w = local(weights, p + "mix.")
        if layer["type"] == "latent_attention":
            if m.get("kv_from") is None:
                kept[i] = latents(x, w, m, eps)
                c, kr = kept[i]
            else:
                c, kr = kept[m["kv_from"]]
            y = latent_attention(x, w, m, c, kr)
        else:
            y = lightning(x, w, m, eps)
        x = x + offset_norm(weights, p + "norm1", y, eps)
        if layer["mlp"] is not None:
            y = mixture(x, local(weights, p + "mlp."), layer["mlp"])
            x = x + offset_norm(weights, p + "norm2", y, eps)
        x = x + token_side(x, side[:, i * n:(i + 1) * n],
                           local(weights, p + "side."), eps)
        trail.append(x)
    return (offset_norm(weights, "final.norm", x, eps)
            @ weights["head"].to(F64).T), trail


def greedy(config, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(config, weights, toks)[0][-1].argmax()))
    return toks[len(prompt):]
