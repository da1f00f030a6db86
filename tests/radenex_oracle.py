"""Plain, slow implementation of the Radenex design, one function per
mechanism, in float64 on the CPU.

It shares no code with the framework: whole sequences only, no cache, no
batching, loops over heads and tokens.  Weights are a dict name -> tensor, the
configuration is the parsed config.json.
"""

from __future__ import annotations

import math

import torch

from mutusun_oracle import squared_relu
from sumosun_oracle import F64, read_safetensors, rms  # noqa: F401
from tefezen_oracle import local


# ---------------------------------------------------------------- rotation

def base_frequencies(dims, base):
    return [base ** (-2.0 * i / dims) for i in range(dims // 2)]


def linear_frequencies(dims, base, factor):
    return [f / factor for f in base_frequencies(dims, base)]


def yarn_frequencies(dims, base, factor, original, fast, slow):
    """Fast pairs keep their frequency, slow ones are divided by `factor`, a
    ramp between; and the factor on cosine and sine."""
    def pair_with(turns):
        return dims * math.log(original / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(pair_with(fast)), 0)
    hi = min(math.ceil(pair_with(slow)), dims - 1)
    out = []
    for i, f in enumerate(base_frequencies(dims, base)):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_halves(x, angle, freqs, gain=1.0):
    """x [T, D] with row t turned by angle[t] * freqs[i]: dimension i of the
    first 2 * len(freqs) meets the one half of these further on."""
    y, n = x.clone(), len(freqs)
    for i, f in enumerate(freqs):
        a = angle.to(F64) * f
        c, s = torch.cos(a) * gain, torch.sin(a) * gain
        u, v = x[:, i], x[:, i + n]
        y[:, i] = u * c - v * s
        y[:, i + n] = v * c + u * s
    return y


# --------------------------------------------------------------- attention

def softmax_with_sink(s, sink):
    """Weights of scores s under a denominator with exp(sink) more."""
    m = max(float(s.max()), float(sink))
    e = torch.exp(s - m)
    return e / (e.sum() + math.exp(float(sink) - m))


def visible(i, size, keep):
    """Positions that i sees: the window, and the first `keep`."""
    return [j for j in range(i + 1) if i - j < size or j < keep]


def sink_attention(q, k, v, scale, sink, seen):
    """One head: q, k [T, D], v [T, E]; token i sees the positions seen(i)."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F64)
    for i in range(q.shape[0]):
        j = seen(i)
        out[i] = softmax_with_sink((k[j] @ q[i]) * scale, sink) @ v[j]
    return out


def window_attention(h, w, m, eps):
    """The mixer 'attention'; w maps local names to tensors."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    D, E, rot, mask = m["dim"], m["vdim"], m["rot"], m["mask"]
    pos = torch.arange(T)
    freqs = linear_frequencies(rot["dims"], rot["base"],
                               rot["scaling"]["factor"])
    turn = base_frequencies(E, rot["base"])
    q = (h @ w["q"].T).view(T, H, D)
    k = (h @ w["k"].T).view(T, G, D)
    v = (h @ w["v"].T).view(T, G, E)
    heads = []
    for n in range(H):
        g = n // (H // G)
        o = sink_attention(
            rms(rotate_halves(q[:, n], pos, freqs), eps),
            rms(rotate_halves(k[:, g], pos, freqs), eps),
            rotate_halves(v[:, g], pos, turn), m["scale"], 0.0,
            lambda i: visible(i, mask["size"], mask["keep_first"]))
        heads.append(rotate_halves(o, -pos, turn))
    return torch.cat(heads, -1) @ w["o"].T


def latent_attention(h, w, m, eps):
    """The mixer 'latent_attention'."""
    T, H, r, rot = h.shape[0], m["heads"], m["kv_rank"], m["rot"]
    D, E, s = m["dim"], m["vdim"], rot["scaling"]
    pos = torch.arange(T)
    freqs, gain = yarn_frequencies(rot["dims"], rot["base"], s["factor"],
                                   s["original"], s["fast"], s["slow"])
    q = (h @ w["q"].T).view(T, H, D + m["rot_dim"])
    both = h @ w["dkv"].T
    c = rms(both[:, :r], eps) * w["dkv.norm"]
    kr = rotate_halves(both[:, r:], pos, freqs, gain)
    k = (c @ w["uk"].T).view(T, H, D)
    v = (c @ w["uv"].T).view(T, H, E)
    gate = torch.sigmoid(h @ w["g"].T)
    heads = []
    for n in range(H):
        qr = rotate_halves(q[:, n, D:], pos, freqs, gain)
        o = sink_attention(torch.cat([q[:, n, :D], qr], -1),
                           torch.cat([k[:, n], kr], -1), v[:, n], m["scale"],
                           w["sink"][n], lambda i: list(range(i + 1)))
        heads.append(gate[:, n:n + 1] * o)
    return torch.cat(heads, -1) @ w["o"].T


MIXERS = {"attention": window_attention, "latent_attention": latent_attention}


# --------------------------------------------------------------- the model

def layer_runs(config):
    """Layer indices in the order in which they run."""
    n, loop = len(config["layers"]), config["loop"]
    a, b = loop["start"], loop["stop"]
    return [*range(a), *list(range(a, b)) * loop["times"], *range(b, n)]


def forward(config, weights, tokens):
    """All logits [T, vocab] and the residual after every layer run."""
    eps = config["norm"]["eps"]
    x = weights["embed"].to(F64)[torch.as_tensor(tokens)]
    trail = []
    for i in layer_runs(config):
        layer, p = config["layers"][i], f"l{i}."
        h = rms(x, eps) * weights[p + "norm1"].to(F64)
        y = MIXERS[layer["type"]](h, local(weights, p + "mix."),
                                  layer["mixer"], eps)
        if layer["mlp"] is not None:
            y = y + squared_relu(h, local(weights, p + "mlp."))
        x = x + y
        trail.append(x)
    return (rms(x, eps) * weights["final.norm"].to(F64)
            @ weights["head"].to(F64).T), trail


def greedy(config, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(config, weights, toks)[0][-1].argmax()))
    return toks[len(prompt):]
