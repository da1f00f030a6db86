"""Plain, slow implementation of the Mutusun design, one function per
mechanism, in float64 on the CPU.

It shares no code with the framework: whole sequences only, no cache, no
batching, loops over heads and tokens.  Weights are a dict name -> tensor, the
configuration is the parsed config.json.
"""

from __future__ import annotations

import torch

from sumosun_oracle import F64, read_safetensors, rms  # noqa: F401
from tefezen_oracle import local, offset_norm


# ------------------------------------------------------- input convolution

def causal_conv(h, w):
    """h [T, width] plus its convolution over time, one filter per channel;
    w [width, taps], the last tap meets the token itself."""
    taps = w.shape[1]
    out = h.clone()
    for t in range(h.shape[0]):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


# --------------------------------------------------------------- attention

def capped(score, cap):
    return cap * torch.tanh(score / cap)


def chunk_start(i, size):
    return i - i % size


def sigmoid_attention(q, k, v, scale, cap, bias, size):
    """One head: q, k [T, D], v [T, E]; token i sees its chunk up to itself;
    weights are not normalized."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F64)
    for i in range(q.shape[0]):
        lo = chunk_start(i, size)
        s = capped((k[lo:i + 1] @ q[i]) * scale, cap)
        out[i] = torch.sigmoid(s + bias) @ v[lo:i + 1]
    return out


def attention(h, w, m, eps):
    """The mixer 'attention'; w maps local names to tensors."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = rms((h @ w["q"].T).view(T, H, m["dim"]), eps) * w["q.norm"]
    k = rms((h @ w["k"].T).view(T, G, m["dim"]), eps) * w["k.norm"]
    v = (h @ w["v"].T).view(T, G, m["vdim"])
    heads = [sigmoid_attention(q[:, n], k[:, n // (H // G)],
                               v[:, n // (H // G)], m["scale"], m["softcap"],
                               w["pb"][n], m["mask"]["size"])
             for n in range(H)]
    return torch.cat(heads, -1) @ w["o"].T


# ------------------------------------------------------------ feed-forward

def squared_relu(h, w):
    return (h @ w["up"].T).clamp(min=0) ** 2 @ w["down"].T


def expert(h, w, p, limit):
    g = (h @ w[p + "gate"].T).clamp(max=limit)
    u = (h @ w[p + "up"].T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w[p + "down"].T


def route(z, correction, top):
    """Router logits [T, n] -> chosen outputs and weights [T, top]: softmax
    over all, the correction moves the choice only."""
    s = torch.exp(z - z.max(-1, keepdim=True).values)
    s = s / s.sum(-1, keepdim=True)
    ids = torch.argsort(s + correction, -1, descending=True)[:, :top]
    return ids, torch.gather(s, 1, ids)


def mixture(h, w, m):
    r = m["router"]
    ids, weight = route(h @ w["router"].T, w["correction"], r["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(ids.shape[1]):
            e = int(ids[t, j])
            y = h[t] if e >= r["experts"] \
                else expert(h[t], w, f"e{e}.", m["expert"]["limit"])
            out[t] += weight[t, j] * y
    return out


# --------------------------------------------------------------- the model

def forward(config, weights, tokens):
    """All logits [T, vocab] and the residual after every layer."""
    eps = config["norm"]["eps"]
    x = weights["embed"].to(F64)[torch.as_tensor(tokens)]
    trail = []
    for i, layer in enumerate(config["layers"]):
        p = f"l{layer.get('weights_of', i)}."

        def sublayer(x, n, branch):
            h = offset_norm(weights, f"{p}norm{n}", x, eps)
            h = causal_conv(h, weights[f"{p}canon{n}"].to(F64))
            return x + offset_norm(weights, f"{p}norm{n}b", branch(h), eps)

        w = local(weights, p + "mix.")
        x = sublayer(x, 1, lambda h: attention(h, w, layer["mixer"], eps))
        m = layer["mlp"]
        if m is not None:
            f = local(weights, p + "mlp.")
            x = sublayer(x, 2, lambda h: mixture(h, f, m)
                         if m["kind"] == "moe" else squared_relu(h, f))
        trail.append(x)
    return (offset_norm(weights, "final.norm", x, eps)
            @ weights["head"].to(F64).T), trail


def greedy(config, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(config, weights, toks)[0][-1].argmax()))
    return toks[len(prompt):]
