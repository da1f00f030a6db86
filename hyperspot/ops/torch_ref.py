"""Pure-PyTorch reference implementations of every engine op.

These are the numerics ground truth for the CDNA4 HIP kernels (tests compare
the gfx950 kernels against these in fp32) and the CPU execution path for
CI — this container has no GPU.  They are written for clarity, not speed.

Conventions shared with the HIP kernels (csrc/):
  - token-major activations: x is [T, hidden] (T = flattened tokens of the
    whole batch, prefill + decode mixed)
  - q/k/v are [T, n_heads, head_dim] after the qkv projection split
  - paged KV cache: k_cache/v_cache are [num_blocks, kv_heads, block, head_dim]
  - slot_mapping[t] = block_id * block_size + offset for token t
  - RoPE is GPT-NeoX style (rotate halves, not interleaved pairs)
"""

from __future__ import annotations

import torch


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    dt = x.dtype
    xf = x.float()
    out = xf * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
    return (out * weight.float()).to(dt)


def fused_add_rmsnorm(x: torch.Tensor, residual: torch.Tensor,
                      weight: torch.Tensor, eps: float):
    """residual += x; return (rmsnorm(residual), residual)."""
    res = (residual.float() + x.float())
    out = res * torch.rsqrt(res.pow(2).mean(-1, keepdim=True) + eps)
    out = (out * weight.float()).to(x.dtype)
    return out, res.to(x.dtype)


def rope_cos_sin(positions: torch.Tensor, head_dim: int, theta: float,
                 dtype: torch.dtype = torch.float32) -> torch.Tensor:
    """Return [T, head_dim] table: first half cos, second half sin."""
    inv = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float32,
                                        device=positions.device) / head_dim))
    freqs = positions.float()[:, None] * inv[None, :]          # [T, D/2]
    return torch.cat([freqs.cos(), freqs.sin()], dim=-1).to(dtype)


def _rotate_neox(x: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor):
    # x: [T, H, D]; cos/sin: [T, D/2]
    d2 = x.shape[-1] // 2
    x1, x2 = x[..., :d2].float(), x[..., d2:].float()
    c, s = cos[:, None, :], sin[:, None, :]
    return torch.cat([x1 * c - x2 * s, x2 * c + x1 * s], dim=-1).to(x.dtype)


def apply_rope(q: torch.Tensor, k: torch.Tensor, positions: torch.Tensor,
               theta: float):
    """In-place-semantics RoPE on q [T,H,D] and k [T,KV,D]."""
    d = q.shape[-1]
    table = rope_cos_sin(positions, d, theta)
    cos, sin = table[:, : d // 2], table[:, d // 2:]
    return _rotate_neox(q, cos, sin), _rotate_neox(k, cos, sin)


def kv_cache_append(k: torch.Tensor, v: torch.Tensor,
                    k_cache: torch.Tensor, v_cache: torch.Tensor,
                    slot_mapping: torch.Tensor) -> None:
    """Scatter k/v [T, KV, D] into paged caches [NB, KV, BS, D]."""
    nb, kvh, bs, d = k_cache.shape
    blk = slot_mapping // bs
    off = slot_mapping % bs
    k_cache[blk, :, off] = k.to(k_cache.dtype)
    v_cache[blk, :, off] = v.to(v_cache.dtype)


def paged_attn_decode(q: torch.Tensor, k_cache: torch.Tensor,
                      v_cache: torch.Tensor, block_tables: torch.Tensor,
                      seq_lens: torch.Tensor, scale: float) -> torch.Tensor:
    """One-token-per-sequence attention over the paged cache.

    q: [B, H, D]; block_tables: [B, max_blocks] int32; seq_lens: [B] int32
    (length INCLUDING the current token, whose k/v are already in the cache).
    """
    B, H, D = q.shape
    nb, KV, BS, _ = k_cache.shape
    group = H // KV
    out = torch.empty_like(q)
    for b in range(B):
        n = int(seq_lens[b])
        nblk = (n + BS - 1) // BS
        blocks = block_tables[b, :nblk].long()
        k = k_cache[blocks].permute(1, 0, 2, 3).reshape(KV, nblk * BS, D)[:, :n]
        v = v_cache[blocks].permute(1, 0, 2, 3).reshape(KV, nblk * BS, D)[:, :n]
        qb = q[b].float().view(KV, group, D)                   # [KV, G, D]
        att = torch.einsum("kgd,knd->kgn", qb, k.float()) * scale
        p = att.softmax(-1)
        o = torch.einsum("kgn,knd->kgd", p, v.float())
        out[b] = o.reshape(H, D).to(q.dtype)
    return out


def prefill_attn_paged(q: torch.Tensor, k_cache: torch.Tensor,
                       v_cache: torch.Tensor, block_tables: torch.Tensor,
                       ctx_lens: torch.Tensor, row_seq: torch.Tensor,
                       scale: float) -> torch.Tensor:
    """Per-row causal attention over the paged cache (chunked-prefill
    continuation reference: row t attends slots 0..ctx_lens[t])."""
    T, H, D = q.shape
    nb, KV, BS, _ = k_cache.shape
    group = H // KV
    out = torch.empty_like(q)
    for t in range(T):
        si = int(row_seq[t])
        c = int(ctx_lens[t])
        nblk = (c + BS - 1) // BS
        blocks = block_tables[si, :nblk].long()
        k = k_cache[blocks].permute(1, 0, 2, 3).reshape(KV, nblk * BS,
                                                        D)[:, :c].float()
        v = v_cache[blocks].permute(1, 0, 2, 3).reshape(KV, nblk * BS,
                                                        D)[:, :c].float()
        qt = q[t].float().view(KV, group, D)
        att = torch.einsum("kgd,knd->kgn", qt, k) * scale
        p = att.softmax(-1)
        o = torch.einsum("kgn,knd->kgd", p, v)
        out[t] = o.reshape(H, D).to(q.dtype)
    return out


def prefill_attn(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                 seq_start: torch.Tensor, scale: float) -> torch.Tensor:
    """Varlen causal self-attention for prefill.

    q [T,H,D], k/v [T,KV,D]; seq_start: [num_seqs+1] int32 cumulative offsets.
    """
    T, H, D = q.shape
    KV = k.shape[1]
    group = H // KV
    out = torch.empty_like(q)
    for i in range(seq_start.numel() - 1):
        s, e = int(seq_start[i]), int(seq_start[i + 1])
        n = e - s
        qs = q[s:e].float().view(n, KV, group, D)
        ks = k[s:e].float()
        vs = v[s:e].float()
        att = torch.einsum("mkgd,nkd->kgmn", qs, ks) * scale
        mask = torch.full((n, n), float("-inf"), device=q.device).triu(1)
        att = att + mask
        p = att.softmax(-1)
        o = torch.einsum("kgmn,nkd->mkgd", p, vs)
        out[s:e] = o.reshape(n, H, D).to(q.dtype)
    return out


def silu_mul(gate_up: torch.Tensor) -> torch.Tensor:
    """SwiGLU activation: input [T, 2*I] (gate | up) -> [T, I]."""
    i = gate_up.shape[-1] // 2
    g, u = gate_up[..., :i].float(), gate_up[..., i:].float()
    return (torch.nn.functional.silu(g) * u).to(gate_up.dtype)


def sample(logits: torch.Tensor, temperature: torch.Tensor,
           top_p: torch.Tensor, top_k: torch.Tensor,
           uniform: torch.Tensor) -> torch.Tensor:
    """Per-row temperature / top-k / top-p sampling.

    logits [B, V] float; temperature/top_p [B] float; top_k [B] int
    (0 = off); uniform [B] in [0,1) drives the categorical draw so the HIP
    kernel and the reference are comparable given the same randoms.
    temperature == 0 selects greedy argmax for that row.
    """
    B, V = logits.shape
    out = torch.empty(B, dtype=torch.long, device=logits.device)
    lf = logits.float()
    for b in range(B):
        t = float(temperature[b])
        if t == 0.0:
            out[b] = int(lf[b].argmax())
            continue
        row = lf[b] / t
        k = int(top_k[b])
        if 0 < k < V:
            kth = row.topk(k).values[-1]
            row = row.masked_fill(row < kth, float("-inf"))
        probs = row.softmax(-1)
        p = float(top_p[b])
        if p < 1.0:
            sp, idx = probs.sort(descending=True)
            cum = sp.cumsum(-1)
            keep = cum - sp < p          # keep tokens until cumulative >= p
            sp = sp * keep
            sp = sp / sp.sum()
            # inverse-CDF draw on the sorted distribution
            c = sp.cumsum(-1)
            j = int(torch.searchsorted(c, uniform[b].to(c.dtype), right=False).clamp(max=V - 1))
            out[b] = int(idx[j])
        else:
            c = probs.cumsum(-1)
            j = int(torch.searchsorted(c, uniform[b].to(c.dtype), right=False).clamp(max=V - 1))
            out[b] = j
    return out


def moe_route(hidden: torch.Tensor, router_w: torch.Tensor, top_k: int):
    """Softmax-topk routing: returns (weights [T,K], expert_ids [T,K])."""
    logits = hidden.float() @ router_w.float().t()
    probs = logits.softmax(-1)
    w, ids = probs.topk(top_k, dim=-1)
    w = w / w.sum(-1, keepdim=True)
    return w, ids


# ---------------------------------------------------------------------------
# Hybrid designs: dynamic-tanh norm, interleaved rotary, windowed differential
# attention over transposed-V pages, recurrent layers with a state pool.
# ---------------------------------------------------------------------------

def dyt(x: torch.Tensor, norm) -> torch.Tensor:
    """norm = (w, b, alpha), all float; computed and returned in float."""
    w, b, alpha = norm
    return torch.tanh(alpha * x.float()) * w + b


def gelu_mul(gate_up: torch.Tensor) -> torch.Tensor:
    i = gate_up.shape[-1] // 2
    g = torch.nn.functional.gelu(gate_up[..., :i].float(), approximate="tanh")
    return (g * gate_up[..., i:].float()).to(gate_up.dtype)


def rope_pairs_append(q, k, v, positions, freqs, slot_mapping, k_cache,
                      v_cache, head_dim: int) -> None:
    """Rotate q [T, n*D] in place; append rotated k and transposed v."""
    T, (_, G, BS, MD) = q.shape[0], k_cache.shape
    a = positions.double()[:, None] * freqs[None, :]
    c, s = a.cos().float()[:, None, :], a.sin().float()[:, None, :]
    r = 2 * freqs.numel()

    def rotate(x):
        x = x.reshape(T, -1, head_dim).float()
        u, w = x[..., 0:r:2], x[..., 1:r:2]
        y = x.clone()
        y[..., 0:r:2] = u * c - w * s
        y[..., 1:r:2] = w * c + u * s
        return y.reshape(T, -1)

    q.copy_(rotate(q))
    ok = slot_mapping >= 0
    blk, off = slot_mapping[ok] // BS, slot_mapping[ok] % BS
    k_cache[blk, :, off] = rotate(k)[ok].view(-1, G, MD).to(k_cache.dtype)
    v_cache[blk, :, :, off] = v[ok].reshape(int(ok.sum()), G, -1)


def window_diff_attention(q, k_cache, v_cache, block_tables, positions,
                          row_seq, lam, window: int, scale: float,
                          diff: float, eps: float) -> torch.Tensor:
    T = q.shape[0]
    _, G, BS, MD = k_cache.shape
    D, E = MD // 2, v_cache.shape[2]
    H = q.shape[1] // MD
    lq1, lk1, lq2, lk2 = lam.float()
    lambda_ = ((lq1 * lk1).sum().exp() - (lq2 * lk2).sum().exp() + diff)
    out = torch.empty(T, H * E, dtype=q.dtype, device=q.device)
    for t in range(T):
        s = int(row_seq[t]) if row_seq is not None else t
        p = int(positions[t])
        lo = max(0, p - window + 1)
        idx = torch.arange(lo, p + 1, device=q.device)
        blk, off = block_tables[s][idx // BS].long(), idx % BS
        k = k_cache[blk, :, off].float().view(-1, G, 2, D)
        v = v_cache[blk, :, :, off].float()                    # [n, G, E]
        qt = q[t].float().view(G, H // G, 2, D)
        att = torch.einsum("gxmd,ngmd->gxmn", qt, k) * scale
        o = torch.einsum("gxmn,nge->gxme", att.softmax(-1), v)
        o = o[:, :, 0] - lambda_ * o[:, :, 1]
        o = o / (o.pow(2).mean(-1, keepdim=True) + eps).sqrt() * (1 - diff)
        out[t] = o.reshape(-1).to(q.dtype)
    return out


def gla_log_decay(a1h, a2, a2b, tau: float) -> torch.Tensor:
    z = a1h.float() @ a2.float().t() + a2b
    return torch.nn.functional.logsigmoid(z) / tau


def mlstm_log_gates(raw, ib, fb, cap: float):
    H = ib.numel()
    i = cap * torch.tanh((raw[:, :H] + ib) / cap)
    f = torch.nn.functional.logsigmoid(
        cap * torch.tanh((raw[:, H:] + fb) / cap))
    return i, f


def _sequences(seq_start, slots, positions):
    """(first row, end row, slot, starts from zero) of every sequence; without
    seq_start each row is a sequence of its own (decode)."""
    n = slots.numel()
    ss = seq_start.tolist() if seq_start is not None else list(range(n + 1))
    for i in range(n):
        a, b, slot = int(ss[i]), int(ss[i + 1]), int(slots[i])
        if b > a:
            yield a, b, slot, slot < 0 or int(positions[a]) == 0


def gla_scan(q, k, v, log_decay, state, seq_start, slots, positions,
             qscale: float) -> torch.Tensor:
    """Unnormalised o [T, H, E] float; the state pool is updated."""
    _, H, D, E = state.S.shape
    T = q.shape[0]
    qf = q.float().reshape(T, H, D) * qscale
    kf, vf = k.float().reshape(T, H, D), v.float().reshape(T, H, E)
    a = log_decay.view(T, H, D).exp()
    o = torch.zeros(T, H, E, device=q.device)
    for t0, t1, slot, fresh in _sequences(seq_start, slots, positions):
        S = torch.zeros(H, D, E, device=q.device) if fresh \
            else state.S[slot].clone()
        for t in range(t0, t1):
            S = S * a[t][:, :, None] + kf[t][:, :, None] * vf[t][:, None, :]
            o[t] = (S * qf[t][:, :, None]).sum(1)
        if slot >= 0:
            state.S[slot] = S
    return o


def mlstm_scan(q, k, v, log_i, log_f, state, seq_start, slots, positions,
               qscale: float) -> torch.Tensor:
    _, H, D, E = state.S.shape
    T = q.shape[0]
    qf = q.float().reshape(T, H, D) * qscale
    kf, vf = k.float().reshape(T, H, D), v.float().reshape(T, H, E)
    o = torch.zeros(T, H, E, device=q.device)
    for t0, t1, slot, fresh in _sequences(seq_start, slots, positions):
        if fresh:
            S = torch.zeros(H, D, E, device=q.device)
            n = torch.zeros(H, D, device=q.device)
            m = torch.zeros(H, device=q.device)
        else:
            S, n, m = (x[slot].clone() for x in state)
        for t in range(t0, t1):
            m_new = torch.maximum(log_f[t] + m, log_i[t])
            fs = (log_f[t] + m - m_new).exp()
            ki = kf[t] * (log_i[t] - m_new).exp()[:, None]
            S = S * fs[:, None, None] + ki[:, :, None] * vf[t][:, None, :]
            n = n * fs[:, None] + ki
            m = m_new
            den = torch.maximum((n * qf[t]).sum(-1).abs(), (-m).exp()) + 1e-6
            o[t] = (S * qf[t][:, :, None]).sum(1) / den[:, None]
        if slot >= 0:
            state.S[slot], state.n[slot], state.m[slot] = S, n, m
    return o


def recurrent_out(o, g, w, gate: str, eps: float, dtype) -> torch.Tensor:
    """Per-head RMS norm, weight ([E] shared or [H*E]) and output gate."""
    T, H, E = o.shape
    y = o / (o.pow(2).mean(-1, keepdim=True) + eps).sqrt()
    y = y * w.view(-1, E)
    gf = g.float()
    gf = torch.sigmoid(gf) if gate == "sigmoid" \
        else torch.nn.functional.silu(gf)
    return (y.reshape(T, H * E) * gf).to(dtype)


# ---------------------------------------------------------------------------
# RMS-normed float residual, latent attention, lightning attention, experts
# ---------------------------------------------------------------------------

def rms_scale(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """Computed and returned in float."""
    x = x.float()
    return x / (x.pow(2).mean(-1, keepdim=True) + eps).sqrt() * w


def latent_rope_append(q, kv, w, positions, freqs, slot_mapping, cache,
                       heads: int, rank: int, eps: float,
                       gain: float = 1.0) -> None:
    """Rotate the last part of each head of q [T, H*(D+R)] in place; append
    the normed latent and the rotated key part of kv [T, rank + R]."""
    T, R = q.shape[0], 2 * freqs.numel()
    if R:
        a = positions.double()[:, None] * freqs[None, :]
        c, s = (gain * a.cos()).float()[:, None, :], \
            (gain * a.sin()).float()[:, None, :]

    def rotate(x):                                  # [T, n, R]
        if not R:
            return x
        x = x.float()
        u, v = x[..., 0::2], x[..., 1::2]
        return torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)

    qh = q.unflatten(-1, (heads, -1))
    D = qh.shape[-1] - R
    qh[..., D:] = rotate(qh[..., D:]).to(q.dtype)
    if kv is None:
        return
    row = torch.cat([rms_scale(kv[:, :rank], w, eps),
                     rotate(kv[:, None, rank:])[:, 0]], -1).to(cache.dtype)
    ok = slot_mapping >= 0
    cache.view(-1, cache.shape[-1])[slot_mapping[ok]] = row[ok]


def softmax_with_sink(s, sink):
    """Softmax over the last axis; `sink` broadcasts against the rest and adds
    exp(sink) to the denominator (None: a plain softmax)."""
    if sink is None:
        return s.softmax(-1)
    both = torch.cat([s, sink.expand(s.shape[:-1])[..., None]], -1)
    return both.softmax(-1)[..., :-1]


def latent_attention(q, cache, block_tables, positions, row_seq, uk, uv,
                     heads: int, window: int, scale: float, sink=None,
                     gate=None) -> torch.Tensor:
    """q [T, H*(D+R)] rotated; uk [rank, H*D], uv [H*E, rank]; sink [H], gate
    [T, H] before its sigmoid."""
    T, BS, rank = q.shape[0], cache.shape[1], uk.shape[0]
    D, E = uk.shape[1] // heads, uv.shape[0] // heads
    qh = q.float().view(T, heads, -1)
    # queries in latent coordinates: one row per head against the cache
    qa = torch.cat([torch.einsum("thd,rhd->thr", qh[..., :D],
                                 uk.float().view(rank, heads, D)),
                    qh[..., D:]], -1)
    o = torch.empty(T, heads, rank, device=q.device)
    for t in range(T):
        s = int(row_seq[t]) if row_seq is not None else t
        p = int(positions[t])
        idx = torch.arange(max(0, p - window + 1), p + 1, device=q.device)
        rows = cache[block_tables[s][idx // BS].long(), idx % BS].float()
        att = softmax_with_sink(qa[t] @ rows.t() * scale, sink)
        o[t] = att @ rows[:, :rank]
    out = torch.einsum("thr,her->the", o, uv.float().view(heads, E, rank))
    if gate is not None:
        out = out * torch.sigmoid(gate.float())[:, :, None]
    return out.reshape(T, heads * E).to(q.dtype)


def lightning_scan(q, k, v, decay, state, seq_start, slots,
                   positions) -> torch.Tensor:
    """o [T, H, E] float; SiLU is applied to q, k and v here; the state pool
    is updated."""
    _, H, D, E = state.S.shape
    T = q.shape[0]
    silu = torch.nn.functional.silu
    qf, kf = (silu(x.float()).reshape(T, H, D) for x in (q, k))
    vf = silu(v.float()).reshape(T, H, E)
    o = torch.zeros(T, H, E, device=q.device)
    for t0, t1, slot, fresh in _sequences(seq_start, slots, positions):
        S = torch.zeros(H, D, E, device=q.device) if fresh \
            else state.S[slot].clone()
        for t in range(t0, t1):
            S = S * decay[:, None, None] \
                + kf[t][:, :, None] * vf[t][:, None, :]
            o[t] = (S * qf[t][:, :, None]).sum(1)
        if slot >= 0:
            state.S[slot] = S
    return o


def clamped_glu(gate_up: torch.Tensor, limit: float) -> torch.Tensor:
    """g sigmoid(1.702 g) (u + 1) of a merged [gate | up] projection, with
    g = min(gate, limit) and u = up clamped to +-limit."""
    g, u = gate_up.float().chunk(2, -1)
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)).to(gate_up.dtype)


def mixture(x, router, up, down, shared_up, shared_down, top: int,
            rules=(None, 0, None, True)):
    """[T, W] float: chosen experts under their weights, plus the shared
    expert under its sigmoid gate; `rules` as in ops.experts."""
    correction, identity, limit, identity_here = rules
    E = up.shape[0]
    n = E + identity
    z = x.float() @ router.float().t()
    if correction is None:
        s, ids = z[:, :n].topk(top, dim=-1)
        weight = s.softmax(-1)
    else:
        s = z[:, :n].softmax(-1)
        ids = (s + correction).topk(top, dim=-1).indices
        weight = s.gather(1, ids)

    def expert(h, up, down):
        y = h @ up.t()
        y = silu_mul(y) if limit is None else clamped_glu(y, limit)
        return (y @ down.t()).float()

    out = x.float() * (weight * (ids >= E)).sum(-1, keepdim=True) \
        * identity_here
    for e in range(E):
        t, j = (ids == e).nonzero(as_tuple=True)
        if t.numel():
            out.index_add_(0, t, weight[t, j][:, None]
                           * expert(x[t], up[e], down[e]))
    if shared_up is not None:
        out += torch.sigmoid(z[:, n:]) * expert(x, shared_up[0],
                                                shared_down[0])
    return out


# ---------------------------------------------------------------------------
# Convolved sublayer inputs, chunked sigmoid attention
# ---------------------------------------------------------------------------

def causal_conv(h, w, tail, seq_start, slots, positions) -> torch.Tensor:
    """h [T, W] plus its convolution over time; w [taps, W] float with the
    token's own tap last; tail [slots, taps - 1, W] is read and renewed."""
    taps = w.shape[0]
    out = torch.empty_like(h)
    for a, b, slot, fresh in _sequences(seq_start, slots, positions):
        past = torch.zeros(taps - 1, h.shape[1], dtype=h.dtype,
                           device=h.device) if fresh else tail[slot]
        x = torch.cat([past, h[a:b]])
        y = h[a:b].float()
        for j in range(taps):
            y = y + w[j] * x[j:j + b - a].float()
        out[a:b] = y.to(h.dtype)
        if slot >= 0:
            tail[slot] = x[b - a:]
    return out


def norm_append(q, k, v, qw, kw, slot_mapping, k_cache, v_cache,
                eps: float) -> None:
    """RMS norm of every head of q [T, H*D] in place; append normed k and
    transposed v."""
    _, G, BS, D = k_cache.shape
    norm = lambda x, w: rms_scale(x.unflatten(-1, (-1, D)), w, eps).flatten(1)
    q.copy_(norm(q, qw))
    ok = slot_mapping >= 0
    blk, off = slot_mapping[ok] // BS, slot_mapping[ok] % BS
    k_cache[blk, :, off] = norm(k, kw)[ok].view(-1, G, D).to(k_cache.dtype)
    v_cache[blk, :, :, off] = v[ok].reshape(int(ok.sum()), G, -1)


def sigmoid_attention(q, k_cache, v_cache, block_tables, positions, row_seq,
                      bias, chunk: int, scale: float, cap: float):
    T = q.shape[0]
    _, G, BS, D = k_cache.shape
    H = q.shape[1] // D
    out = torch.empty(T, H * v_cache.shape[2], dtype=q.dtype, device=q.device)
    for t in range(T):
        s = int(row_seq[t]) if row_seq is not None else t
        p = int(positions[t])
        idx = torch.arange(p // chunk * chunk, p + 1, device=q.device)
        blk, off = block_tables[s][idx // BS].long(), idx % BS
        k = k_cache[blk, :, off].float()                       # [n, G, D]
        v = v_cache[blk, :, :, off].float()                    # [n, G, E]
        z = torch.einsum("gxd,ngd->gxn", q[t].float().view(G, H // G, D), k)
        z = cap * torch.tanh(z * scale / cap) + bias.view(G, H // G, 1)
        out[t] = torch.einsum("gxn,nge->gxe", z.sigmoid(),
                              v).reshape(-1).to(q.dtype)
    return out


# ---------------------------------------------------------------------------
# Windowed attention with kept first tokens, sinks and turned values
# ---------------------------------------------------------------------------

def turn_pairs(x, positions, freqs, gain: float = 1.0) -> torch.Tensor:
    """x [T, n, D] float with the neighbouring pairs of the first
    2 * len(freqs) dimensions turned by position times frequency."""
    a = positions.double()[:, None] * freqs[None, :]
    c, s = (gain * a.cos()).float()[:, None], (gain * a.sin()).float()[:, None]
    r = 2 * freqs.numel()
    u, v = x[..., 0:r:2], x[..., 1:r:2]
    return torch.cat([torch.stack([u * c - v * s, v * c + u * s], -1)
                      .flatten(-2), x[..., r:]], -1)


def rope_norm_append(q, k, v, positions, freqs, turn, slot_mapping, k_cache,
                     v_cache, gain: float, eps) -> None:
    T, (_, G, BS, D) = q.shape[0], k_cache.shape

    def heads(x):
        x = turn_pairs(x.float().unflatten(-1, (-1, D)), positions, freqs,
                       gain)
        return x if eps is None else rms_scale(x, 1.0, eps)

    q.copy_(heads(q).flatten(1))
    ok = slot_mapping >= 0
    blk, off = slot_mapping[ok] // BS, slot_mapping[ok] % BS
    k_cache[blk, :, off] = heads(k)[ok].to(k_cache.dtype)
    v = turn_pairs(v.float().unflatten(-1, (G, -1)), positions, turn)
    v_cache[blk, :, :, off] = v[ok].to(v_cache.dtype)


def window_attention(out, q, k_cache, v_cache, block_tables, positions,
                     row_seq, turn, sink, window: int, keep: int,
                     scale: float) -> None:
    T = q.shape[0]
    _, G, BS, D = k_cache.shape
    H, E = q.shape[1] // D, v_cache.shape[2]
    o = torch.empty(T, H, E, device=q.device)
    if sink is not None:
        sink = sink.view(G, H // G)
    for t in range(T):
        s = int(row_seq[t]) if row_seq is not None else t
        p = int(positions[t])
        lo = max(0, p - window + 1)
        idx = torch.cat([torch.arange(min(keep, lo), device=q.device),
                         torch.arange(lo, p + 1, device=q.device)])
        blk, off = block_tables[s][idx // BS].long(), idx % BS
        k = k_cache[blk, :, off].float()                       # [n, G, D]
        v = v_cache[blk, :, :, off].float()                    # [n, G, E]
        z = torch.einsum("gxd,ngd->gxn", q[t].float().view(G, H // G, D), k)
        o[t] = torch.einsum("gxn,nge->gxe", softmax_with_sink(z * scale, sink),
                            v).reshape(H, E)
    out.copy_(turn_pairs(o, -positions, turn).flatten(1))
