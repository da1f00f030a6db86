#!/usr/bin/env python3
"""Isolated kernel microbenchmarks (GPU only) — us/call + achieved GB/s.

Usage: python bench_kernels.py [--iters N]
           [--which attn|gemm|fp8|hybrid|latent|sigmoid|kept|all]

Shapes mirror the flagship bench (Llama-3-8B bf16, bs=256 ctx=512 decode):
the numbers here are the per-kernel budget lines behind bench.py's step
time, compared against the HBM3E stream roofline (~8 TB/s).
"""

from __future__ import annotations

import argparse
import json

import torch


def timed(fn, iters, warmup=20):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    s = torch.cuda.Event(enable_timing=True)
    e = torch.cuda.Event(enable_timing=True)
    s.record()
    for _ in range(iters):
        fn()
    e.record()
    torch.cuda.synchronize()
    return s.elapsed_time(e) * 1e3 / iters  # us/call


def bench_attn(iters):
    import hyperspot.ops as ops
    from hyperspot.ops import torch_ref
    torch.manual_seed(0)
    dev = "cuda:0"
    for (bs, ctx, kvh, group, D) in [(256, 512, 8, 4, 128),
                                     (256, 2048, 8, 4, 128),
                                     (64, 512, 8, 4, 128),
                                     (256, 512, 1, 8, 128),
                                     (64, 8192, 8, 4, 128),
                                     (16, 32768, 8, 4, 128)]:
        BS = 16
        nblk = (ctx + BS - 1) // BS
        tot_blocks = bs * nblk + 7
        k_cache = torch.randn(tot_blocks, kvh, BS, D, dtype=torch.bfloat16,
                              device=dev) * 0.3
        v_cache = torch.randn_like(k_cache) * 0.3
        q = torch.randn(bs, kvh * group, D, dtype=torch.bfloat16,
                        device=dev) * 0.5
        perm = torch.randperm(bs * nblk, device=dev, dtype=torch.int32)
        block_tables = perm.view(bs, nblk).contiguous()
        seq_lens = torch.full((bs,), ctx, dtype=torch.int32, device=dev)
        scale = D ** -0.5

        out = ops.paged_attn_decode(q, k_cache, v_cache, block_tables,
                                    seq_lens, scale)
        ref = torch_ref.paged_attn_decode(
            q.float().cpu(), k_cache.float().cpu(), v_cache.float().cpu(),
            block_tables.cpu(), seq_lens.cpu(), scale)
        err = (out.float().cpu() - ref).abs().max().item()
        us = timed(lambda: ops.paged_attn_decode(
            q, k_cache, v_cache, block_tables, seq_lens, scale), iters)
        kv_bytes = bs * ctx * kvh * D * 2 * 2
        roof_us = kv_bytes / 8e12 * 1e6
        print(json.dumps({
            "kernel": "paged_attn_decode",
            "shape": f"bs{bs}_ctx{ctx}_kvh{kvh}_g{group}_d{D}",
            "us": round(us, 1), "GBps": round(kv_bytes / us / 1e3, 0),
            "roofline_us": round(roof_us, 1),
            "x_roofline": round(us / roof_us, 2),
            "max_abs_err": round(err, 5)}), flush=True)


def bench_gemm(iters):
    dev = "cuda:0"
    for (m, k, n, tag) in [(256, 4096, 6144, "qkv"),
                           (256, 4096, 4096, "o"),
                           (256, 4096, 28672, "gate_up"),
                           (256, 14336, 4096, "down"),
                           (64, 4096, 6144, "qkv_bs64"),
                           (8192, 4096, 28672, "prefill_gate_up")]:
        x = torch.randn(m, k, dtype=torch.bfloat16, device=dev)
        w = torch.randn(n, k, dtype=torch.bfloat16, device=dev)
        us = timed(lambda: torch.nn.functional.linear(x, w), iters)
        bytes_ = (m * k + n * k + m * n) * 2
        flops = 2 * m * k * n
        print(json.dumps({
            "kernel": f"linear_{tag}", "shape": f"{m}x{k}x{n}",
            "us": round(us, 1),
            "GBps": round(bytes_ / us / 1e3, 0),
            "TFs": round(flops / us / 1e6, 0),
            "roofline_us": round(max(bytes_ / 8e12, flops / 2.5e15) * 1e6,
                                 1)}), flush=True)


def bench_fp8_gemm(iters):
    from hyperspot.parallel.layers import quant_fp8_rowwise, quantize_weight_fp8
    dev = "cuda:0"
    for (m, k, n, tag) in [(1024, 4096, 6144, "qkv"),
                           (1024, 4096, 28672, "gate_up"),
                           (1024, 14336, 4096, "down"),
                           (256, 4096, 28672, "gate_up_bs256")]:
        x = torch.randn(m, k, dtype=torch.bfloat16, device=dev)
        w = torch.randn(n, k, dtype=torch.bfloat16, device=dev) * 0.02
        wq, ws = quantize_weight_fp8(w)
        ws_row = ws[None, :].contiguous()
        us_bf16 = timed(lambda: torch.nn.functional.linear(x, w), iters)

        def fp8_full():
            xq, xs = quant_fp8_rowwise(x)
            return torch._scaled_mm(xq, wq.t(), scale_a=xs[:, None],
                                    scale_b=ws_row, out_dtype=torch.bfloat16)
        us_fp8 = timed(fp8_full, iters)
        xq, xs = quant_fp8_rowwise(x)
        xs_col = xs[:, None].contiguous()
        us_fp8_mm = timed(lambda: torch._scaled_mm(
            xq, wq.t(), scale_a=xs_col, scale_b=ws_row,
            out_dtype=torch.bfloat16), iters)
        print(json.dumps({
            "kernel": f"fp8_{tag}", "shape": f"{m}x{k}x{n}",
            "us_bf16": round(us_bf16, 1), "us_fp8_withquant": round(us_fp8, 1),
            "us_fp8_mm_only": round(us_fp8_mm, 1)}), flush=True)


DEV = "cuda:0"


def timed_graph(fn, iters, calls=10):
    """us/call inside a replayed graph: no host time between the kernels."""
    fn()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        for _ in range(calls):
            fn()
    return timed(g.replay, max(1, iters // calls), warmup=3) / calls


def report_kernel(iters, name, shape, fn, nbytes, flops=0, timer=timed):
    """Time against the larger of the HBM floor (8 TB/s) and the bf16 matrix
    floor (2.5 PFLOP/s)."""
    us = timer(fn, iters)
    roof = max(nbytes / 8e12, flops / 2.5e15) * 1e6
    print(json.dumps({"kernel": name, "shape": shape, "us": round(us, 1),
                      "roofline_us": round(roof, 2),
                      "x_roofline": round(us / roof, 2)}), flush=True)


def meta_for(lens, mode="prefill", ctx=0):
    """(metadata, pages) of portions of these lengths after ctx tokens."""
    from hyperspot.models.llama import ForwardMeta, prefill_tiles
    n = len(lens)
    starts = [0]
    for x in lens:
        starts.append(starts[-1] + x)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)
    pos = [ctx + p for x in lens for p in range(x)]
    nblk = (max(lens) + ctx + 15) // 16
    tiles, ts = prefill_tiles(lens)
    bt = torch.randperm(n * nblk, device=DEV).int().view(n, nblk)
    p = torch.tensor(pos, device=DEV)
    seq = torch.tensor([i for i, x in enumerate(lens) for _ in range(x)],
                       device=DEV)
    slots = bt[seq, p // 16].long() * 16 + p % 16
    return ForwardMeta(
        mode=mode, positions=p, slot_mapping=slots, seq_start=i32(starts),
        max_seqlen=max(lens), row_seq=seq.int(), ctx_lens=(p + 1).int(),
        block_tables=bt, seq_lens=(p + 1).int(),
        state_slots=i32(list(range(n))), tiles=i32(tiles),
        tile_start=i32(ts)), n * nblk


def bench_hybrid(iters):
    """Kernels of the hybrid design and the like kernels of the plain decoder
    at width 4096: time against the larger of the HBM floor (8 TB/s) and the
    bf16 matrix floor (2.5 PFLOP/s)."""
    import hyperspot.ops as ops
    from hyperspot.engine.kv_cache import KVPages, RecurrentState
    from hyperspot.ops import hybrid
    dev, bf = "cuda:0", torch.bfloat16
    dev, bf = DEV, torch.bfloat16
    report = lambda *a: report_kernel(iters, *a)

    W, H, G, D, E, win = 4096, 32, 8, 64, 128, 1024
    HS = 16                                     # recurrent heads
    rnd = lambda *s, d=bf: (torch.randn(*s, device=dev) * 0.3).to(d)
    norm = (torch.ones(W, device=dev), torch.zeros(W, device=dev),
            torch.full((1,), 0.5, device=dev))
    for lens in ([2048], [8192], [1024] * 8):
        m, nb = meta_for(lens)
        T, tag = sum(lens), "x".join(map(str, (len(lens), lens[0])))
        # windowed differential attention
        qkv = rnd(T, H * 2 * D + G * 2 * D + G * E)
        q, k, v = qkv.split([H * 2 * D, G * 2 * D, G * E], -1)
        cache = KVPages(torch.zeros(nb, G, 16, 2 * D, dtype=bf, device=dev),
                        torch.zeros(nb, G, E, 16, dtype=bf, device=dev))
        fr = 1e5 ** (-torch.arange(0, 32, 2, device=dev).double() / 32)
        io = 2 * T * (H * (2 * D + E) + G * (2 * D + E))
        report("rope_pairs_append", tag, lambda: hybrid.rope_pairs_append(
            q, k, v, m, fr, cache, D),
            2 * T * (2 * H * 32 * 2 + 2 * G * (2 * D + E)))
        lam = rnd(4, D, d=torch.float32)
        pairs = sum(min(p + 1, win) for x in lens for p in range(x))
        report("window_attn_prefill", tag,
               lambda: hybrid.window_diff_attention(
                   q, cache, m, lam, win, 0.125, 0.4, 1e-5),
               io, pairs * H * 2 * 2 * (D + E))
        # plain causal attention of the closest model (head size 128)
        qkv2 = rnd(T, (H + 2 * G) * 128)
        q2, k2, v2 = (x.view(T, -1, 128) for x in qkv2.split(
            [H * 128, G * 128, G * 128], -1))
        kc = torch.zeros(2, nb, G, 16, 128, dtype=bf, device=dev)
        cs = torch.randn(max(lens), 128, device=dev)
        report("rope_kv_append", tag, lambda: ops.rope_kv_append(
            q2, k2, v2, m.positions, cs, m.slot_mapping, kc[0], kc[1]),
            2 * T * 128 * (2 * H + 4 * G))
        pairs2 = sum(x * (x + 1) // 2 for x in lens)
        report("attn_prefill_mfma", tag, lambda: ops.attention(
            q2, k2, v2, kc[0], kc[1], m, 0.088),
            2 * T * 128 * (2 * H + 2 * G), pairs2 * H * 4 * 128)
        # recurrent layers
        d, e, R = HS * D, HS * E, 24
        pr = rnd(T, 2 * d + 2 * e + R)
        gq, gk, gv, gg, ga = pr.split([d, d, e, e, R], -1)
        a2, a2b = rnd(d, R), torch.zeros(d, device=dev)
        st = RecurrentState(torch.zeros(len(lens), HS, D, E, device=dev))
        wn = torch.ones(E, device=dev)
        # the state and its per-tile copies are the kernel's own traffic; the
        # floor counts what the layer must read and write
        fl = T * HS * 2 * (2 * D * E + 32 * (D + E))
        report("gla_prefill", tag, lambda: hybrid.gla_mix(
            gq, gk, gv, gg, ga, a2, a2b, wn, st, m, 8.0, 1e-5),
            2 * T * (2 * d + 3 * e + R), fl)
        pr2 = rnd(T, 2 * d + 2 * e)
        lq, lk, lv, lg = pr2.split([d, d, e, e], -1)
        raw, hb = rnd(T, 2 * HS, d=torch.float32), torch.zeros(HS, device=dev)
        ls = RecurrentState(st.S.clone(),
                            torch.zeros(len(lens), HS, D, device=dev),
                            torch.zeros(len(lens), HS, device=dev))
        wl = torch.ones(e, device=dev)
        report("mlstm_prefill", tag, lambda: hybrid.mlstm_mix(
            lq, lk, lv, lg, raw, hb, hb, wl, ls, m, 15.0, 1e-5),
            2 * T * (2 * d + 3 * e), fl)
        x, r = rnd(T, W), rnd(T, W, d=torch.float32)
        report("add_dyt", tag, lambda: hybrid.add_dyt(x, r, norm, norm),
               T * W * 12)
        x2, r2, w2 = rnd(T, W), rnd(T, W), torch.ones(W, dtype=bf, device=dev)
        report("fused_add_rmsnorm", tag, lambda: ops.fused_add_rmsnorm(
            x2, r2, w2, 1e-5), T * W * 8)
        gu = rnd(T, 2 * 14336)
        report("gelu_mul", tag, lambda: hybrid.gelu_mul(gu), T * 14336 * 6)
        report("silu_mul", tag, lambda: ops.silu_mul(gu), T * 14336 * 6)
    for B in (1, 32, 256):
        ctx = 1024
        m, nb = meta_for([1] * B, "decode", ctx)
        tag = f"b{B}_ctx{ctx}"
        qkv = rnd(B, H * 2 * D + G * 2 * D + G * E)
        q, k, v = qkv.split([H * 2 * D, G * 2 * D, G * E], -1)
        cache = KVPages(rnd(nb, G, 16, 2 * D), rnd(nb, G, E, 16))
        report("rope_pairs_append", tag, lambda: hybrid.rope_pairs_append(
            q, k, v, m, fr, cache, D),
            2 * B * (2 * H * 32 * 2 + 2 * G * (2 * D + E)))
        report("window_attn_decode", tag,
               lambda: hybrid.window_diff_attention(
                   q, cache, m, lam, win, 0.125, 0.4, 1e-5),
               2 * B * min(ctx + 1, win) * G * (2 * D + E))
        qkv2 = rnd(B, (H + 2 * G) * 128)
        q2, k2, v2 = (x.view(B, -1, 128) for x in qkv2.split(
            [H * 128, G * 128, G * 128], -1))
        kc = rnd(2, nb, G, 16, 128)
        cs = torch.randn(ctx + 1, 128, device=dev)
        report("rope_kv_append", tag, lambda: ops.rope_kv_append(
            q2, k2, v2, m.positions, cs, m.slot_mapping, kc[0], kc[1]),
            2 * B * 128 * (2 * H + 4 * G))
        report("paged_attn_decode", tag, lambda: ops.paged_attn_decode(
            q2, kc[0], kc[1], m.block_tables, m.seq_lens, 0.088),
            4 * B * (ctx + 1) * G * 128)
        d, e, R = HS * D, HS * E, 24
        pr = rnd(B, 2 * d + 2 * e + R)
        gq, gk, gv, gg, ga = pr.split([d, d, e, e, R], -1)
        a2, a2b = rnd(d, R), torch.zeros(d, device=dev)
        st = RecurrentState(torch.zeros(B, HS, D, E, device=dev))
        report("gla_step", tag, lambda: hybrid.gla_mix(
            gq, gk, gv, gg, ga, a2, a2b, wn, st, m, 8.0, 1e-5), B * HS * D * E * 8)
        pr2 = rnd(B, 2 * d + 2 * e)
        lq, lk, lv, lg = pr2.split([d, d, e, e], -1)
        raw, hb = rnd(B, 2 * HS, d=torch.float32), torch.zeros(HS, device=dev)
        ls = RecurrentState(st.S.clone(), torch.zeros(B, HS, D, device=dev),
                            torch.zeros(B, HS, device=dev))
        wl = torch.ones(e, device=dev)
        report("mlstm_step", tag, lambda: hybrid.mlstm_mix(
            lq, lk, lv, lg, raw, hb, hb, wl, ls, m, 15.0, 1e-5),
            B * HS * D * E * 8)
        x, r = rnd(B, W), rnd(B, W, d=torch.float32)
        report("add_dyt", tag, lambda: hybrid.add_dyt(x, r, norm, norm),
               B * W * 12)
        x2, r2, w2 = rnd(B, W), rnd(B, W), torch.ones(W, dtype=bf, device=dev)
        report("fused_add_rmsnorm", tag, lambda: ops.fused_add_rmsnorm(
            x2, r2, w2, 1e-5), B * W * 8)
        gu = rnd(B, 2 * 14336)
        report("gelu_mul", tag, lambda: hybrid.gelu_mul(gu), B * 14336 * 6)
        report("silu_mul", tag, lambda: ops.silu_mul(gu), B * 14336 * 6)


def bench_latent(iters, W):
    """Kernels of the Tefezen design at width W and the like kernels of the
    Mixtral-like model."""
    import hyperspot.ops as ops
    from hyperspot.engine.kv_cache import LatentKV, RecurrentState
    from hyperspot.models.llama import (SPAN_TOKENS, LatentSpan,
                                        prefill_tiles)
    from hyperspot.ops import experts, hybrid, latent
    dev, bf, f32 = DEV, torch.bfloat16, torch.float32
    n_ = ops._native()
    report = lambda name, tag, fn, nbytes, flops=0: report_kernel(
        iters, name, f"w{W}_{tag}", fn, nbytes, flops, timed_graph)
    rnd = lambda *s, d=bf: (torch.randn(*s, device=dev) * 0.3).to(d)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)
    H, D, R, E, rank, win = W // 128, 128, 64, 128, 512, 1024
    G, NE, top, F, side = H // 4, 65536 // W, 4, W // 2, 128
    uk, uv, kw = rnd(rank, H * D), rnd(H * E, rank), rnd(rank, d=f32)
    fr = 1e4 ** (-torch.arange(0, R, 2, device=dev).double() / R)
    decay = torch.linspace(0.5, 0.999, H, device=dev)
    up, down = rnd(NE, 2 * F, W) * 0.1, rnd(NE, W, F) * 0.1
    su, sd, router = rnd(1, 2 * F, W), rnd(1, W, F), rnd(NE + 1, W)
    nw, table = torch.ones(W, device=dev), rnd(1000, side)
    w2 = torch.ones(W, dtype=bf, device=dev)

    def common(T, tag):
        x, r = rnd(T, W), rnd(T, W, d=f32)
        report("add_rms", tag, lambda: hybrid.add_rms(x, r, nw, 1e-5, bf),
               T * W * 12)
        r2 = rnd(T, W)
        report("fused_add_rmsnorm", tag, lambda: ops.fused_add_rmsnorm(
            x, r2, w2, 1e-5), T * W * 8)
        o, g = rnd(T, W, d=f32), rnd(T, W)
        report("rms_gate", tag, lambda: hybrid.rms_gate(
            o, g, nw, 1e-5, None, W), T * W * 8)
        z, ids = rnd(T, side), torch.randint(0, 1000, (T,), device=dev)
        report("gelu_gate", tag, lambda: hybrid.gelu_gate(z, table, ids, 0),
               T * side * 6)
        gu = rnd(T, 2 * F)
        report("silu_mul", tag, lambda: ops.silu_mul(gu), T * F * 6)
        # experts: every chosen expert's weights once, rows in and out
        used = min(NE, T * top)
        per = 3 * W * F
        nbytes = 2 * (used * per + T * W) + 6 * T * W
        report("experts (with shared, norm, add)", tag,
               lambda: experts.mixture_add_rms(
                   x, router, up, down, su, sd, top, r, nw, 1e-5),
               nbytes + 2 * per + 8 * T * W, T * (top + 1) * 2 * per)
        report("experts (routed only, sum)", tag, lambda: experts.mixture(
            x, router[:NE], up, down, None, None, top), nbytes,
            T * top * 2 * per)

        def other():
            p = (x.float() @ router[:NE].float().t()).softmax(-1)
            wt, ids = p.topk(top, dim=-1)
            wt = wt / wt.sum(-1, keepdim=True)
            ops.moe_ffn(x, up, down, wt.to(bf), ids.int())
        report("moe (route, moe_ffn)", tag, other, nbytes, T * top * 2 * per)

    for lens in ([2048], [8192], [1024] * 8):
        m, nb = meta_for(lens)
        T, tag = sum(lens), "x".join(map(str, (len(lens), lens[0])))
        m.latent = {win: LatentSpan(
            m.slot_mapping, m.seq_start[:-1].contiguous(),
            i32([0] * len(lens)), i32(prefill_tiles(lens, SPAN_TOKENS)[0]),
            None)}
        q, kv = rnd(T, H * (D + R) + rank + R).split(
            [H * (D + R), rank + R], -1)
        cache = LatentKV(torch.zeros(nb, 16, rank + R, dtype=bf, device=dev))
        report("latent_rope_append", tag, lambda: latent.rope_append(
            q, kv, kw, m, fr, cache, H, 1e-5),
            T * (4 * H * R + 4 * (rank + R)))
        pairs = sum(min(p + 1, win) for x in lens for p in range(x))
        lat, out = rnd(T, rank + R), rnd(T, H * E)
        kn, vt, sp = lat[:, :rank] @ uk, uv @ lat[:, :rank].t(), m.latent[win]
        report("latent_gather", tag, lambda: n_.latent_gather(
            lat, cache.kv, sp.slots), T * (rank + R) * 4)
        report("latent_attn_prefill", tag, lambda: n_.latent_attn_prefill(
            out, q, kn, lat, vt, m.positions, m.seq_start, sp.start, sp.first,
            sp.tiles, H, win, 0.07), 2 * T * H * (2 * D + R + 2 * E),
            pairs * H * 2 * (D + R + E))
        report("latent attention, with expansion", tag,
               lambda: latent.attention(q, cache, m, uk, uv, H, win, 0.07),
               2 * T * (H * (D + R + E) + rank + R),
               pairs * H * 2 * (D + R + E) + T * rank * H * (D + E) * 2)
        q2, k2, v2 = (x.view(T, -1, 128) for x in rnd(
            T, (H + 2 * G) * 128).split([H * 128, G * 128, G * 128], -1))
        kc = torch.zeros(2, nb, G, 16, 128, dtype=bf, device=dev)
        cs = torch.randn(max(lens), 128, device=dev)
        report("rope_kv_append", tag, lambda: ops.rope_kv_append(
            q2, k2, v2, m.positions, cs, m.slot_mapping, kc[0], kc[1]),
            2 * T * 128 * (2 * H + 4 * G))
        report("attn_prefill_mfma", tag, lambda: ops.attention(
            q2, k2, v2, kc[0], kc[1], m, 0.088),
            2 * T * 128 * (2 * H + 2 * G),
            sum(x * (x + 1) // 2 for x in lens) * H * 4 * 128)
        lq, lk, lv, lg = rnd(T, 4 * W).split([W] * 4, -1)
        st = RecurrentState(torch.zeros(len(lens), H, 128, 128, device=dev))
        report("lightning_prefill", tag, lambda: hybrid.lightning_mix(
            lq, lk, lv, decay, st, m), T * W * 10,
            T * H * 2 * (2 * 128 * 128 + 32 * 256))
        ga, a2 = rnd(T, 4 * W + 24), rnd(W, 24)
        gq, gk, gv, gg, ga = ga.split([W] * 4 + [24], -1)
        a2b, wn = torch.zeros(W, device=dev), torch.ones(128, device=dev)
        report("gla_prefill", tag, lambda: hybrid.gla_mix(
            gq, gk, gv, gg, ga, a2, a2b, wn, st, m, 8.0, 1e-5),
            2 * T * (5 * W + 24), T * H * 2 * (2 * 128 * 128 + 32 * 256))
        common(T, tag)
    for B in (1, 32, 256):
        ctx = 1024
        m, nb = meta_for([1] * B, "decode", ctx)
        tag = f"b{B}_ctx{ctx}"
        q, kv = rnd(B, H * (D + R) + rank + R).split(
            [H * (D + R), rank + R], -1)
        cache = LatentKV(rnd(nb, 16, rank + R))
        report("latent_rope_append", tag, lambda: latent.rope_append(
            q, kv, kw, m, fr, cache, H, 1e-5),
            B * (4 * H * R + 4 * (rank + R)))
        qa, out = rnd(B, H, rank), rnd(B, H * E)
        report("latent_absorb", tag, lambda: n_.latent_absorb(
            qa, q, uk, None, H), 2 * H * (D * rank + B * (D + rank)),
            2 * B * H * D * rank)
        nbytes = 2 * B * (win * (rank + R) + H * (2 * rank + R))
        flops = 2 * B * win * H * (2 * rank + R)
        split = latent.absorbed_split(B * -(-H // 32), win)
        part = torch.empty(B, H, split, rank + 4, device=dev)
        report("latent_attn_decode", f"{tag}_split{split}",
               lambda: n_.latent_attn_decode(
                   part, qa, q, cache.kv, m.block_tables, m.positions, None,
                   None, split, win, 0.07), nbytes, flops)
        report("latent_merge_values", tag, lambda: n_.latent_merge_values(
            out, part, uv, None, B, H, split),
            2 * H * (E * rank + B * (E + 2 * split * rank)),
            2 * B * H * E * rank)
        report("latent attention, absorbed", tag, lambda: latent.attention(
            q, cache, m, uk, uv, H, win, 0.07),
            nbytes + 2 * H * rank * (D + E),
            flops + 2 * B * H * rank * (D + E))
        q2, k2, v2 = (x.view(B, -1, 128) for x in rnd(
            B, (H + 2 * G) * 128).split([H * 128, G * 128, G * 128], -1))
        kc = rnd(2, nb, G, 16, 128)
        cs = torch.randn(ctx + 1, 128, device=dev)
        report("rope_kv_append", tag, lambda: ops.rope_kv_append(
            q2, k2, v2, m.positions, cs, m.slot_mapping, kc[0], kc[1]),
            2 * B * 128 * (2 * H + 4 * G))
        report("paged_attn_decode", tag, lambda: ops.paged_attn_decode(
            q2, kc[0], kc[1], m.block_tables, m.seq_lens, 0.088),
            4 * B * (ctx + 1) * G * 128)
        lq, lk, lv, lg = rnd(B, 4 * W).split([W] * 4, -1)
        st = RecurrentState(torch.zeros(B, H, 128, 128, device=dev))
        report("lightning_step", tag, lambda: hybrid.lightning_mix(
            lq, lk, lv, decay, st, m), B * H * 128 * 128 * 8)
        common(B, tag)


def bench_sigmoid(iters, W):
    """Kernels of the Mutusun design at width W and the like kernels of the
    Mixtral-like model."""
    import hyperspot.ops as ops
    from hyperspot.engine.kv_cache import KVPages
    from hyperspot.ops import experts, hybrid
    dev, bf, f32 = DEV, torch.bfloat16, torch.float32
    report = lambda name, tag, fn, nbytes, flops=0: report_kernel(
        iters, name, f"w{W}_{tag}", fn, nbytes, flops, timed_graph)
    rnd = lambda *s, d=bf: (torch.randn(*s, device=dev) * 0.3).to(d)
    H, G, D, chunk, taps = W // 128, W // 512, 128, 16384, 4
    NE, top, F = 65536 // W, 4, W // 2
    NI = NE // 8
    rules = experts.Rules(torch.zeros(NE + NI, device=dev), NI, 7.0)
    qw, kw, bias = rnd(D, d=f32), rnd(D, d=f32), rnd(H, d=f32)
    up, down = rnd(NE, 2 * F, W) * 0.1, rnd(NE, W, F) * 0.1
    router, conv = rnd(NE + NI, W), rnd(taps, W, d=f32)
    nw, w2 = torch.ones(W, device=dev), torch.ones(W, dtype=bf, device=dev)

    def common(m, T, seqs, tag):
        x, r, y = rnd(T, W), rnd(T, W, d=f32), rnd(T, W)
        nxt = hybrid.NextInput(nw, 1e-5, conv, rnd(seqs, taps - 1, W))
        decode = m.mode == "decode"
        tail = 4 * seqs * (taps - 1) * W
        report("add_rms_next" + " (with conv)" * decode, tag,
               lambda: hybrid.add_rms_next(x, r, nw, nxt if decode else
                                           hybrid.NextInput(nw, 1e-5), m),
               T * W * 12 + tail * decode)
        report("fused_add_rmsnorm", tag, lambda: ops.fused_add_rmsnorm(
            x, y, w2, 1e-5), T * W * 8)
        if not decode:
            report("causal_conv", tag, lambda: hybrid.causal_conv(
                x, conv, nxt.tail, m), T * W * 4 + tail)
        u, gu = rnd(T, 6 * F), rnd(T, 12 * F)
        report("squared_relu", tag, lambda: hybrid.squared_relu(u),
               T * F * 24)
        report("clamped_glu", tag, lambda: hybrid.clamped_glu(gu, 7.0),
               T * F * 36)
        report("silu_mul", tag, lambda: ops.silu_mul(gu), T * F * 36)
        # experts: every chosen expert's weights once, rows in and out; one
        # choice in nine needs no expert
        real = T * top * NE / (NE + NI)
        per = 3 * W * F
        nbytes = 2 * (min(NE, real) * per + T * W) + 6 * T * W
        report("experts (with norms, add, conv)", tag,
               lambda: experts.mixture_add_next(
                   x, router, up, down, None, None, top, rules, r, nw, nxt,
                   m), nbytes + 8 * T * W, real * 2 * per)
        report("experts (sum only)", tag, lambda: experts.mixture(
            x, router, up, down, None, None, top, rules), nbytes,
            real * 2 * per)

        def other():
            p = (x.float() @ router[:NE].float().t()).softmax(-1)
            wt, ids = p.topk(top, dim=-1)
            wt = wt / wt.sum(-1, keepdim=True)
            ops.moe_ffn(x, up, down, wt.to(bf), ids.int())
        report("moe (route, moe_ffn)", tag, other,
               2 * (min(NE, T * top) * per + T * W) + 6 * T * W,
               T * top * 2 * per)

    def heads(T):
        return rnd(T, (H + 2 * G) * D).split([H * D, G * D, G * D], -1)

    for lens in ([2048], [8192], [1024] * 8):
        m, nb = meta_for(lens)
        T, tag = sum(lens), "x".join(map(str, (len(lens), lens[0])))
        q, k, v = heads(T)
        cache = KVPages(torch.zeros(nb, G, 16, D, dtype=bf, device=dev),
                        torch.zeros(nb, G, D, 16, dtype=bf, device=dev))
        pairs = sum(x * (x + 1) // 2 for x in lens)
        report("norm_append", tag, lambda: hybrid.norm_append(
            q, k, v, qw, kw, m, cache, 1e-5), 2 * T * D * (2 * H + 4 * G))
        q2, k2, v2 = (x.view(T, -1, D) for x in heads(T))
        kc = torch.zeros(2, nb, G, 16, D, dtype=bf, device=dev)
        cs = torch.randn(max(lens), D, device=dev)
        report("rope_kv_append", tag, lambda: ops.rope_kv_append(
            q2, k2, v2, m.positions, cs, m.slot_mapping, kc[0], kc[1]),
            2 * T * D * (2 * H + 4 * G))
        nbytes = 2 * T * D * (2 * H + 2 * G)
        report("sigmoid_attn_prefill", tag, lambda: hybrid.sigmoid_attention(
            q, cache, m, bias, chunk, 0.09, 30.0), nbytes,
            pairs * H * 4 * D)
        report("attn_prefill_mfma", tag, lambda: ops.attention(
            q2, k2, v2, kc[0], kc[1], m, 0.088), nbytes, pairs * H * 4 * D)
        common(m, T, len(lens), tag)
    for B in (1, 32, 256):
        ctx = 1024
        m, nb = meta_for([1] * B, "decode", ctx)
        tag = f"b{B}_ctx{ctx}"
        q, k, v = heads(B)
        cache = KVPages(rnd(nb, G, 16, D), rnd(nb, G, D, 16))
        report("norm_append", tag, lambda: hybrid.norm_append(
            q, k, v, qw, kw, m, cache, 1e-5), 2 * B * D * (2 * H + 4 * G))
        q2, k2, v2 = (x.view(B, -1, D) for x in heads(B))
        kc = rnd(2, nb, G, 16, D)
        cs = torch.randn(ctx + 1, D, device=dev)
        report("rope_kv_append", tag, lambda: ops.rope_kv_append(
            q2, k2, v2, m.positions, cs, m.slot_mapping, kc[0], kc[1]),
            2 * B * D * (2 * H + 4 * G))
        nbytes = 4 * B * (ctx + 1) * G * D
        report("sigmoid_attn_decode", tag, lambda: hybrid.sigmoid_attention(
            q, cache, m, bias, chunk, 0.09, 30.0), nbytes)
        report("paged_attn_decode", tag, lambda: ops.paged_attn_decode(
            q2, kc[0], kc[1], m.block_tables, m.seq_lens, 0.088), nbytes)
        common(m, B, B, tag)


def bench_kept(iters, W):
    """Kernels of the Radenex design at width W and the like kernels of a
    plain decoder."""
    import hyperspot.ops as ops
    from hyperspot.engine.kv_cache import KVPages, LatentKV
    from hyperspot.engine.layer_spec import UNBOUNDED
    from hyperspot.engine.rotary import frequencies
    from hyperspot.models.llama import (SPAN_TOKENS, LatentSpan,
                                        prefill_tiles)
    from hyperspot.ops import hybrid, latent
    dev, bf, f32 = DEV, torch.bfloat16, torch.float32
    n_ = ops._native()
    report = lambda name, tag, fn, nbytes, flops=0: report_kernel(
        iters, name, f"w{W}_{tag}", fn, nbytes, flops, timed_graph)
    rnd = lambda *s, d=bf: (torch.randn(*s, device=dev) * 0.3).to(d)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)
    H, G, D, R, rank = W // 128, W // 512, 128, 64, 512
    win, keep, ff, plain_ff = 1024, 4, W * 21 // 4, W * 7 // 2
    fr, turn = (frequencies(n, 1e4).to(dev) for n in (R, D))
    sink, nw = torch.zeros(H, device=dev), torch.ones(W, device=dev)
    w2 = torch.ones(W, dtype=bf, device=dev)
    uk, uv, kw = rnd(rank, H * D), rnd(H * D, rank), rnd(rank, d=f32)

    def common(m, T, tag):
        x, r, y = rnd(T, W), rnd(T, W, d=f32), rnd(T, W)
        nxt = hybrid.NextInput(nw, 1e-5)
        report("add_next", tag, lambda: hybrid.add_next(x, r, nxt, m),
               T * W * 12)
        report("fused_add_rmsnorm", tag, lambda: ops.fused_add_rmsnorm(
            x, y, w2, 1e-5), T * W * 8)
        gu = rnd(T, 2 * plain_ff)
        report("silu_mul", tag, lambda: ops.silu_mul(gu), T * plain_ff * 6)

    def plain_heads(T, ctx, nb, m, tag):
        q, k, v = (x.view(T, -1, D) for x in rnd(
            T, (H + 2 * G) * D).split([H * D, G * D, G * D], -1))
        kc = rnd(2, nb, G, 16, D)
        cs = torch.randn(ctx, D, device=dev)
        report("rope_kv_append", tag, lambda: ops.rope_kv_append(
            q, k, v, m.positions, cs, m.slot_mapping, kc[0], kc[1]),
            2 * T * D * (2 * H + 4 * G))
        return q, k, v, kc

    def joined(T, parts):
        """Column views of a merged projection and the side activation."""
        x = rnd(T, sum(parts) + ff).split([*parts, ff], -1)
        out = rnd(T, H * D + ff)
        return x[:-1], out[:, :H * D], hybrid.SideRelu(x[-1],
                                                       out[:, H * D:])

    def appends(T, m, kvp, lat, tag):
        (q, k, v), out, side = joined(T, [H * D, G * D, G * D])
        (lq, kv, g), lout, lside = joined(T, [H * (D + R), rank + R, H])
        for s, sl, what in ((None, None, ""), (side, lside, " (with side)")):
            extra = 4 * T * ff * (s is not None)
            report("rope_norm_append" + what, tag,
                   lambda: hybrid.rope_norm_append(
                       q, k, v, m, fr, turn, kvp, 1.0, 1e-5, s),
                   2 * T * D * (2 * H + 4 * G) + extra)
            report("latent_rope_append" + what, tag,
                   lambda: latent.rope_append(
                       lq, kv, kw, m, fr, lat, H, 1e-5, 1.2, sl),
                   T * (4 * H * R + 4 * (rank + R)) + extra)
        return q, out, lq, g, lout

    for lens in ([2048], [8192], [1024] * 8):
        m, nb = meta_for(lens)
        T, tag = sum(lens), "x".join(map(str, (len(lens), lens[0])))
        m.latent = {UNBOUNDED: LatentSpan(
            m.slot_mapping, m.seq_start[:-1].contiguous(),
            i32([0] * len(lens)), i32(prefill_tiles(lens, SPAN_TOKENS)[0]),
            None)}
        kvp = KVPages(torch.zeros(nb, G, 16, D, dtype=bf, device=dev),
                      torch.zeros(nb, G, D, 16, dtype=bf, device=dev))
        lat = LatentKV(torch.zeros(nb, 16, rank + R, dtype=bf, device=dev))
        q, out, lq, g, lout = appends(T, m, kvp, lat, tag)
        pairs = sum(min(p + 1, win) for x in lens for p in range(x))
        causal = sum(x * (x + 1) // 2 for x in lens)
        nbytes = 2 * T * D * (2 * H + 2 * G)
        for w, name, n in ((win, "windowed", pairs),
                           (UNBOUNDED, "all", causal)):
            report(f"kept_attn_prefill ({name})", tag,
                   lambda: hybrid.window_attention(
                       out, q, kvp, m, turn, sink, w, keep, 0.09, True),
                   nbytes,
                   n * H * 4 * D)
        sp, c = m.latent[UNBOUNDED], rnd(T, rank + R)
        kn, vt = c[:, :rank] @ uk, uv @ c[:, :rank].t()
        report("latent_attn_prefill", tag, lambda: n_.latent_attn_prefill(
            lout, lq, kn, c, vt, m.positions, m.seq_start, sp.start, sp.first,
            sp.tiles, H, UNBOUNDED, 0.07, sink, g),
            2 * T * H * (2 * D + R + 2 * D), causal * H * 2 * (2 * D + R))
        report("latent attention, with expansion", tag,
               lambda: latent.attention(lq, lat, m, uk, uv, H, UNBOUNDED,
                                        0.07, sink, g, lout),
               2 * T * (H * (2 * D + R) + rank + R),
               causal * H * 2 * (2 * D + R) + T * rank * H * 4 * D)
        q2, k2, v2, kc = plain_heads(T, max(lens), nb, m, tag)
        report("attn_prefill_mfma", tag, lambda: ops.attention(
            q2, k2, v2, kc[0], kc[1], m, 0.088), nbytes, causal * H * 4 * D)
        common(m, T, tag)
    for B in (1, 32, 256):
        ctx = 1024
        m, nb = meta_for([1] * B, "decode", ctx)
        tag = f"b{B}_ctx{ctx}"
        kvp = KVPages(rnd(nb, G, 16, D), rnd(nb, G, D, 16))
        lat = LatentKV(rnd(nb, 16, rank + R))
        q, out, lq, g, lout = appends(B, m, kvp, lat, tag)
        nbytes = 4 * B * (ctx + 1) * G * D
        report("kept_attn_decode", tag, lambda: hybrid.window_attention(
            out, q, kvp, m, turn, sink, win, keep, 0.09, True), nbytes)
        nbytes_l = 2 * B * ((ctx + 1) * (rank + R) + H * (2 * rank + R))
        qa, split = rnd(B, H, rank), latent.absorbed_split(
            B * -(-H // 32), m.block_tables.shape[1] * 16)
        part = torch.empty(B, H, split, rank + 4, device=dev)
        report("latent_absorb", tag, lambda: n_.latent_absorb(
            qa, lq, uk, None, H), 2 * H * (D * rank + B * (D + rank)),
            2 * B * H * D * rank)
        report("latent_attn_decode", tag, lambda: n_.latent_attn_decode(
            part if split > 1 else torch.empty_like(qa), qa, lq, lat.kv,
            m.block_tables, m.positions, None, None, split, UNBOUNDED, 0.07,
            sink), nbytes_l,
            2 * B * H * (ctx + 1) * (2 * rank + R))
        if split > 1:
            report("latent_merge_values", tag, lambda: n_.latent_merge_values(
                lout, part, uv, None, B, H, split, g),
                2 * H * (D * rank + B * (D + 2 * split * rank)),
                2 * B * H * D * rank)
        report("latent attention, absorbed", tag, lambda: latent.attention(
            lq, lat, m, uk, uv, H, UNBOUNDED, 0.07, sink, g, lout),
            nbytes_l + 4 * H * rank * D,
            2 * B * H * ((ctx + 1) * (2 * rank + R) + 2 * rank * D))
        q2, k2, v2, kc = plain_heads(B, ctx + 1, nb, m, tag)
        report("paged_attn_decode", tag, lambda: ops.paged_attn_decode(
            q2, kc[0], kc[1], m.block_tables, m.seq_lens, 0.088), nbytes)
        common(m, B, tag)


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--which", default="attn")
    ap.add_argument("--iters", type=int, default=100)
    args = ap.parse_args()
    assert torch.cuda.is_available()
    if args.which in ("attn", "all"):
        bench_attn(args.iters)
    if args.which in ("gemm", "all"):
        bench_gemm(args.iters)
    if args.which in ("hybrid", "all"):
        bench_hybrid(args.iters)
    if args.which in ("latent", "all"):
        for width in (2048, 4096):
            bench_latent(args.iters, width)
    if args.which in ("sigmoid", "all"):
        for width in (2048, 4096):
            bench_sigmoid(args.iters, width)
    if args.which in ("kept", "all"):
        for width in (2048, 4096):
            bench_kept(args.iters, width)
    if args.which in ("fp8", "all"):
        bench_fp8_gemm(args.iters)


if __name__ == "__main__":
    main()
