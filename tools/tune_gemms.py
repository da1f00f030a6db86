#!/usr/bin/env python3
"""Offline hipBLASLt algorithm tuning for the serving GEMM shapes (GPU).

Runs PyTorch TunableOp tuning over every GEMM the engine issues (decode at
the bucketed batch sizes, chunked prefill, TTFT single-prompt prefill,
logits head) and writes profiles/tunableop_gfx950.csv, which ModelRunner
loads read-only at engine init.

Run on an MI355X box:  python tools/tune_gemms.py [--out FILE]

With --design NAME the products of a design's layers that have a feed-forward
beside the mixer are tuned instead, and FILE gains (or renews) the lines of
those whose choice beats the library's own, timed in a replayed graph and
checked against it over several replays.
"""

from __future__ import annotations

import argparse
import os
import sys
import tempfile

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))

ap = argparse.ArgumentParser()
ap.add_argument("--out", default="profiles/tunableop_gfx950.csv")
ap.add_argument("--include-70b", action="store_true")
ap.add_argument("--design", default=None, metavar="NAME")
args = ap.parse_args()

# TunableOp reads its env at tuning-context construction — set everything
# before torch loads.
os.environ["PYTORCH_TUNABLEOP_MAX_TUNING_DURATION_MS"] = "10"
os.environ["PYTORCH_TUNABLEOP_MAX_TUNING_ITERATIONS"] = "30"
if args.design is None:
    os.environ["PYTORCH_TUNABLEOP_ENABLED"] = "1"
    os.environ["PYTORCH_TUNABLEOP_TUNING"] = "1"
    os.environ["PYTORCH_TUNABLEOP_FILENAME"] = args.out
    os.environ["PYTORCH_TUNABLEOP_VERBOSE"] = "1"
else:            # switched on and off by the program, results merged by it
    os.environ["PYTORCH_TUNABLEOP_FILENAME"] = os.path.join(
        tempfile.mkdtemp(), "results.csv")

import torch  # noqa: E402

# Llama-3-8B
SHAPES_8B = dict(hidden=4096, inter=14336, q=4096, kv=1024, vocab=128256)
# Llama-3-70B at TP=8 (per-rank shards) and TP=1 (single 288GB GPU)
SHAPES_70B_TP8 = dict(hidden=8192, inter=28672 // 8, q=8192 // 8,
                      kv=1024 // 8, vocab=128256 // 8)
SHAPES_70B_TP1 = dict(hidden=8192, inter=28672, q=8192, kv=1024,
                      vocab=128256)


def gemm_shapes(include_70b=False):
    ms = [64, 128, 256, 384, 512, 768, 1024, 2048, 8192]
    specs = (SHAPES_8B, SHAPES_70B_TP8, SHAPES_70B_TP1) if include_70b         else (SHAPES_8B,)
    for spec in specs:
        h, it = spec["hidden"], spec["inter"]
        nqkv = spec["q"] + 2 * spec["kv"]
        for m in ms:
            yield m, h, nqkv            # qkv proj
            yield m, spec["q"], h       # o proj
            yield m, h, 2 * it          # gate_up
            yield m, it, h              # down
        for m in [64, 256, 512, 1024]:
            yield m, h, spec["vocab"]   # logits head


def joined_shapes(spec):
    """(rows, k, n) of the merged projections and of the joined sum of every
    kind of layer."""
    from hyperspot.engine.layer_spec import LatentAttention
    up8 = lambda n: (n + 7) // 8 * 8
    w, out = spec.hidden_size, []
    for m, ff in dict.fromkeys((x.mixer, x.ff) for x in spec.layers):
        if isinstance(m, LatentAttention):
            parts = [m.heads * (m.dim + m.rot_dim), m.kv_rank + m.rot_dim,
                     m.heads]
        else:
            parts = [m.heads * m.dim, m.kv_heads * m.dim,
                     m.kv_heads * m.vdim]
        n = sum(map(up8, parts + [ff.ff]))
        out += [(w, n), (m.heads * m.vdim + ff.ff, w)]
    rows = (1, 2, 4, 8, 16, 24, 32, 48, 64, 96, 128, 192, 256, 384, 512, 768,
            1024, 2048, 8192)
    return [(m, k, n) for k, n in dict.fromkeys(out) for m in rows]


def graph_time(fn, calls=5, replays=20):
    """us a call within a replayed graph."""
    fn()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        for _ in range(calls):
            fn()
    for _ in range(3):
        g.replay()
    a, b = (torch.cuda.Event(enable_timing=True) for _ in range(2))
    a.record()
    for _ in range(replays):
        g.replay()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) * 1e3 / (calls * replays)


def same_in_graph(x, w):
    """A replayed graph gives what the library's own choice gives, over and
    over, with other work and other inputs between the replays."""
    t, ok = torch.cuda.tunable, True
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        y = x @ w.t()
    for _ in range(5):
        x.normal_()
        g.replay()
        got = y.float()
        t.enable(False)
        want = (x @ w.t()).float()
        t.enable(True)
        torch.cuda.synchronize()
        err = (got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt()
        ok = ok and float(err) < 1e-2
    return ok


def tune_design(name, out):
    from hyperspot.engine.config import get_model_spec
    t = torch.cuda.tunable
    lines, keep, drop = open(out).read().splitlines(), {}, set()
    for m, k, n in joined_shapes(get_model_spec(name)):
        x = torch.randn(m, k, dtype=torch.bfloat16, device="cuda:0")
        w = torch.randn(n, k, dtype=torch.bfloat16, device="cuda:0") * 0.02
        fn = lambda: x @ w.t()
        plain = graph_time(fn)
        before = {r[:2] for r in t.get_results()}
        t.enable(True)
        t.tuning_enable(True)
        fn()
        t.tuning_enable(False)
        new = [r for r in t.get_results() if r[:2] not in before]
        tuned, good = graph_time(fn), same_in_graph(x, w)
        t.enable(False)
        plain = min(plain, graph_time(fn))
        won = good and tuned < 0.97 * plain
        for op, params, solution, ms in new:
            if won:
                keep[f"{op},{params}"] = f"{op},{params},{solution},{ms:g}"
            else:
                drop.add(f"{op},{params}")
        print(f"{m}x{k}x{n}: {plain:.1f} us, tuned {tuned:.1f} us"
              f"{'' if good else ', WRONG'}{' *' if won else ''}", flush=True)
        del x, w
    head = lambda line: ",".join(line.split(",")[:2])
    lines = [x for x in lines if head(x) not in keep and head(x) not in drop]
    with open(out, "w") as f:
        f.write("\n".join(lines + list(keep.values())) + "\n")
    print(f"{len(keep)} choices kept")


def main():
    assert torch.cuda.is_available()
    if args.design:
        return tune_design(args.design, args.out)
    dev = "cuda:0"
    seen = set()
    shapes = [s for s in gemm_shapes(args.include_70b)
              if not (s in seen or seen.add(s))]
    for i, (m, k, n) in enumerate(shapes):
        x = torch.randn(m, k, dtype=torch.bfloat16, device=dev)
        w = torch.randn(n, k, dtype=torch.bfloat16, device=dev)
        torch.nn.functional.linear(x, w)   # tuning happens on first call
        torch.cuda.synchronize()
        print(f"[{i + 1}/{len(shapes)}] tuned {m}x{k}x{n}", flush=True)
        del x, w
    # fp8 path (ScaledGemm): same shapes, e4m3fn + rowwise scales
    from hyperspot.parallel.layers import (quant_fp8_rowwise,
                                           quantize_weight_fp8)
    for i, (m, k, n) in enumerate(shapes):
        x = torch.randn(m, k, dtype=torch.bfloat16, device=dev)
        w = torch.randn(n, k, dtype=torch.bfloat16, device=dev) * 0.02
        wq, ws = quantize_weight_fp8(w)
        xq, xs = quant_fp8_rowwise(x)
        torch._scaled_mm(xq, wq.t(), scale_a=xs[:, None].contiguous(),
                         scale_b=ws[None, :].contiguous(),
                         out_dtype=torch.bfloat16)
        torch.cuda.synchronize()
        print(f"[fp8 {i + 1}/{len(shapes)}] tuned {m}x{k}x{n}", flush=True)
        del x, w, wq, xq
    # results are flushed by TunableOp at interpreter exit; make sure the
    # directory exists so the write succeeds
    d = os.path.dirname(args.out)
    if d:
        os.makedirs(d, exist_ok=True)
    print("tuning done; results flush to", args.out, "at exit")


if __name__ == "__main__":
    main()
