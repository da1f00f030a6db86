"""Radenex on the GPU: every kernel against the plain float64 implementation,
and whole models in bfloat16 and float32 through prefill, decode graphs,
portions and mixed batches."""

import pytest
import torch

import radenex_oracle as O
import radenex_util as U
from hyperspot import ops
from hyperspot.engine import EngineConfig, LLMEngine, SamplingParams
from hyperspot.engine.kv_cache import KVPages, LatentKV
from hyperspot.engine.replay import Replay
from hyperspot.engine.rotary import (frequencies, head_order,
                                     pair_order)
from hyperspot.ops import hybrid, latent

pytestmark = pytest.mark.gpu
DEV = "cuda"
BF, F32 = torch.bfloat16, torch.float32


def setup_module():
    assert ops.have_native(), "the gfx950 extension must be built"


def rand(*shape, seed=0, gain=1.0, dtype=F32):
    g = torch.Generator().manual_seed(seed)
    return (gain * torch.randn(*shape, generator=g)).to(dtype)


def f64(x):
    return x.detach().cpu().to(torch.float64)


def rel(got, want):
    """Largest row error relative to the overall RMS."""
    d = (f64(got) - want).flatten(1).pow(2).mean(-1).sqrt()
    return float((d / want.pow(2).mean().sqrt()).max())


def tol(dtype):
    return 2e-5 if dtype == F32 else 2e-2


def meta_for(starts, lens, decode=False):
    """Metadata for portions [start, start + len) of as many sequences, with
    shuffled pages, as the runner makes it."""
    from test_mutusun_gpu import meta_for as make
    return make(starts, lens, decode)


# ---------------------------------------------------------------- residual

@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("width", [8, 57, 1000, 2304, 4100, 5004])
def test_plain_add_and_norm(dtype, width):
    y = rand(5, width, seed=9, gain=2, dtype=dtype)
    res, pre = rand(5, width), rand(width, seed=1)
    r = res.to(DEV)
    m, _ = meta_for([0], [5])
    h = hybrid.add_next(y.to(DEV), r, hybrid.NextInput(pre.to(DEV), 1e-3), m)
    want = f64(res) + f64(y)
    assert h.dtype == dtype and rel(r, want) < 1e-6
    assert rel(h, O.rms(want, 1e-3) * f64(pre)) < tol(dtype)


# --------------------------------------------------- rotation, norm, append

def side_views(T, n, dtype, aligned=True):
    """x and out as columns of wider buffers."""
    a = 8 if aligned else 3
    x = rand(T, n + 2 * a, seed=11, gain=2, dtype=dtype)
    out = torch.full((T, n + 2 * a), 7.0, dtype=dtype, device=DEV)
    return x, hybrid.SideRelu(x.to(DEV)[:, a:a + n], out[:, a:a + n]), out, a


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("lens,H,G,D,E,rot", [
    (lens, *sizes) for sizes in (
        (4, 2, 16, 24, 8), (6, 3, 7, 6, 4), (16, 4, 128, 128, 64),
        (3, 1, 96, 40, 96), (1, 1, 1, 2, 0), (2, 2, 520, 8, 512),
        (5, 1, 24, 600, 2))
    for lens in ([15, 25], [1500], [4200]) if len(lens) > 1
    or sizes[2] <= 256 and sizes[3] <= 256 or lens == [1500]])
def test_rope_norm_append(dtype, lens, H, G, D, E, rot):
    m, nb = meta_for([90000] * len(lens), lens)
    T = sum(lens)
    buf = rand(T, (H + G) * D + G * E + 8, dtype=dtype)
    slots = m.slot_mapping.cpu()
    m.slot_mapping[-1] = -1
    pos, x = m.positions.cpu(), f64(buf)
    heads = lambda a, n, d: x[:, a:a + n * d].view(T, n, d)
    freqs, turn = frequencies(rot, 3e3, 1.7), frequencies(E, 3e3)
    turned = [O.rotate_halves(heads((H + G) * D, G, E)[:, g], pos,
                              O.base_frequencies(E, 3e3)) for g in range(G)]
    order = pair_order(D, rot, True)
    n = (5, 24, 2048 + 64)[H % 3]
    for eps, gain, values in ((1e-4, 1.0, True), (None, 1.3, False)):
        src, side, out, a = side_views(T, n, dtype, aligned=n != 5)
        b = buf.to(DEV)
        q, k, v, _ = b.split([H * D, G * D, G * E, 8], -1)
        q.copy_(q[:, head_order(H, D, order)])
        kp = k[:, head_order(G, D, order)]
        vp = v[:, head_order(G, E, pair_order(E, E, values))]
        k.copy_(kp)
        v.copy_(vp)
        cache = KVPages(
            torch.full((nb, G, 16, D), 9.0, dtype=dtype, device=DEV),
            torch.full((nb, G, E, 16), 9.0, dtype=dtype, device=DEV))
        hybrid.rope_norm_append(
            q, k, v, m, freqs.to(DEV),
            (turn if values else turn[:0]).to(DEV), cache, gain, eps, side)

        def head(t):
            t = O.rotate_halves(t, pos, O.linear_frequencies(rot, 3e3, 1.7),
                                gain)
            return (t if eps is None else O.rms(t, eps))[:, order]

        want = f64(src)[:, a:a + n].clamp(min=0) ** 2
        assert rel(side.out, want) < tol(dtype)
        assert (out[:, :a] == 7.0).all() and (out[:, a + n:] == 7.0).all()
        kf = cache.k.permute(0, 2, 1, 3).reshape(-1, G, D).cpu()
        vf = cache.v.permute(0, 3, 1, 2).reshape(-1, G, E).cpu()
        for h in (0, H - 1):
            assert rel(q.reshape(T, H, D)[:, h],
                       head(heads(0, H, D)[:, h])) < tol(dtype)
        for g in (0, G - 1):
            assert rel(kf[slots[:-1], g],
                       head(heads(H * D, G, D)[:, g])[:-1]) < tol(dtype)
            want = turned[g][:, pair_order(E, E, True)] if values \
                else heads((H + G) * D, G, E)[:, g]
            assert rel(vf[slots[:-1], g], want[:-1]) < tol(dtype)
        assert (kf[slots[-1]] == 9.0).all() and (vf[slots[-1]] == 9.0).all()
        assert torch.equal(b[:, -8:].cpu(), buf[:, -8:])


# -------------------------------------------------------- windowed attention

def seen(p, window, keep):
    """visible(), as one index tensor."""
    lo = max(0, p - window + 1)
    return torch.cat([torch.arange(min(keep, lo)), torch.arange(lo, p + 1)])


def test_seen_is_visible():
    for p, w, k in ((0, 1, 0), (9, 3, 2), (9, 3, 20), (30, 40, 5), (7, 7, 1)):
        assert seen(p, w, k).tolist() == O.visible(p, w, k)


def attention_case(H, G, D, E, window, keep, starts, lens, dtype,
                   decode=False, loud=(), scale=None, sink="random",
                   turn=True):
    m, nb = meta_for(starts, lens, decode)
    n, longest = len(lens), max(a + b for a, b in zip(starts, lens))
    k = rand(n, longest, G, D, seed=2, dtype=dtype)
    v = rand(n, longest, G, E, seed=3, dtype=dtype)
    for s, at in loud:
        k[s, at] *= 8
        v[s, at] *= 8
    # what no sequence holds must not matter
    kc = torch.full((nb, G, 16, D), 1e4, dtype=dtype)
    vc = torch.full((nb, G, E, 16), 1e4, dtype=dtype)
    bt = m.block_tables.cpu()
    for i in range(n):
        p = torch.arange(starts[i] + lens[i])
        blk, off = bt[i][p // 16].long(), p % 16
        kc[blk, :, off] = k[i, p]
        vc[blk, :, :, off] = v[i, p]
    T = sum(lens)
    buf = rand(T, H * D + 8, seed=4, dtype=dtype)
    bias = {"random": rand(H, seed=6, gain=2), "zero": torch.zeros(H),
            None: None}[sink]
    scale = scale or 1.5 * D ** -0.5
    wide = torch.full((T, H * E + 16), 7.0, dtype=dtype, device=DEV)
    out = wide[:, 8:8 + H * E]
    freqs = frequencies(E if turn else 0, 50.0)
    run = lambda to, bounded: hybrid.window_attention(
        to, buf.to(DEV)[:, :H * D], KVPages(kc.to(DEV), vc.to(DEV)), m,
        freqs.to(DEV), None if bias is None else bias.to(DEV), window, keep,
        scale, bounded)
    run(out, False)
    assert (wide[:, :8] == 7.0).all() and (wide[:, -8:] == 7.0).all()
    if not loud:                       # small scores: without their maximum
        again = torch.full_like(wide, 7.0)
        run(again[:, 8:8 + H * E], True)
        assert (again[:, :8] == 7.0).all() and (again[:, -8:] == 7.0).all()
        assert rel(again, f64(wide)) < tol(dtype)
    want, row, x = [], 0, f64(buf)
    for i in range(n):
        ki, vi = f64(k[i]), f64(v[i])
        for p in range(starts[i], starts[i] + lens[i]):
            j = seen(p, window, keep)
            q = x[row, :H * D].view(G, H // G, D)
            s = torch.einsum("gxd,ngd->gxn", q, ki[j]).reshape(H, -1) * scale
            if bias is not None:
                s = torch.cat([s, f64(bias)[:, None]], -1)
            a = s.softmax(-1)[:, :len(j)].view(G, H // G, -1)
            o = torch.einsum("gxn,nge->gxe", a, vi[j]).reshape(H, E)
            if turn:
                ang = -p * freqs
                u, w = o[:, 0::2], o[:, 1::2]
                o = torch.stack([u * ang.cos() - w * ang.sin(),
                                 w * ang.cos() + u * ang.sin()], -1)
            want.append(o.reshape(-1))
            row += 1
    return out, torch.stack(want)


SIZES = [(2, 1, 8, 8), (6, 2, 64, 48), (3, 3, 48, 40), (16, 4, 128, 128),
         (17, 1, 16, 128), (40, 2, 32, 16), (4, 1, 64, 256), (3, 1, 120, 200),
         (16, 1, 256, 256), (5, 5, 200, 136), (6, 3, 7, 6), (1, 1, 1, 2),
         (2, 1, 16, 600)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,G,D,E", SIZES)
def test_attention_prefill(dtype, H, G, D, E):
    """Portions with and without earlier tokens in one step; starts and ends
    off every tile, page and window border."""
    got, want = attention_case(H, G, D, E, 37, 3, [0, 50, 0, 21, 3],
                               [70, 17, 5, 16, 30], dtype)
    assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("window,keep", [
    (1, 0), (1, 64), (2, 1), (31, 5), (32, 32), (64, 65), (65, 16), (64, 0),
    (200, 130), (100, 250), (5000, 7), (1 << 30, 0), (7, 1 << 30)])
def test_attention_prefill_windows(dtype, window, keep):
    got, want = attention_case(2, 1, 16, 24, window, keep, [0, 190],
                               [300, 140], dtype)
    assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("D,E", [(16, 24), (40, 128), (128, 128), (64, 200),
                                 (104, 256), (256, 256)])
@pytest.mark.parametrize("window,keep", [(45, 4), (300, 70)])
def test_attention_prefill_by_pairs_of_heads(D, E, window, keep):
    """Enough tiles and heads that one workgroup takes two heads."""
    got, want = attention_case(64, 2, D, E, window, keep, [0, 333, 70],
                               [700, 300, 30], BF)
    assert rel(got, want) < 2e-2


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,G,D,E", SIZES)
@pytest.mark.parametrize("rows", [1, 20])
def test_attention_decode(dtype, H, G, D, E, rows):
    ctx = [0, 15, 16, 17, 31, 32, 300, 301, 255, 256][:rows] * 2
    ctx = ([300] if rows == 1 else ctx)[:rows]
    for window, keep in ((37, 4), (200, 33), (10, 290), (400, 0)):
        got, want = attention_case(H, G, D, E, window, keep, ctx, [1] * rows,
                                   dtype, decode=True)
        assert rel(got, want) < tol(dtype)


def test_decode_of_many_rows_is_not_split():
    assert hybrid.decode_split(520, 400) == 1
    got, want = attention_case(2, 1, 16, 24, 20, 9,
                               [i % 70 for i in range(520)], [1] * 520, BF,
                               decode=True)
    assert rel(got, want) < 2e-2


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("sink", ["random", "zero", None])
@pytest.mark.parametrize("turn", [True, False])
@pytest.mark.parametrize("start,lens", [(300, [1]), (0, [1]), (300, [70]),
                                        (0, [40])])
def test_options(dtype, sink, turn, start, lens):
    """With and without sinks and turned values, negative scales; a row that
    sees few keys gives the sink a large share."""
    for scale in (0.4, -0.3, 2.0):
        got, want = attention_case(4, 2, 16, 24, 200, 3, [start], lens, dtype,
                                   lens == [1], sink=sink, turn=turn,
                                   scale=scale)
        assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("lens", [[1], [2], [16], [17], [80]])
@pytest.mark.parametrize("window,keep", [(20, 3), (200, 0)])
def test_loud_key_at_the_edges(dtype, lens, window, keep):
    """One key far above all others: last seen by position at + window - 1;
    among the first tokens, the last kept one is seen for good."""
    for at, first, shows in (
            (64, 64 + window - 1, True), (64, 64 + window, False),
            (keep - 1, 2 * window, True), (keep, 2 * window, False)):
        if at < 0:
            continue
        case = lambda loud: attention_case(
            2, 1, 16, 24, window, keep, [first], lens, dtype,
            decode=lens == [1], loud=loud)
        got, want = case([(0, at)])
        assert rel(got, want) < tol(dtype)
        moved = rel(want[:1], case([])[1][:1])
        assert moved > 0.3 if shows else moved == 0


# --------------------------------------------------------- latent attention

def latent_case(H, D, R, E, rank, window, starts, lens, dtype, decode=False,
                sink=True, gate=True):
    import test_tefezen_gpu as other
    m, nb = other.meta_for(starts, lens, window, decode)
    n, longest = len(lens), max(a + b for a, b in zip(starts, lens))
    rows = rand(n, longest, rank + R, seed=2, gain=0.5, dtype=dtype)
    cache = torch.full((nb, 16, rank + R), 1e4, dtype=dtype)
    bt = m.block_tables.cpu()
    for i in range(n):
        p = torch.arange(starts[i] + lens[i])
        cache[bt[i][p // 16].long(), p % 16] = rows[i, p]
    T = sum(lens)
    buf = rand(T, H * (D + R) + 8, seed=4, dtype=dtype)
    g = rand(T, H + 5, seed=8, gain=2, dtype=dtype)
    uk = rand(rank, H * D, seed=6, gain=rank ** -0.5, dtype=dtype)
    uv = rand(H * E, rank, seed=7, gain=rank ** -0.5, dtype=dtype)
    bias = rand(H, seed=9, gain=2)
    scale = 1.3 * (D + R) ** -0.5
    wide = torch.full((T, H * E + 16), 7.0, dtype=dtype, device=DEV)
    out = wide[:, 8:8 + H * E]
    latent.attention(buf.to(DEV)[:, :H * (D + R)], LatentKV(cache.to(DEV)), m,
                     uk.to(DEV), uv.to(DEV), H, window, scale,
                     bias.to(DEV) if sink else None,
                     g.to(DEV)[:, 2:2 + H] if gate else None, out)
    assert (wide[:, :8] == 7.0).all() and (wide[:, -8:] == 7.0).all()
    want, row, x, b = [], 0, f64(buf), f64(bias)
    ku = f64(uk).view(rank, H, D).permute(1, 0, 2)      # [H, rank, D]
    vu = f64(uv).view(H, E, rank)
    for i in range(n):
        c, kr = f64(rows[i])[:, :rank], f64(rows[i])[:, rank:]
        key = torch.cat([c @ ku, kr.expand(H, -1, -1)], -1)   # [H, n, D + R]
        val = c @ vu.transpose(1, 2)                          # [H, n, E]
        for p in range(starts[i], starts[i] + lens[i]):
            lo = max(0, p - window + 1)
            q = x[row, :H * (D + R)].view(H, D + R, 1)
            s = (key[:, lo:p + 1] @ q)[..., 0] * scale
            if sink:
                s = torch.cat([s, b[:, None]], -1)
            a = s.softmax(-1)[:, :p + 1 - lo]
            o = (a[:, None] @ val[:, lo:p + 1])[:, 0]
            if gate:
                o = o * torch.sigmoid(f64(g)[row, 2:2 + H])[:, None]
            want.append(o.reshape(-1))
            row += 1
    return out, torch.stack(want)


LATENT = [(2, 8, 8, 8, 16), (5, 64, 32, 48, 104), (3, 48, 16, 40, 72),
          (16, 24, 8, 32, 128), (17, 16, 24, 128, 200), (2, 128, 64, 128, 512),
          (33, 32, 64, 16, 256), (1, 192, 64, 256, 512), (3, 7, 6, 9, 11),
          (1, 1, 2, 1, 1), (2, 16, 80, 24, 600)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,D,R,E,rank", LATENT)
def test_latent_prefill(dtype, H, D, R, E, rank):
    got, want = latent_case(H, D, R, E, rank, 1 << 30, [0, 50, 0, 21, 3],
                            [150, 17, 5, 16, 30], dtype)
    assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,D,R,E,rank", LATENT)
@pytest.mark.parametrize("rows", [1, 20])
def test_latent_decode(dtype, H, D, R, E, rank, rows):
    ctx = [0, 15, 16, 17, 31, 32, 300, 301, 255, 256][:rows] * 2
    ctx = ([300] if rows == 1 else ctx)[:rows]
    for window in (1 << 30, 37):
        got, want = latent_case(H, D, R, E, rank, window, ctx, [1] * rows,
                                dtype, decode=True)
        assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("sink,gate", [(True, False), (False, True),
                                       (False, False)])
def test_latent_options(dtype, sink, gate):
    for starts, lens in (([0, 200], [1, 1]), ([0, 90], [40, 12]),
                         ([i % 40 for i in range(600)], [1] * 600)):
        got, want = latent_case(4, 16, 8, 24, 40, 1 << 30, starts, lens,
                                dtype, decode=max(lens) == 1, sink=sink,
                                gate=gate)
        assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("n", [5, 24, 2048, 5000])
def test_latent_append_with_gain_and_side(dtype, n):
    import test_tefezen_gpu as other
    H, D, R, rank, T = 3, 8, 16, 24, 40
    m, nb = other.meta_for([0, 90000], [15, 25], 10)
    buf = rand(T, H * (D + R) + rank + R, dtype=dtype)
    q, kv = buf.to(DEV).split([H * (D + R), rank + R], -1)
    w, fr = rand(rank, seed=3), frequencies(R, 3e4)
    cache = LatentKV(torch.zeros(nb, 16, rank + R, dtype=dtype, device=DEV))
    src, side, out, a = side_views(T, n, dtype, aligned=n != 5)
    latent.rope_append(q, kv, w.to(DEV), m, fr.to(DEV), cache, H, 1e-4, 1.4,
                       side)
    assert rel(side.out, f64(src)[:, a:a + n].clamp(min=0) ** 2) < tol(dtype)
    assert (out[:, :a] == 7.0).all() and (out[:, a + n:] == 7.0).all()
    order, pos, x = pair_order(R, R, True), m.positions.cpu(), f64(buf)
    inv = torch.tensor(order).argsort()
    f = O.base_frequencies(R, 3e4)
    turned = lambda t: O.rotate_halves(t[:, inv], pos, f, 1.4)[:, order]
    for h in range(H):
        at = h * (D + R)
        assert torch.equal(q[:, at:at + D].cpu(), buf[:, at:at + D])
        assert rel(q[:, at + D:at + D + R],
                   turned(x[:, at + D:at + D + R])) < tol(dtype)
    raw = x[:, H * (D + R):]
    want = torch.cat([O.rms(raw[:, :rank], 1e-4) * f64(w),
                      turned(raw[:, rank:])], -1)
    flat = cache.kv.view(-1, rank + R)[m.slot_mapping]
    assert rel(flat, want) < tol(dtype)


# ------------------------------------------------------------ whole models

DTYPES = ["bfloat16", "float32"]


def limits(dtype, cfg, w):
    """Allowed error per position for a request's tokens."""
    if dtype == "float32":
        return lambda toks: 3e-4
    return lambda toks: U.rounding_limits(O.forward, cfg, w, toks)


def within(got, cfg, w, toks, lim):
    e = U.errors(got, O.forward(cfg, w, toks)[0]) / lim
    assert got.isfinite().all() and float(e.max()) < 1, float(e.max())


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    cfg = U.standard()
    w = U.weights(cfg, seed=1)
    return cfg, w, U.write(tmp_path_factory.mktemp("std"), cfg, w)


def replay(folder, dtype, max_tokens=512, eager=False):
    return Replay(folder, dtype, max_tokens, device=DEV, eager=eager)


def test_model_portions(model):
    cfg, w, folder = model
    toks = U.tokens(160, cfg["vocab"], seed=1)
    for dtype in DTYPES:
        lim = limits(dtype, cfg, w)(toks)
        for cuts in ([160], [1], [2], [63, 65, 2, 5], [30, 1], [17, 16]):
            within(U.feed(replay(folder, dtype), "a", toks, cuts), cfg, w,
                   toks, lim)


@pytest.mark.parametrize("dtype", DTYPES)
def test_model_mixed_batches_reuse(model, dtype):
    from test_radenex import LENS, fill_caches, mixed_run
    cfg, w, folder = model
    r = replay(folder, dtype, 4 * 128)
    fill_caches(r, 5.0)
    assert mixed_run(r, cfg, w, LENS, limits=limits(dtype, cfg, w)) < 1
    assert r.engine.runner.block_manager.num_free == 32


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", [
    "ones", "odd", "window only", "latent only", "all rotated",
    "negative scale", "many heads", "more kept than seen", "equal sizes"])
def test_model_other_sizes(tmp_path, dtype, name):
    from test_radenex import ODD, mixed_run
    cfg = ODD[name]
    w = U.weights(cfg, seed=6)
    r = replay(U.write(tmp_path, cfg, w), dtype)
    toks = U.tokens(50, cfg["vocab"])
    lim = limits(dtype, cfg, w)
    for i, cuts in enumerate(([50], [20, 1], [2])):
        within(U.feed(r, f"a{i}", toks, cuts), cfg, w, toks, lim(toks))
    assert mixed_run(r, cfg, w, [30, 9, 21], limits=lim) < 1


@pytest.mark.parametrize("cuts", [[80], [10, 1], [30, 2, 1], [16, 17, 2]])
@pytest.mark.parametrize("dtype", DTYPES)
def test_model_window_edge_and_kept_tokens(tmp_path, dtype, cuts):
    from test_radenex import loud, loud_key_model
    for n, (size, keep, at, shows) in enumerate((
            (33, 3, 7, False), (9, 3, 2, True), (9, 3, 3, False))):
        cfg, w = loud_key_model(size, keep)
        a, b = loud([3 + i % 50 for i in range(80)], at)
        r = replay(U.write(tmp_path / str(n), cfg, w), dtype)
        got = U.feed(r, "a", a, cuts)
        within(got, cfg, w, a, limits(dtype, cfg, w)(a))
        d = (U.feed(r, "b", b, cuts) - got).abs().amax(-1)
        assert d[at + size - 1] > 0.3
        assert d[at + size:].min() > 0.3 if shows \
            else d[at + size:].max() == 0


def test_large_layers_in_bfloat16(tmp_path):
    """Sizes of the padded kernels' largest cases, and several tiles."""
    cfg = U.config([
        U.window(heads=18, kv_heads=2, dim=128, vdim=128, size=150, keep=70,
                 scale=0.1, rot=64, mlp=U.dense(2056)),
        U.latent(heads=18, dim=128, rot_dim=64, vdim=128, kv_rank=512,
                 scale=0.1, mlp=U.dense(512)),
        U.window(heads=3, kv_heads=3, dim=256, vdim=256, size=100, keep=4,
                 scale=0.1, rot=256, mlp=None)],
        width=256, vocab=300, loop=(1, 2, 2))
    w = U.weights(cfg, seed=4)
    r = replay(U.write(tmp_path, cfg, w), "bfloat16")
    toks = U.tokens(330, cfg["vocab"], seed=2)
    lim = limits("bfloat16", cfg, w)(toks)
    for i, cuts in enumerate(([330], [130, 1, 2, 140], [300, 1])):
        within(U.feed(r, f"a{i}", toks, cuts), cfg, w, toks, lim)


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_match_eager(model, dtype):
    """Decode graphs replayed again and again, batch sizes changing, eager
    steps in between."""
    cfg, w, folder = model
    a, b = replay(folder, dtype), replay(folder, dtype, eager=True)
    toks = [U.tokens(60, cfg["vocab"], seed=s) for s in range(4)]
    for r in (a, b):
        r.step([{"id": str(i), "tokens": t[:20 + i]}
                for i, t in enumerate(toks)])
    for n in range(20):
        who = [i for i in range(4) if (n + i) % 4 or n % 5 == 0]
        step = [{"id": str(i), "tokens": [toks[i][30 + n]], "want": [0]}
                for i in who]
        x, y = a.step(step), b.step(step)
        assert U.error(x, y.double()) < 2e-2 * (dtype == "bfloat16") + 1e-5
        torch.cuda.synchronize()
    assert a.engine.runner._graphs and not b.engine.runner._graphs


@pytest.mark.parametrize("dtype", DTYPES)
def test_prefill_graph_matches_eager(model, dtype):
    """Captured prompts, and decoding from what they left in the pages."""
    cfg, w, folder = model
    outs = []
    for eager in (False, True):
        eng = LLMEngine(EngineConfig(
            model=folder, dtype=dtype, max_num_seqs=4, max_model_len=512,
            num_gpu_blocks=128, enforce_eager=eager,
            prefill_graph_sizes=(128, 256)), device=DEV)
        logits = []
        for rep in range(3):
            for n in (5, 100, 128, 130, 255):
                from hyperspot.engine.request import Request
                toks = U.tokens(n + 1, cfg["vocab"], seed=n)
                req = Request(f"{rep}-{n}", toks[:n], SamplingParams())
                for tail in (n, 1):
                    batch = eng.scheduler.schedule_portions([(req, tail)])
                    logits.append(eng.runner.forward(batch).float().cpu()
                                  .clone())
                    req.prompt_token_ids.append(toks[n])
                eng.scheduler.release(req)
        outs.append(torch.cat(logits))
        assert bool(eng.runner._pgraphs) != eager
    assert U.error(outs[0], outs[1].double()) < (3e-2 if dtype == "bfloat16"
                                                 else 1e-5)


@pytest.mark.parametrize("kw", [
    {}, {"mixed_batches": True, "max_num_batched_tokens": 24},
    {"max_num_seqs": 2, "enforce_eager": True}])
def test_greedy_generation_float32(model, kw):
    cfg, w, folder = model
    prompts = [U.tokens(n, cfg["vocab"], seed=20 + n) for n in (5, 40, 1, 23)]
    base = dict(model=folder, dtype="float32", max_num_seqs=4,
                max_num_batched_tokens=64, max_model_len=256,
                num_gpu_blocks=64, graph_batch_sizes=(1, 2, 4))
    base.update(kw)
    got = LLMEngine(EngineConfig(**base), device=DEV).generate(
        prompts, SamplingParams(temperature=0.0, max_tokens=12))
    assert got == [O.greedy(cfg, w, p, 12) for p in prompts]
