"""Mutusun on the GPU: every kernel against the plain float64 implementation,
and whole models in bfloat16 and float32 through prefill, decode graphs,
portions and mixed batches."""

import copy

import pytest
import torch

import mutusun_oracle as O
import mutusun_util as U
from hyperspot import ops
from hyperspot.engine import EngineConfig, LLMEngine, SamplingParams
from hyperspot.engine.kv_cache import KVPages
from hyperspot.engine.replay import Replay
from hyperspot.models.llama import ForwardMeta, prefill_tiles
from hyperspot.ops import experts, hybrid

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


def ints(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


def tol(dtype):
    return 2e-5 if dtype == F32 else 2e-2


def meta_for(starts, lens, decode=False, slots=None):
    """Metadata for portions [start, start + len) of as many sequences, with
    shuffled pages, as the runner makes it."""
    n, ends = len(lens), [a + b for a, b in zip(starts, lens)]
    nblk = (max(ends) + 15) // 16
    g = torch.Generator().manual_seed(5)
    bt = torch.randperm(n * nblk, generator=g).int().view(n, nblk)
    ss = [0]
    for x in lens:
        ss.append(ss[-1] + x)
    pos = torch.tensor([p for a, b in zip(starts, ends) for p in range(a, b)])
    seq = torch.tensor([i for i, x in enumerate(lens) for _ in range(x)])
    t64, ts = prefill_tiles(lens)
    return ForwardMeta(
        mode="decode" if decode else "prefill", positions=pos.to(DEV),
        slot_mapping=(bt[seq, pos // 16].long() * 16 + pos % 16).to(DEV),
        seq_start=ints(ss), row_seq=seq.int().to(DEV),
        block_tables=bt.to(DEV),
        state_slots=ints(list(range(n)) if slots is None else slots),
        tiles=ints(t64), tile_start=ints(ts)), n * nblk


# ------------------------------------------------------- between sublayers

@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("width", [8, 57, 1000, 2304, 4100, 5004])
def test_add_and_norms(dtype, width):
    y = rand(5, width, seed=9, gain=2, dtype=dtype)
    res, post, pre = (rand(*s, seed=i) for i, s in
                      enumerate(((5, width), (width,), (width,))))
    m, _ = meta_for([0], [5])
    nxt = hybrid.NextInput(pre.to(DEV), 1e-3)
    r = res.to(DEV)
    h = hybrid.next_input(r, nxt, m, dtype)
    assert rel(h, O.rms(f64(res), 1e-3) * f64(pre)) < tol(dtype)
    assert torch.equal(r.cpu(), res)
    h = hybrid.add_rms_next(y.to(DEV), r, post.to(DEV), nxt, m)
    want = f64(res) + O.rms(f64(y), 1e-3) * f64(post)
    assert rel(r, want) < 1e-5
    assert rel(h, O.rms(want, 1e-3) * f64(pre)) < tol(dtype)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 9, 10, 70])
@pytest.mark.parametrize("width", [20, 33, 1500])
def test_convolution(dtype, taps, width):
    """One sequence in portions down to single tokens, decoded tokens through
    the fused step, beside another sequence and one that keeps nothing.  The
    slots start out as garbage."""
    T = 260
    x, w = rand(T, width), rand(width, taps, seed=1, gain=0.5)
    pre = rand(width, seed=3)
    conv = w.t().contiguous().to(DEV)
    tail = torch.full((4, taps - 1, width), float("nan"), dtype=dtype,
                      device=DEV)
    nxt = hybrid.NextInput(pre.to(DEV), 1e-3, conv, tail)
    res = x.to(DEV)
    # inputs as the layer makes them, in its element type
    h = f64((O.rms(f64(x), 1e-3) * f64(pre)).to(dtype))
    out, at = [], 0
    for n in (1, 1, 2, 70, 1, 3, 130, 1, 51):
        if n == 1 and at:
            m, _ = meta_for([at, 0, 3], [1] * 3, True, [2, 1, -1])
            y = hybrid.next_input(
                torch.cat([res[at:at + 1], res[:1], res[:1]]), nxt, m, dtype)
            y = y[:1]
        else:
            m, _ = meta_for([at, 0, 0], [n, 65, 3], False, [2, 1, -1])
            y = hybrid.next_input(
                torch.cat([res[at:at + n], res[:65], res[:3]]), nxt, m, dtype)
            want = O.causal_conv(h[:65], f64(w))
            assert rel(y[n:n + 65], want) < tol(dtype)
            assert rel(y[n + 65:], want[:3]) < tol(dtype)
        out.append(y[:n])
        at += n
    assert at == T
    assert rel(torch.cat(out), O.causal_conv(h, f64(w))) < tol(dtype)
    assert tail[[0, 3]].isnan().all()
    if taps > 1:
        last = torch.cat([torch.zeros(70, width).double(), h])[1 - taps:]
        assert (f64(tail[2]) - last).abs().max() < 2e-2 * (dtype == BF) + 1e-5


@pytest.mark.parametrize("dtype", [BF, F32])
def test_convolution_batch_equals_each_alone(dtype):
    lens, starts, W = [70, 1, 2, 64, 129], [0, 17, 64, 5, 300], 96
    h = rand(sum(lens), W, dtype=dtype).to(DEV)
    conv = rand(4, W, seed=1).to(DEV)
    first = rand(5, 3, W, seed=3, dtype=dtype).to(DEV)
    together, row = first.clone(), 0
    got = hybrid.causal_conv(h, conv, together, meta_for(starts, lens)[0])
    for i, n in enumerate(lens):
        alone = first.clone()
        m = meta_for([starts[i]], [n], slots=[i])[0]
        y = hybrid.causal_conv(h[row:row + n].contiguous(), conv, alone, m)
        assert torch.equal(y, got[row:row + n])
        assert torch.equal(alone[i], together[i])
        row += n


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("n", [1, 7, 24, 2048])
def test_activations(dtype, n):
    x = rand(5, 2 * n, gain=3, dtype=dtype)
    x[0, 0], x[1, 0], x[2, -1] = -40, 40, -40
    g, u = f64(x).chunk(2, -1)
    for limit in (0.5, 7.0):
        a = g.clamp(max=limit)
        want = a * torch.sigmoid(1.702 * a) * (u.clamp(-limit, limit) + 1)
        assert rel(hybrid.clamped_glu(x.to(DEV), limit), want) < tol(dtype)
    assert rel(hybrid.squared_relu(x.to(DEV)),
               f64(x).clamp(min=0) ** 2) < tol(dtype)


# --------------------------------------------------------------- attention

@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,G,D,E", [(4, 2, 16, 24), (6, 3, 7, 5),
                                     (16, 4, 128, 128), (3, 1, 96, 40),
                                     (1, 1, 1, 1), (2, 2, 520, 8)])
@pytest.mark.parametrize("lens", [[15, 25], [1500], [4200]])
def test_norm_append(dtype, H, G, D, E, lens):
    m, nb = meta_for([900] * len(lens), lens)
    T = sum(lens)
    buf = rand(T, (H + G) * D + G * E + 8, dtype=dtype)
    b = buf.to(DEV)
    q, k, v, _ = b.split([H * D, G * D, G * E, 8], -1)
    qw, kw = rand(D, seed=3), rand(D, seed=4)
    slots = m.slot_mapping.cpu()
    m.slot_mapping[-1] = -1
    cache = KVPages(torch.full((nb, G, 16, D), 9.0, dtype=dtype, device=DEV),
                    torch.full((nb, G, E, 16), 9.0, dtype=dtype, device=DEV))
    hybrid.norm_append(q, k, v, qw.to(DEV), kw.to(DEV), m, cache, 1e-4)
    x = f64(buf)
    heads = lambda a, n, d: x[:, a:a + n * d].view(T, n, d)
    assert rel(q.reshape(T, H, D), O.rms(heads(0, H, D), 1e-4) * f64(qw)) \
        < tol(dtype)
    kf = cache.k.permute(0, 2, 1, 3).reshape(-1, G, D).cpu()
    vf = cache.v.permute(0, 3, 1, 2).reshape(-1, G, E).cpu()
    assert rel(kf[slots[:-1]],
               (O.rms(heads(H * D, G, D), 1e-4) * f64(kw))[:-1]) < tol(dtype)
    assert torch.equal(f64(vf[slots[:-1]]),
                       heads((H + G) * D, G, E)[:-1])
    assert (kf[slots[-1]] == 9.0).all() and (vf[slots[-1]] == 9.0).all()
    assert torch.equal(b[:, -8:].cpu(), buf[:, -8:])


def attention_case(H, G, D, E, chunk, starts, lens, dtype, decode=False,
                   loud=(), scale=None, cap=6.0):
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
    buf = rand(sum(lens), H * D + 8, seed=4, dtype=dtype)
    bias = rand(H, seed=6)
    scale = scale or 1.5 * D ** -0.5
    got = hybrid.sigmoid_attention(
        buf.to(DEV)[:, :H * D], KVPages(kc.to(DEV), vc.to(DEV)), m,
        bias.to(DEV), chunk, scale, cap)
    want, row, x = [], 0, f64(buf)
    for i in range(n):
        ki, vi = f64(k[i]), f64(v[i])
        for p in range(starts[i], starts[i] + lens[i]):
            lo = O.chunk_start(p, chunk)
            q = x[row, :H * D].view(G, H // G, D)
            s = torch.einsum("gxd,ngd->gxn", q, ki[lo:p + 1]) * scale
            a = torch.sigmoid(O.capped(s, cap)
                              + f64(bias).view(G, H // G, 1))
            want.append(torch.einsum("gxn,nge->gxe", a,
                                     vi[lo:p + 1]).reshape(-1))
            row += 1
    return got, torch.stack(want)


SIZES = [(2, 1, 8, 8), (6, 2, 64, 48), (3, 3, 48, 40), (16, 4, 128, 128),
         (17, 1, 16, 128), (40, 2, 32, 16), (4, 1, 64, 256), (3, 1, 120, 200),
         (4, 2, 256, 256), (5, 5, 200, 136), (6, 3, 7, 9), (1, 1, 1, 1),
         (2, 1, 16, 600)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,G,D,E", SIZES)
def test_attention_prefill(dtype, H, G, D, E):
    """Portions with and without earlier tokens in one step; starts and ends
    off every tile, page and chunk border."""
    got, want = attention_case(H, G, D, E, 37, [0, 50, 0, 21, 3],
                               [70, 17, 5, 16, 30], dtype)
    assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("chunk", [1, 2, 31, 32, 64, 65, 200, 5000, 1 << 30])
def test_attention_prefill_chunks(dtype, chunk):
    got, want = attention_case(2, 1, 16, 24, chunk, [0, 130], [300, 140],
                               dtype)
    assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("D,E", [(16, 24), (40, 128), (128, 128), (64, 200),
                                 (104, 256), (256, 256)])
@pytest.mark.parametrize("chunk", [45, 300])
def test_attention_prefill_by_pairs_of_heads(D, E, chunk):
    """Enough tiles and heads that one workgroup takes two heads."""
    got, want = attention_case(64, 2, D, E, chunk, [0, 333, 70],
                               [700, 300, 30], BF)
    assert rel(got, want) < 2e-2


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,G,D,E", SIZES)
@pytest.mark.parametrize("rows", [1, 20])
def test_attention_decode(dtype, H, G, D, E, rows):
    ctx = [0, 15, 16, 17, 31, 32, 300, 301, 255, 256][:rows] * 2
    ctx = ([300] if rows == 1 else ctx)[:rows]
    for chunk in (37, 256, 400):
        got, want = attention_case(H, G, D, E, chunk, ctx, [1] * rows, dtype,
                                   decode=True)
        assert rel(got, want) < tol(dtype)


def test_decode_of_many_rows_is_not_split():
    assert hybrid.decode_split(520, 400) == 1
    got, want = attention_case(2, 1, 16, 24, 60, [i % 70 for i in range(520)],
                               [1] * 520, BF, decode=True)
    assert rel(got, want) < 2e-2


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("scale,cap", [(0.1, 0.5), (2.0, 300.0), (-0.7, 3.0),
                                       (30.0, 20.0)])
def test_caps(dtype, scale, cap):
    """Scores far below, around and far above the cap."""
    for decode in (False, True):
        got, want = attention_case(4, 2, 16, 24, 50, [45], [1 if decode
                                                            else 60],
                                   dtype, decode, scale=scale, cap=cap)
        assert rel(got, want) < tol(dtype)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("lens", [[1], [2], [16], [17], [80]])
def test_loud_key_at_the_chunk_edge(dtype, lens):
    """One key far above all others, last in its chunk, first seen from
    outside by the next position; and one first in its chunk."""
    chunk, at = 20, 59
    for first in (at, at + 1):
        got, want = attention_case(2, 1, 16, 24, chunk, [first], lens, dtype,
                                   decode=lens == [1], loud=[(0, at)])
        assert rel(got, want) < tol(dtype)
        quiet = attention_case(2, 1, 16, 24, chunk, [first], lens, dtype,
                               decode=lens == [1])[1]
        moved = rel(want[:1], quiet[:1])
        assert moved > 0.3 if first == at else moved == 0
    for first in (60, 79, 80):
        got, want = attention_case(2, 1, 16, 24, chunk, [first], lens, dtype,
                                   decode=lens == [1], loud=[(0, 60)])
        assert rel(got, want) < tol(dtype)


# ----------------------------------------------------------------- experts

def expert_case(T, W, E, identity, top, F, dtype, limit=0.8):
    n = E + identity
    x = rand(T, W, dtype=dtype)
    router = rand(n, W, seed=1, gain=W ** -0.5, dtype=dtype)
    corr = rand(n, seed=5, gain=0.3)
    up = rand(E, 2 * F, W, seed=2, gain=W ** -0.5, dtype=dtype)
    down = rand(E, W, F, seed=3, gain=F ** -0.5, dtype=dtype)
    w = {}
    for i in range(E):
        w.update({f"e{i}.gate": f64(up[i, :F]), f"e{i}.up": f64(up[i, F:]),
                  f"e{i}.down": f64(down[i])})
    args = [t.to(DEV) for t in (x, router, up, down)] + [None, None, top]
    rules = experts.Rules(corr.to(DEV), identity, limit)
    # experts as the kernels choose them: a close call may go either way
    z = f64(hybrid.gate_projection(args[0], args[1]))
    ids, weight = O.route(z, f64(corr), top)
    want = torch.zeros(T, W, dtype=torch.float64)
    part = torch.zeros_like(want)
    for t in range(T):
        for j in range(top):
            e = int(ids[t, j])
            if e >= E:
                part[t] += weight[t, j] * f64(x)[t]
            else:
                want[t] += weight[t, j] * O.expert(f64(x)[t], w, f"e{e}.",
                                                   limit)
    return args, rules, want, part


CASES = [(1, 64, 5, 3, 2, 24), (3, 24, 1, 0, 1, 8), (40, 64, 8, 2, 3, 56),
         (100, 72, 4, 4, 8, 40), (33, 264, 50, 20, 5, 16),
         (90, 32, 280, 20, 2, 8), (200, 128, 3, 1, 2, 128),
         (300, 128, 2, 1, 2, 256), (7, 21, 6, 3, 2, 5), (2, 3, 2, 1, 2, 1),
         (12, 32, 2, 30, 3, 8), (2, 5000, 3, 1, 2, 16)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("T,W,E,identity,top,F", CASES)
def test_mixture(dtype, T, W, E, identity, top, F):
    args, rules, want, part = expert_case(T, W, E, identity, top, F, dtype)
    assert rel(experts.mixture(*args, rules), want + part) < tol(dtype)
    got = experts.mixture(*args, rules._replace(identity_here=False))
    d = (f64(got) - want).flatten(1).pow(2).mean(-1).sqrt().max()
    assert float(d / (want + part).pow(2).mean().sqrt()) < tol(dtype)
    # the whole step to the next input, in a prompt and decoding
    res, w, pre = rand(T, W, seed=8), rand(W, seed=9), rand(W, seed=10)
    conv = rand(3, W, seed=11)
    total = f64(res) + O.rms(want + part, 1e-3) * f64(w)
    h = O.rms(total, 1e-3) * f64(pre)
    for decode in (False, True):
        m, _ = meta_for([0] * T, [1] * T, True) if decode \
            else meta_for([0], [T])
        r = res.to(DEV)
        tail = torch.full((T, 2, W), 7.0, dtype=dtype, device=DEV)
        nxt = hybrid.NextInput(pre.to(DEV), 1e-3, conv.to(DEV), tail)
        got = experts.mixture_add_next(*args, rules, r, w.to(DEV), nxt, m)
        assert got.dtype == dtype and rel(r, total) < tol(dtype)
        after = h * (1 + f64(conv[2])) if decode \
            else O.causal_conv(h, f64(conv).T)
        assert rel(got, after) < 2 * tol(dtype)
    r = res.to(DEV)
    x = experts.mixture_add_rms(*args, r, w.to(DEV), 1e-3, rules)
    assert rel(r, total) < tol(dtype) and rel(x, total) < tol(dtype)


def test_mixture_paths(monkeypatch):
    """The same step through tiles of 16, 32 and 64 rows and of 256 rows."""
    native, seen = ops._native(), []

    class Spy:
        def __getattr__(self, name):
            def call(*a):
                if name in ("experts_up", "moe_gemm"):
                    seen.append(a[-1] if name == "experts_up" else 256)
                return getattr(native, name)(*a)
            return call

    monkeypatch.setattr(experts, "_native", lambda: Spy())
    for T in (30, 110, 190, 600):
        args, rules, want, part = expert_case(T, 128, 8, 2, 2, 128, BF)
        assert rel(experts.mixture(*args, rules), want + part) < 2e-2
    assert list(dict.fromkeys(seen)) == [16, 32, 64, 256]


def test_routing_ties_and_broken_rows():
    """Equal shares: the lowest numbers win; a row that is not a number still
    gets valid choices; identity experts are -1, weights are not renormed."""
    E, identity, top = 66, 4, 3
    n = E + identity
    z = torch.zeros(5, n)
    z[1, 69] = z[1, 64] = z[1, 2] = 2.0
    z[2] = float("nan")
    z[3] = torch.arange(float(n))
    z[4, :2] = float("-inf")
    corr = torch.zeros(n)
    wt = torch.empty(5, top, device=DEV)
    ids = torch.empty(5, top, dtype=torch.int32, device=DEV)
    route = lambda: ops._native().experts_route(
        wt, ids, z.to(DEV), E, top, corr.to(DEV), identity)
    route()
    assert ids.tolist() == [[0, 1, 2], [2, 64, -1], [0, 1, 2], [-1, -1, -1],
                            [2, 3, 4]]
    p = z[[0, 1, 3, 4]].softmax(-1)
    want = torch.stack([p[0, :3], p[1, [2, 64, 69]], p[2, [69, 68, 67]],
                        p[3, 2:5]])
    assert torch.allclose(wt[[0, 1, 3, 4]].cpu(), want)
    corr[50] = 2.0                   # chosen first, weight unchanged
    route()
    assert ids[:, 0].tolist() == [50] * 5
    assert torch.allclose(wt[1, 0].cpu(), p[1, 50])


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


def all_chosen(cfg):
    """Every token uses every expert: 16-bit rounding changes no choice."""
    c = copy.deepcopy(cfg)
    for layer in c["layers"]:
        if layer["mlp"] and layer["mlp"]["kind"] == "moe":
            r = layer["mlp"]["router"]
            r["top"] = r["experts"] + r["identity"]
    return c


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """dtype -> configuration, weights, folder"""
    out = {}
    for dtype, cfg in (("float32", U.standard()),
                       ("bfloat16", all_chosen(U.standard()))):
        w = U.weights(cfg, seed=1)
        out[dtype] = cfg, w, U.write(tmp_path_factory.mktemp(dtype), cfg, w)
    return out


def replay(folder, dtype, max_tokens=512, eager=False):
    return Replay(folder, dtype, max_tokens, device=DEV, eager=eager)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[200], [1], [2], [63, 65, 2, 5], [30, 1]])
def test_model_portions(models, dtype, cuts):
    cfg, w, folder = models[dtype]
    toks = U.tokens(200, cfg["vocab"], seed=1)
    within(U.feed(replay(folder, dtype), "a", toks, cuts), cfg, w, toks,
           limits(dtype, cfg, w)(toks))


@pytest.mark.parametrize("dtype", DTYPES)
def test_model_mixed_batches_reuse(models, dtype):
    from test_mutusun import fill_caches, mixed_run
    cfg, w, folder = models[dtype]
    r = replay(folder, dtype, 4 * 128)
    fill_caches(r, 5.0)
    lens = [70, 3, 120, 41, 1, 90, 17, 64, 33, 2]
    assert mixed_run(r, cfg, w, lens, limits=limits(dtype, cfg, w)) < 1
    assert r.engine.runner.block_manager.num_free_rows == 4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", [
    "ones", "odd", "many taps", "two taps", "one of each run thrice",
    "negative scale, tight cap", "many heads", "identity mostly",
    "equal sizes"])
def test_model_other_sizes(tmp_path, dtype, name):
    from test_mutusun import ODD, mixed_run
    cfg = ODD[name] if dtype == "float32" else all_chosen(ODD[name])
    w = U.weights(cfg, seed=6)
    r = replay(U.write(tmp_path, cfg, w), dtype)
    toks = U.tokens(50, cfg["vocab"])
    lim = limits(dtype, cfg, w)
    for i, cuts in enumerate(([50], [20, 1], [2])):
        within(U.feed(r, f"a{i}", toks, cuts), cfg, w, toks, lim(toks))
    assert mixed_run(r, cfg, w, [30, 9, 21], limits=lim) < 1


@pytest.mark.parametrize("cuts", [[80], [10, 1], [30, 2, 1], [16, 17, 2]])
@pytest.mark.parametrize("dtype", DTYPES)
def test_model_chunk_edge(tmp_path, dtype, cuts):
    from test_mutusun import loud_key_model
    cfg, w = loud_key_model()
    toks = [3 + i % 50 for i in range(80)]
    toks[7] = 1
    r = replay(U.write(tmp_path, cfg, w), dtype)
    got = U.feed(r, "a", toks, cuts)
    within(got, cfg, w, toks, limits(dtype, cfg, w)(toks))
    toks[7] = 2
    d = (U.feed(r, "b", toks, cuts) - got).abs().amax(-1)
    assert d[32] > 0.3 and d[33:].max() == 0


def test_large_layers_in_bfloat16(tmp_path):
    """Sizes of the padded kernels' largest cases and the 256-row tiles."""
    own = [U.layer(heads=18, kv_heads=2, dim=128, vdim=128, chunk=150,
                   scale=0.2, mlp=U.moe(2, 1, 3, 128, 2.0)),
           U.layer(heads=3, kv_heads=3, dim=256, vdim=256, chunk=100,
                   scale=0.1, mlp=U.dense(512))]
    cfg = U.config(own + [U.again(own, 0)], width=256, vocab=300)
    w = U.weights(cfg, seed=4)
    r = replay(U.write(tmp_path, cfg, w), "bfloat16")
    toks = U.tokens(330, cfg["vocab"], seed=2)
    lim = limits("bfloat16", cfg, w)(toks)
    for i, cuts in enumerate(([330], [130, 1, 2, 140], [300, 1])):
        within(U.feed(r, f"a{i}", toks, cuts), cfg, w, toks, lim)


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_match_eager(models, dtype):
    """Decode graphs replayed again and again, batch sizes changing, eager
    steps in between."""
    cfg, w, folder = models[dtype]
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
        assert U.error(x, y.double()) < 1e-2 * (dtype == "bfloat16") + 1e-5
        torch.cuda.synchronize()
    assert a.engine.runner._graphs and not b.engine.runner._graphs


@pytest.mark.parametrize("dtype", DTYPES)
def test_prefill_graph_matches_eager(models, dtype):
    """Captured prompts, and decoding from what they left in the slots."""
    cfg, w, folder = models[dtype]
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
    assert U.error(outs[0], outs[1].double()) < (2e-2 if dtype == "bfloat16"
                                                 else 1e-5)


@pytest.mark.parametrize("kw", [
    {}, {"mixed_batches": True, "max_num_batched_tokens": 24},
    {"max_num_seqs": 2, "enforce_eager": True}])
def test_greedy_generation_float32(models, kw):
    cfg, w, folder = models["float32"]
    prompts = [U.tokens(n, cfg["vocab"], seed=20 + n) for n in (5, 40, 1, 23)]
    base = dict(model=folder, dtype="float32", max_num_seqs=4,
                max_num_batched_tokens=64, max_model_len=256,
                num_gpu_blocks=64, graph_batch_sizes=(1, 2, 4))
    base.update(kw)
    got = LLMEngine(EngineConfig(**base), device=DEV).generate(
        prompts, SamplingParams(temperature=0.0, max_tokens=12))
    assert got == [O.greedy(cfg, w, p, 12) for p in prompts]
