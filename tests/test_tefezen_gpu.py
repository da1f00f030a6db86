"""Tefezen on the GPU: every kernel against the plain float64 implementation,
and whole models in bfloat16 and float32 through prefill, decode graphs,
portions and mixed batches."""

import copy

import pytest
import torch

import tefezen_oracle as O
import tefezen_util as U
from hyperspot import ops
from hyperspot.engine import EngineConfig, LLMEngine, SamplingParams
from hyperspot.engine.kv_cache import LatentKV, RecurrentState
from hyperspot.engine.replay import Replay
from hyperspot.models.llama import (ABSORB_TOKENS, SPAN_TOKENS, ForwardMeta,
                                    LatentSpan, prefill_tiles)
from hyperspot.ops import experts, hybrid, latent

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


def dev(*tensors):
    return [t.to(DEV) for t in tensors]


# ---------------------------------------------------------------- residual

@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("width", [8, 57, 1000, 2304, 5004])
def test_residual_kernels(dtype, width):
    tol = 1e-5 if dtype == F32 else 1e-2
    table, ids = rand(40, width, seed=1, dtype=dtype), [3, 39, 0, 3, 17]
    w = rand(width, seed=2)
    x, res = hybrid.embed_scaled(table.to(DEV),
                                 torch.tensor(ids, device=DEV), 3.5)
    want = f64(table)[ids] * 3.5
    assert rel(res, want) < 1e-6 and rel(x, want) < tol
    assert (x is res) == (dtype == F32)
    h = rand(5, width, seed=9, gain=2, dtype=dtype)
    x = hybrid.add_rms(h.to(DEV), res, w.to(DEV), 1e-3, dtype)
    want = want + O.rms(f64(h), 1e-3) * f64(w)
    assert rel(res, want) < 1e-5 and rel(x, want) < tol
    assert rel(hybrid.rms_scale(res, w.to(DEV), 1e-3, dtype),
               O.rms(want, 1e-3) * f64(w)) < tol
    # norm over all columns, gate from a column view of a wider buffer
    buf = rand(5, width + 12, seed=5, dtype=dtype)
    g = buf[:, 4:4 + width]
    o = rand(5, width, seed=6)
    want = O.rms(f64(o), 1e-3) * f64(w) * torch.sigmoid(f64(g))
    gd = buf.to(DEV)[:, 4:4 + width]
    assert rel(hybrid.rms_gate(o.to(DEV), gd, w.to(DEV), 1e-3, None, width),
               want) < tol
    ss = hybrid.row_squares(o.to(DEV))
    assert rel(ss[:, None], f64(o).pow(2).sum(-1, keepdim=True)) < 1e-5
    assert rel(hybrid.rms_gate(o.to(DEV), gd, w.to(DEV), 1e-3, 2 * ss,
                               2 * width), want) < tol


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("n,cols,column", [(3, 10, 5), (16, 64, 32),
                                           (128, 512, 384)])
def test_gelu_gate(dtype, n, cols, column):
    z, table = rand(7, n, gain=2, dtype=dtype), rand(9, cols, dtype=dtype)
    ids = [8, 0, 1, 8, 3, 2, 2]
    want = O.gelu_tanh(f64(z)) * f64(table)[ids, column:column + n]
    got = hybrid.gelu_gate(*dev(z, table, torch.tensor(ids)), column)
    assert rel(got, want) < (1e-5 if dtype == F32 else 1e-2)


# -------------------------------------------------------- latent attention

def meta_for(starts, lens, window, decode=False):
    """Metadata for portions [start, start + len) of as many sequences, with
    shuffled pages, as the runner makes it."""
    n, ends = len(lens), [a + b for a, b in zip(starts, lens)]
    nblk = (max(ends) + 15) // 16
    g = torch.Generator().manual_seed(5)
    bt = torch.randperm(n * nblk, generator=g).int().view(n, nblk)
    ss, row0 = [0], 0
    for x in lens:
        ss.append(ss[-1] + x)
    pos = torch.tensor([p for a, b in zip(starts, ends) for p in range(a, b)])
    seq = torch.tensor([i for i, x in enumerate(lens) for _ in range(x)])
    slot = lambda i, p: bt[i, p // 16].long() * 16 + p % 16
    kv, first, start, tiles, rows = [], [], [], [], []
    for i, (a, m) in enumerate(zip(starts, lens)):
        start.append(len(kv))
        first.append(max(0, a - window + 1))
        if m <= ABSORB_TOKENS:
            rows += range(row0, row0 + m)
        else:
            kv += slot(i, torch.arange(first[-1], a + m)).tolist()
            kv += [-1] * (-len(kv) % 8)
            tiles += [[i, t] for t in range(0, m, SPAN_TOKENS)]
        row0 += m
    span = LatentSpan(
        torch.tensor(kv, dtype=torch.long, device=DEV), ints(start),
        ints(first), ints(tiles).view(-1, 2), ints(rows) if rows else None)
    t64, ts = prefill_tiles(lens)
    return ForwardMeta(
        mode="decode" if decode else "prefill", positions=pos.to(DEV),
        slot_mapping=slot(seq, pos).to(DEV), seq_start=ints(ss),
        row_seq=seq.int().to(DEV), block_tables=bt.to(DEV),
        state_slots=ints(list(range(n))), tiles=ints(t64),
        tile_start=ints(ts), latent={window: span}), n * nblk


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,D,R,rank", [(2, 8, 8, 16), (3, 7, 6, 9),
                                        (16, 128, 64, 512), (1, 5, 0, 3)])
def test_rope_append(dtype, H, D, R, rank):
    tol = 1e-5 if dtype == F32 else 1e-2
    T = 40
    m, nb = meta_for([0, 90000], [15, 25], 10)
    buf = rand(T, H * (D + R) + rank + R, dtype=dtype)
    b = buf.to(DEV)
    q, kv = b.split([H * (D + R), rank + R], -1)
    w = rand(rank, seed=3)
    cache = LatentKV(torch.full((nb, 16, rank + R), 9.0, dtype=dtype,
                                device=DEV))
    slots = m.slot_mapping.cpu()
    m.slot_mapping[-1] = -1
    fr = 3e4 ** (-torch.arange(0, R, 2).double() / max(R, 1))
    latent.rope_append(q, kv, w.to(DEV), m, fr.to(DEV), cache, H, 1e-4)
    pos, x = m.positions.cpu(), f64(buf)
    for h in range(H):
        a = h * (D + R)
        assert torch.equal(q[:, a:a + D].cpu(), buf[:, a:a + D])
        if R:
            assert rel(q[:, a + D:a + D + R], O.rotate_pairs(
                x[:, a + D:a + D + R], pos, R, 3e4)) < tol
    raw = x[:, H * (D + R):]
    want = O.rms(raw[:, :rank], 1e-4) * f64(w)
    if R:
        want = torch.cat([want, O.rotate_pairs(raw[:, rank:], pos, R, 3e4)],
                         -1)
    flat = cache.kv.view(-1, rank + R).cpu()
    assert rel(flat[slots[:-1]], want[:-1]) < tol
    assert (flat[slots[-1]] == 9.0).all()          # slot -1 kept nothing


def attention_case(H, D, R, E, rank, window, starts, lens, dtype,
                   decode=False, loud=(), gain=0.5):
    m, nb = meta_for(starts, lens, window, decode)
    n, longest = len(lens), max(a + b for a, b in zip(starts, lens))
    rows = rand(n, longest, rank + R, seed=2, gain=gain, dtype=dtype)
    for s, at in loud:
        rows[s, at] *= 8
    # what no sequence holds must not matter
    cache = torch.full((nb, 16, rank + R), 1e4, dtype=dtype)
    bt = m.block_tables.cpu()
    for i in range(n):
        for p in range(starts[i] + lens[i]):
            cache[bt[i, p // 16], p % 16] = rows[i, p]
    buf = rand(sum(lens), H * (D + R) + 8, seed=4, dtype=dtype)
    uk = rand(rank, H * D, seed=6, gain=rank ** -0.5, dtype=dtype)
    uv = rand(H * E, rank, seed=7, gain=rank ** -0.5, dtype=dtype)
    scale = 1.3 * (D + R) ** -0.5
    q = buf.to(DEV)[:, :H * (D + R)]
    got = latent.attention(q, LatentKV(cache.to(DEV)), m, uk.to(DEV),
                           uv.to(DEV), H, window, scale)
    want, row = [], 0
    x, k, v = f64(buf), f64(uk), f64(uv)
    for i in range(n):
        c, kr = f64(rows[i])[:, :rank], f64(rows[i])[:, rank:]
        for p in range(starts[i], starts[i] + lens[i]):
            lo, out = max(0, p - window + 1), []
            for h in range(H):
                qh = x[row, h * (D + R):(h + 1) * (D + R)]
                key = torch.cat([c[lo:p + 1] @ k[:, h * D:(h + 1) * D],
                                 kr[lo:p + 1]], -1)
                a = (key @ qh * scale).softmax(0)
                out.append(a @ (c[lo:p + 1] @ v[h * E:(h + 1) * E].T))
            want.append(torch.cat(out))
            row += 1
    return got, torch.stack(want)


SIZES = [(2, 8, 8, 8, 16), (5, 64, 32, 48, 104), (3, 48, 16, 40, 72),
         (16, 24, 8, 32, 128), (17, 16, 24, 128, 200), (2, 128, 64, 128, 512),
         (33, 32, 64, 16, 256), (1, 192, 64, 256, 512), (2, 96, 32, 256, 64),
         (3, 7, 6, 9, 11), (1, 1, 2, 1, 1), (2, 16, 80, 24, 600)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,D,R,E,rank", SIZES)
def test_attention_prefill(dtype, H, D, R, E, rank):
    """Long and short portions with and without earlier tokens in one step;
    starts and ends off every tile and page border."""
    got, want = attention_case(H, D, R, E, rank, 37, [0, 50, 0, 21, 3],
                               [70, 17, 5, 16, 30], dtype)
    assert rel(got, want) < (2e-5 if dtype == F32 else 2e-2)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("window", [1, 2, 31, 64, 65, 200, 5000])
def test_attention_prefill_windows(dtype, window):
    got, want = attention_case(2, 16, 8, 24, 40, window, [0, 130],
                               [300, 140], dtype)
    assert rel(got, want) < (2e-5 if dtype == F32 else 2e-2)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,D,R,E,rank", SIZES)
@pytest.mark.parametrize("rows", [1, 20])
def test_attention_decode(dtype, H, D, R, E, rank, rows):
    ctx = [0, 15, 16, 17, 31, 32, 300, 301, 255, 256][:rows] * 2
    ctx = ([300] if rows == 1 else ctx)[:rows]
    for window in (37, 200):
        got, want = attention_case(H, D, R, E, rank, window, ctx,
                                   [1] * rows, dtype, decode=True)
        assert rel(got, want) < (2e-5 if dtype == F32 else 2e-2)


def test_decode_of_many_rows_is_not_split():
    assert latent.absorbed_split(512, 400) == 1
    got, want = attention_case(2, 16, 8, 24, 40, 60,
                               [i % 70 for i in range(520)], [1] * 520, BF,
                               decode=True)
    assert rel(got, want) < 2e-2


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("lens", [[1], [2], [16], [17], [80]])
def test_loud_key_at_the_window_edge(dtype, lens):
    """One key far above all others, last seen by position 64 + 19."""
    window, at = 20, 64
    for first in (at + window - 1, at + window):
        got, want = attention_case(2, 16, 8, 24, 40, window, [first], lens,
                                   dtype, decode=lens == [1],
                                   loud=[(0, at)])
        assert rel(got, want) < (2e-5 if dtype == F32 else 2e-2)
        quiet = attention_case(2, 16, 8, 24, 40, window, [first], lens,
                               dtype, decode=lens == [1])[1]
        moved = rel(want[:1], quiet[:1])
        assert moved > 0.3 if first < at + window else moved == 0


# ----------------------------------------------------- lightning attention

REC = [(2, 16, 24), (3, 8, 40), (2, 128, 128), (1, 64, 256), (2, 7, 5),
       (1, 1, 1), (1, 130, 300)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("H,D,E", REC)
def test_lightning(dtype, H, D, E):
    """Prompt portions, then decoding; decays from 0 to 1."""
    T = 200
    buf = rand(T, H * (2 * D + E) + 8, seed=1, dtype=dtype)
    decay = torch.tensor([0.999, 0.3, 0.0][:H] if H > 1 else [1.0])
    st = RecurrentState(torch.full((3, H, D, E), 7.0, device=DEV))
    b, out, at = buf.to(DEV), [], 0
    for n in (70, 2, 64, 1, 1, 30, 1, 31):
        m, _ = meta_for([at], [n], 8, decode=n == 1)
        m.state_slots = ints([1])
        q, k, v, _ = b[at:at + n].split([H * D, H * D, H * E, 8], -1)
        out.append(hybrid.lightning_mix(q, k, v, decay.to(DEV), st, m))
        at += n
    assert at == T
    got = torch.cat(out).view(T, H, E)
    q, k, v, _ = O.silu(f64(buf)).split([H * D, H * D, H * E, 8], -1)
    for h in range(H):
        want = O.decayed_recurrence(
            q[:, h * D:(h + 1) * D], k[:, h * D:(h + 1) * D],
            v[:, h * E:(h + 1) * E], float(decay[h]))
        assert rel(got[:, h], want) < (2e-5 if dtype == F32 else 3e-2)
    assert (st.S[[0, 2]] == 7.0).all()


@pytest.mark.parametrize("dtype", [BF, F32])
def test_lightning_batch_equals_each_alone(dtype):
    H, D, E, lens, starts = 2, 32, 48, [70, 3, 64, 129], [0, 17, 64, 5]
    buf = rand(sum(lens), H * (2 * D + E), dtype=dtype).to(DEV)
    decay = torch.tensor([0.9, 0.99], device=DEV)
    first = rand(4, H, D, E, seed=3).to(DEV)

    def run(x, m, st):
        q, k, v = x.split([H * D, H * D, H * E], -1)
        return hybrid.lightning_mix(q, k, v, decay, st, m)

    together = RecurrentState(first.clone())
    got = run(buf, meta_for(starts, lens, 8)[0], together)
    row = 0
    for i, n in enumerate(lens):
        st = RecurrentState(first.clone())
        m = meta_for([starts[i]], [n], 8)[0]
        m.state_slots = ints([i])
        alone = run(buf[row:row + n], m, st)
        assert torch.equal(alone, got[row:row + n])
        assert torch.equal(st.S[i], together.S[i])
        row += n


# ----------------------------------------------------------------- experts

def expert_case(T, W, E, top, F, Fs, dtype, seed=0):
    x = rand(T, W, seed=seed, dtype=dtype)
    router = rand(E + (Fs > 0), W, seed=1, gain=W ** -0.5, dtype=dtype)
    mat = lambda n, a, b, s: rand(n, a, b, seed=s, gain=b ** -0.5,
                                  dtype=dtype)
    up, down = mat(E, 2 * F, W, 2), mat(E, W, F, 3)
    su, sd = (mat(1, 2 * Fs, W, 4), mat(1, W, Fs, 5)) if Fs else (None, None)
    w = {"router": f64(router[:E])}
    pairs = [(f"e{i}.", up[i], down[i], F) for i in range(E)]
    if Fs:
        pairs.append(("shared.", su[0], sd[0], Fs))
        w["shared.sg"] = f64(router[E:])
    for p, a, b, f in pairs:
        w.update({p + "gate": f64(a[:f]), p + "up": f64(a[f:]),
                  p + "down": f64(b)})
    m = {"router": {"top": top}}
    if Fs:
        m["shared"] = {}
    args = [t if t is None else t.to(DEV)
            for t in (x, router, up, down, su, sd)] + [top]
    # experts as the kernels choose them: a close call may go either way
    z = hybrid.gate_projection(args[0], args[1])[:, :E].cpu()
    ids, _ = O.route(f64(z), top)
    want = torch.zeros(T, W, dtype=torch.float64)
    for t in range(T):
        s = f64(z)[t, ids[t]].softmax(0)
        for j in range(top):
            want[t] += s[j] * O.expert(f64(x)[t], w, f"e{int(ids[t, j])}.")
    if Fs:
        want += torch.sigmoid(f64(x) @ w["shared.sg"].T) \
            * O.expert(f64(x), w, "shared.")
    return args, want


CASES = [(1, 64, 5, 2, 24, 40), (3, 24, 1, 1, 8, 8), (40, 64, 8, 3, 56, 0),
         (100, 72, 4, 4, 40, 104), (33, 264, 70, 5, 16, 24),
         (90, 32, 300, 2, 8, 8), (200, 128, 3, 2, 128, 128),
         (65, 128, 2, 2, 256, 64), (7, 21, 6, 2, 5, 9), (2, 3, 2, 2, 1, 1)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("T,W,E,top,F,Fs", CASES)
def test_mixture(dtype, T, W, E, top, F, Fs):
    args, want = expert_case(T, W, E, top, F, Fs, dtype)
    tol = 2e-5 if dtype == F32 else 2e-2
    assert rel(experts.mixture(*args), want) < tol
    res, w = rand(T, W, seed=8), rand(W, seed=9)
    r = res.to(DEV)
    x = experts.mixture_add_rms(*args, r, w.to(DEV), 1e-3)
    want = f64(res) + O.rms(want, 1e-3) * f64(w)
    assert rel(r, want) < tol and rel(x, want) < tol
    assert x.dtype == dtype


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
    for T, E in ((30, 8), (90, 8), (150, 8), (500, 8)):
        args, want = expert_case(T, 128, E, 2, 128, 64, BF)
        assert rel(experts.mixture(*args), want) < 2e-2
    assert list(dict.fromkeys(seen)) == [16, 32, 64, 256]


def test_routing_ties_and_broken_rows():
    """Equal logits: the lowest numbers win; a row that is not a number still
    gets valid choices and leaves the others alone."""
    E, top = 70, 3
    z = torch.zeros(5, E + 1)
    z[1, 69] = z[1, 64] = z[1, 2] = 2.0
    z[2] = float("nan")
    z[3] = torch.arange(E + 1.0)
    z[4, :2] = float("-inf")
    wt = torch.empty(5, top + 1, device=DEV)
    ids = torch.empty(5, top, dtype=torch.int32, device=DEV)
    ops._native().experts_route(wt, ids, z.to(DEV), E, top)
    assert ids.tolist() == [[0, 1, 2], [2, 64, 69], [0, 1, 2], [69, 68, 67],
                            [2, 3, 4]]
    assert torch.allclose(wt[0].cpu(), torch.tensor([1 / 3] * 3 + [0.5]))
    s = torch.tensor([69.0, 68.0, 67.0]).softmax(0)
    assert torch.allclose(wt[3, :3].cpu(), s)


def test_sorting_covers_every_choice():
    native = ops._native()
    for T, kinds, bm in ((1, 5, 16), (500, 9, 64), (4000, 1025, 1),
                         (3000, 3, 256)):
        g = torch.Generator().manual_seed(T)
        ids = torch.randint(0, kinds, (T,), generator=g).int().to(DEV)
        tiles = min(T, (T + kinds * (bm - 1)) // bm)
        i32 = lambda n: torch.full((n,), 77, dtype=torch.int32, device=DEV)
        order, expert, place = i32(tiles * bm), i32(tiles), i32(T)
        native.experts_sort(order, expert, place, ids, kinds, bm)
        order, expert, place = (t.cpu() for t in (order, expert, place))
        assert torch.equal(order[place.long()], torch.arange(T).int())
        assert int((order >= 0).sum()) == T
        at = place.long() // bm
        assert torch.equal(expert[at], ids.cpu())


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
        if layer["mlp"]:
            r = layer["mlp"]["router"]
            r["top"] = r["experts"]
    return c


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """dtype -> configuration, weights, folder"""
    out = {}
    for dtype, cfg in (("float32", U.standard()),
                       ("bfloat16", all_chosen(U.standard()))):
        w = U.weights(cfg)
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
    from test_tefezen import fill_caches, mixed_run
    cfg, w, folder = models[dtype]
    r = replay(folder, dtype, 4 * 128)
    fill_caches(r, 5.0)
    lens = [70, 3, 120, 41, 1, 90, 17, 64, 33, 2]
    assert mixed_run(r, cfg, w, lens, limits=limits(dtype, cfg, w)) < 1
    assert r.engine.runner.block_manager.num_free_rows == 4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["ones", "odd", "attention only",
                                  "recurrent only", "negative scale",
                                  "many heads", "equal sizes"])
def test_model_other_sizes(tmp_path, dtype, name):
    from test_tefezen import ODD, mixed_run
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
def test_model_window_edge(tmp_path, dtype, cuts):
    from test_tefezen import loud_key_model
    cfg, w = loud_key_model()
    toks = [3 + i % 50 for i in range(80)]
    toks[7] = 1
    r = replay(U.write(tmp_path, cfg, w), dtype)
    got = U.feed(r, "a", toks, cuts)
    within(got, cfg, w, toks, limits(dtype, cfg, w)(toks))
    toks[7] = 2
    d = (U.feed(r, "b", toks, cuts) - got).abs().amax(-1)
    assert d[39] > 0.1 and d[40:].max() == 0


def test_large_layers_in_bfloat16(tmp_path):
    """Sizes of the padded kernels' largest cases and the 256-row tiles."""
    cfg = U.config([
        U.latent(heads=18, dim=128, rot_dim=64, vdim=128, kv_rank=512,
                 window=150, mlp=U.moe(2, 2, 128, 256)),
        U.lightning(heads=4, dim=128, vdim=128, mlp=U.moe(2, 2, 128, 128)),
        U.latent(heads=3, dim=64, rot_dim=64, vdim=96, kv_rank=512,
                 window=40, kv_from=0, mlp=None)], width=256, vocab=300,
        side=32)
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


def test_prefill_graph_matches_eager(models):
    cfg, w, folder = models["bfloat16"]
    outs = []
    for eager in (False, True):
        eng = LLMEngine(EngineConfig(
            model=folder, max_num_seqs=4, max_model_len=512,
            num_gpu_blocks=128, enforce_eager=eager,
            prefill_graph_sizes=(128, 256)), device=DEV)
        logits = []
        for rep in range(3):
            for n in (5, 100, 128, 130, 256):
                from hyperspot.engine.request import Request
                req = Request(f"{rep}-{n}", U.tokens(n, cfg["vocab"], seed=n),
                              SamplingParams())
                batch = eng.scheduler.schedule_portions([(req, n)])
                logits.append(eng.runner.forward(batch).float().cpu().clone())
                eng.scheduler.release(req)
        outs.append(torch.cat(logits))
        assert bool(eng.runner._pgraphs) != eager
    assert U.error(outs[0], outs[1].double()) < 2e-2


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
