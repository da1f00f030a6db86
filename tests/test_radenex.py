"""Radenex on the CPU: every mechanism against the plain float64
implementation, whole models through portions, mixed batches, reused pages,
and generation through the engine."""

import copy
import json
import math
import os
import subprocess
import sys

import pytest
import torch

import radenex_oracle as O
import radenex_util as U
import sumosun_oracle as S
from hyperspot.engine import EngineConfig, LLMEngine, SamplingParams
from hyperspot.engine.replay import Replay
from hyperspot.engine.rotary import (Yarn, frequencies, gain, head_order,
                                     pair_order)
from hyperspot.models.llama import ForwardMeta
from hyperspot.ops import hybrid, latent, torch_ref

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = 2e-4          # float32 against float64, relative to the logits' RMS
SEEN = 5e-3         # what a planted mistake moves at least


@pytest.fixture(scope="module")
def std(tmp_path_factory):
    cfg = U.standard()
    w = U.weights(cfg, seed=1)
    return cfg, w, U.write(tmp_path_factory.mktemp("std"), cfg, w)


def replay(folder, max_tokens=512):
    return Replay(folder, "float32", max_tokens, device="cpu")


def f64(*shape, seed=0, gain=1.0):
    g = torch.Generator().manual_seed(seed)
    return gain * torch.randn(*shape, generator=g, dtype=torch.float64)


def close(a, b, tol=1e-5):
    err = (a.double() - b).abs().max() / b.abs().max().clamp_min(1e-9)
    assert float(err) < tol, float(err)


# ---------------------------------------------------------------- rotation

YARNS = [(16, 1e4, 8.0, 1024, 32.0, 1.0), (8, 5e3, 4.0, 64, 8.0, 0.5),
         (64, 1e6, 40.0, 4096, 32.0, 1.0),
         (4, 10.0, 2.0, 8, 1e6, 1e-6),        # both ends of the ramp cut off
         (12, 1e4, 3.0, 500, 1.0, 1.0),       # a step where others ramp
         (2, 1e3, 1.0, 100, 5.0, 2.0)]


@pytest.mark.parametrize("dims,base,factor,original,fast,slow", YARNS)
def test_yarn_frequencies(dims, base, factor, original, fast, slow):
    y = Yarn(factor, original, fast, slow)
    want, g = O.yarn_frequencies(dims, base, factor, original, fast, slow)
    close(frequencies(dims, base, y),
          torch.tensor(want, dtype=torch.float64), 1e-12)
    assert math.isclose(gain(y), g) and gain(3.0) == 1.0


def test_yarn_regimes():
    """Fast pairs keep their frequency, slow ones lose the whole factor."""
    f = frequencies(64, 1e6, Yarn(40.0, 4096, 32.0, 1.0))
    plain = frequencies(64, 1e6)
    assert f[0] == plain[0]
    close(f[-1:], plain[-1:] / 40.0, 1e-12)
    mid = f / plain
    assert ((mid > 1 / 40.0 + 1e-3) & (mid < 1 - 1e-3)).sum() >= 3


@pytest.mark.parametrize("size,dims,first", [(10, 6, 0), (9, 4, 3), (8, 8, 0),
                                             (5, 0, 2), (2, 2, 0)])
def test_pair_order(size, dims, first):
    """Turning neighbours in the new order is turning halves in the old."""
    order = pair_order(size, dims, True, first)
    assert sorted(order) == list(range(size))
    assert pair_order(size, dims, False, first) == list(range(size))
    x, pos = f64(7, size), torch.arange(7) * 13
    freqs = frequencies(dims, 300.0, 1.7)
    want = x.clone()
    want[:, first:first + dims] = O.rotate_halves(
        x[:, first:first + dims], pos, O.linear_frequencies(dims, 300.0, 1.7))
    y = x[:, order].float()
    y[:, first:] = torch_ref.turn_pairs(y[:, None, first:], pos, freqs)[:, 0]
    close(y, want[:, order])
    both = head_order(3, size, order)
    assert both[size:2 * size].tolist() == [size + i for i in order]


@pytest.mark.parametrize("turn", [True, False])
@pytest.mark.parametrize("norm", [True, False])
@pytest.mark.parametrize("H,G,D,E,rot", [(4, 2, 6, 4, 4), (3, 3, 8, 2, 8),
                                         (2, 1, 5, 6, 0), (1, 1, 2, 8, 2)])
def test_rope_norm_append(H, G, D, E, rot, norm, turn):
    T, eps = 9, 1e-2
    q, k, v = f64(T, H * D), f64(T, G * D, seed=1), f64(T, G * E, seed=2)
    pos = torch.tensor([0, 1, 2, 50, 51, 900, 901, 70000, 3])
    slots = torch.tensor([5, 40, 0, 3, 33, 17, -1, 21, 46])
    cache = [torch.full((3, G, 16, D), 9.0), torch.full((3, G, E, 16), 9.0)]
    qf, order = q.float(), pair_order(D, rot, True)
    vo = pair_order(E, E, turn)
    x, out = f64(T, 11, seed=5), torch.zeros(T, 11)
    m = ForwardMeta("prefill", pos, slots)
    perm = lambda t, n, d, o: t[:, head_order(n, d, o)].float()
    qf = perm(q, H, D, order)
    from hyperspot.engine.kv_cache import KVPages
    hybrid.rope_norm_append(
        qf, perm(k, G, D, order), perm(v, G, E, vo), m,
        frequencies(rot, 80.0, 1.3),
        frequencies(E if turn else 0, 80.0), KVPages(*cache), 1.25,
        eps if norm else None, hybrid.SideRelu(x.float(), out))
    close(out, x.clamp(min=0) ** 2)

    def head(t):
        t = O.rotate_halves(t, pos, O.linear_frequencies(rot, 80.0, 1.3),
                            1.25)
        return (O.rms(t, eps) if norm else t)[:, order]

    ok = slots >= 0
    kf = cache[0].permute(0, 2, 1, 3).reshape(48, G, D)
    vf = cache[1].permute(0, 3, 1, 2).reshape(48, G, E)
    for n in range(H):
        close(qf.view(T, H, D)[:, n], head(q.view(T, H, D)[:, n]))
    for n in range(G):
        close(kf[slots[ok], n], head(k.view(T, G, D)[:, n])[ok])
        vn = v.view(T, G, E)[:, n]
        if turn:
            vn = O.rotate_halves(vn, pos, O.base_frequencies(E, 80.0))
        close(vf[slots[ok], n], vn[:, vo][ok])
    assert (kf[[1, 2, 47]] == 9.0).all() and (vf[[1, 2, 47]] == 9.0).all()


# --------------------------------------------------------------- attention

@pytest.mark.parametrize("window,keep", [(1, 0), (1, 1), (2, 3), (15, 0),
                                         (16, 16), (17, 15), (33, 4), (20, 17),
                                         (5, 45), (500, 0), (500, 9)])
def test_attention_pages_windows_and_kept_tokens(window, keep):
    """Keys that stand out on both sides of window, page and kept tokens'
    borders; pages in any order, and what is not the sequence's is not a
    number."""
    T, H, G, D, E = 50, 4, 2, 6, 4
    q, k = f64(T, H, D, gain=0.5), f64(T, G, D, seed=1, gain=0.5)
    v, sink = f64(T, G, E, seed=2), f64(H, seed=3)
    for at in (0, 3, 4, 14, 15, 16, 17, 31, 32, 33):
        k[at] *= 6
    freqs, turn = O.base_frequencies(E, 70.0), frequencies(E, 70.0)
    order, pos = pair_order(E, E, True), torch.arange(T)
    table = torch.tensor([[3, 0, 2, 1]])
    kc = torch.full((4, G, 16, D), float("nan"))
    vc = torch.full((4, G, E, 16), float("nan"))
    for g in range(G):
        turned = O.rotate_halves(v[:, g], pos, freqs)
        for t in range(T):
            kc[table[0, t // 16], g, t % 16] = k[t, g].float()
            vc[table[0, t // 16], g, :, t % 16] = turned[t, order].float()
    for s in (sink, torch.zeros(H), None):
        out = torch.zeros(T, H * E)
        torch_ref.window_attention(
            out, q.float().view(T, -1), kc, vc, table, pos,
            torch.zeros(T, dtype=torch.int32), turn,
            None if s is None else s.float(), window, keep, 1.3)
        for h in range(H):
            o = O.sink_attention(
                q[:, h], k[:, h // 2],
                O.rotate_halves(v[:, h // 2], pos, freqs), 1.3,
                -1e9 if s is None else s[h],
                lambda i: O.visible(i, window, keep))
            want = O.rotate_halves(o, -pos, freqs)[:, order]
            close(out.view(T, H, E)[:, h], want, 1e-4)


@pytest.mark.parametrize("sink", [-30.0, 0.0, 3.0, 60.0])
def test_sink(sink):
    """A sink takes its share once, whatever its size, and is not scaled."""
    s = f64(5, 7, gain=3.0)
    got = torch_ref.softmax_with_sink(s.float(), torch.full((5,), sink))
    for i in range(5):
        close(got[i], O.softmax_with_sink(s[i], sink))
    total = s.exp().sum(-1)
    close(got.sum(-1), total / (total + math.exp(sink)))


def test_latent_attention_sink_gate_and_gain():
    T, H, D, R, E, rank, eps = 40, 3, 6, 4, 5, 8, 1e-3
    m = {"heads": H, "dim": D, "rot_dim": R, "vdim": E, "kv_rank": rank,
         "scale": 0.6, "rot": {"dims": R, "base": 900.0, "scaling": {
             "factor": 6.0, "original": 30, "fast": 4.0, "slow": 0.2}}}
    W = 12
    h = f64(T, W)
    w = {n: f64(*s, seed=i) for i, (n, s) in enumerate({
        "q": (H * (D + R), W), "dkv": (rank + R, W), "dkv.norm": (rank,),
        "uk": (H * D, rank), "uv": (H * E, rank), "sink": (H,), "g": (H, W),
        "o": (W, H * E)}.items(), 1)}
    w["o"] = torch.eye(H * E, dtype=torch.float64)
    want = O.latent_attention(h, w, m, eps)
    y = Yarn(6.0, 30, 4.0, 0.2)
    qo = head_order(H, D + R, pair_order(D + R, R, True, D))
    q = (h @ w["q"].T)[:, qo].float()
    kv = (h @ w["dkv"].T)[:, pair_order(rank + R, R, True, rank)].float()
    table = torch.tensor([[2, 0, 1]], dtype=torch.int32)
    pos = torch.arange(T)
    meta = ForwardMeta("prefill", pos, table[0, pos // 16] * 16 + pos % 16,
                       row_seq=torch.zeros(T, dtype=torch.int32),
                       block_tables=table)
    from hyperspot.engine.kv_cache import LatentKV
    cache = LatentKV(torch.zeros(3, 16, rank + R))
    latent.rope_append(q, kv, w["dkv.norm"].float(), meta,
                       frequencies(R, 900.0, y), cache, H, eps, gain(y))
    out = torch.empty(T, H * E + 3)[:, :H * E]
    latent.attention(q, cache, meta, w["uk"].T.float().contiguous(),
                     w["uv"].float(), H, 1 << 30, 0.6, w["sink"].float(),
                     (h @ w["g"].T).float(), out)
    close(out, want, 1e-4)


def test_plain_add_and_norm():
    y, res, pre = f64(5, 24, gain=3), f64(5, 24, seed=1), f64(24, seed=3)
    r = res.float()
    got = hybrid.add_next(y.float(), r, hybrid.NextInput(pre.float(), 0.1),
                          None)
    close(r, res + y)
    close(got, O.rms(res + y, 0.1) * pre)


# ------------------------------------------------------------ whole models

@pytest.mark.parametrize("layer", [
    U.window(), U.latent(), U.window(mlp=None), U.latent(mlp=None)])
def test_each_layer_alone_in_a_model(tmp_path, layer):
    cfg = U.config([layer])
    w = U.weights(cfg, seed=3)
    r = replay(U.write(tmp_path, cfg, w))
    toks = U.tokens(45, cfg["vocab"])
    got = U.feed(r, "a", toks, [30, 1])
    assert U.error(got, O.forward(cfg, w, toks)[0]) < TOL


def test_prompt_and_residual_stream(std):
    cfg, w, folder = std
    toks = U.tokens(70, cfg["vocab"])
    want, trail = O.forward(cfg, w, toks)
    r = replay(folder)
    assert U.error(U.feed(r, "a", toks, [70]), want) < TOL
    from hyperspot.engine.request import Request
    req = Request("x", toks, SamplingParams())
    got = []
    r.engine.runner.forward(
        r.engine.scheduler.schedule_portions([(req, 70)]), trail=got)
    assert len(got) == len(trail) == 2 + 3 * 3
    for a, b in zip(got, trail):
        assert a.dtype == torch.float32
        close(a, b, 1e-4)


def test_planted_mistakes_show(std):
    """The comparison is sharp enough: one wrong detail in the plain
    implementation moves it far past the tolerance."""
    cfg, w, folder = std
    toks = U.tokens(45, cfg["vocab"])
    got = U.feed(replay(folder), "a", toks, [45])

    def changed(edit_cfg=None, edit_w=None):
        c, v = copy.deepcopy(cfg), dict(w)
        if edit_cfg:
            edit_cfg(c)
        if edit_w:
            edit_w(v)
        return U.error(got, O.forward(c, v, toks)[0])

    def mixer(i, **kw):
        return lambda c: c["layers"][i]["mixer"].update(kw)

    def rot(i, **kw):
        return lambda c: c["layers"][i]["mixer"]["rot"].update(kw)

    def scaling(i, **kw):
        return lambda c: c["layers"][i]["mixer"]["rot"]["scaling"].update(kw)

    def mask(i, **kw):
        return lambda c: c["layers"][i]["mixer"]["mask"].update(kw)

    def roll(name, by=1):
        return lambda v: v.update({name: v[name].roll(by, 0)})

    assert changed() < TOL
    for i in (1, 3, 4):
        m = cfg["layers"][i]["mixer"]["mask"]
        for d in (-1, 1):
            assert changed(mask(i, size=m["size"] + d)) > SEEN, i
            assert changed(mask(i, keep_first=m["keep_first"] + d)) > SEEN, i
        assert changed(rot(i, base=200.0)) > SEEN
        assert changed(scaling(i, factor=4.0)) > SEEN
        assert changed(mixer(i, scale=0.4)) > SEEN
    for i in (0, 2):
        assert changed(mixer(i, scale=0.4)) > SEEN
        for kw in ({"factor": 5.0}, {"original": 16}, {"fast": 0.9},
                   {"slow": 0.1}):
            assert changed(scaling(i, **kw)) > SEEN / 10, (i, kw)
        assert changed(rot(i, base=200.0)) > SEEN
    for kw in ({"start": 2}, {"stop": 3}, {"times": 2}):
        assert changed(lambda c: c["loop"].update(kw)) > SEEN, kw
    for name in ("l0.norm1", "l4.norm1", "final.norm", "l0.mix.dkv.norm",
                 "l0.mix.sink", "l2.mix.sink", "l2.mix.g", "l1.mlp.up",
                 "l0.mlp.down", "l1.mix.q", "l3.mix.v", "l2.mix.uk",
                 "l0.mix.uv"):
        assert changed(edit_w=roll(name)) > SEEN, name


@pytest.mark.parametrize("name,make", [
    # no sink, a scaled one; values not turned back; no gain; pairs next to
    # each other; another eps
    ("softmax_with_sink", lambda old: lambda s, sink: old(s, -1e9)),
    ("softmax_with_sink", lambda old: lambda s, sink: old(s, 0.3 * sink + 0.1)),
    ("rotate_halves", lambda old: lambda x, a, f, gain=1.0:
        old(x, a, f, gain) if a[-1] >= 0 else x),
    ("rotate_halves", lambda old: lambda x, a, f, gain=1.0: old(x, a, f)),
    ("rotate_halves", lambda old: lambda x, a, f, gain=1.0:
        S.rotate_pairs(x, a, 2 * len(f), 500.0)),
    ("rms", lambda old: lambda x, eps: old(x, 3e-2))])
def test_planted_mechanism_mistakes_show(std, monkeypatch, name, make):
    cfg, w, folder = std
    toks = U.tokens(60, cfg["vocab"])
    got = U.feed(replay(folder), "a", toks, [60])
    monkeypatch.setattr(O, name, make(getattr(O, name)))
    assert U.error(got, O.forward(cfg, w, toks)[0]) > SEEN


@pytest.mark.parametrize("cuts", [[1], [2], [3, 2, 7, 64], [16], [17, 15],
                                  [63, 65, 2], [20, 1], [64, 1]])
def test_portions_match_whole(std, cuts):
    cfg, w, folder = std
    toks = U.tokens(140, cfg["vocab"], seed=1)
    want = O.forward(cfg, w, toks)[0]
    assert U.error(U.feed(replay(folder), "a", toks, cuts), want) < TOL


def test_long_decoding(std):
    cfg, w, folder = std
    toks = U.tokens(230, cfg["vocab"], seed=2)
    got = U.feed(replay(folder), "a", toks, [5, 1])
    assert U.error(got, O.forward(cfg, w, toks)[0]) < TOL


def test_single_token_prompt(std):
    cfg, w, folder = std
    assert U.error(U.feed(replay(folder), "a", [5], [1]),
                   O.forward(cfg, w, [5])[0]) < TOL


@pytest.mark.parametrize("loop", [(0, 0, 1), (0, 5, 2), (4, 5, 4), (2, 2, 7)])
def test_looped_layers_equal_copies(std, tmp_path, loop):
    """A later pass is a copy of the layers with caches of its own."""
    cfg, w, _ = std
    a = U.config(cfg["layers"], loop=loop)
    runs = O.layer_runs(a)
    assert len(runs) == 5 + (loop[1] - loop[0]) * (loop[2] - 1)
    b = U.config([cfg["layers"][i] for i in runs])
    v = {n: t for n, t in w.items() if not n.startswith("l")}
    for n, i in enumerate(runs):
        v.update({f"l{n}." + k.split(".", 1)[1]: t.clone()
                  for k, t in w.items() if k.startswith(f"l{i}.")})
    toks, cuts = U.tokens(60, cfg["vocab"], seed=5), [40, 7, 1]
    x, y = (U.feed(replay(U.write(tmp_path / n, c, p)), "a", toks, cuts)
            for n, c, p in (("a", a, w), ("b", b, v)))
    assert torch.equal(x, y)


def loud_key_model(size=33, keep=3):
    """One layer of windowed attention in which every query asks for the key
    of token 1, whatever the distance: it lies in an unrotated dimension."""
    cfg = U.config([U.window(heads=1, kv_heads=1, dim=8, vdim=16, size=size,
                             keep=keep, scale=1.0, rot=4, mlp=None)])
    w = U.weights(cfg, seed=8)
    w["l0.norm1"][:] = 1.0
    w["embed"][:, 0] = 0.0
    w["embed"][1, 0] = 3.0                       # only token 1 uses column 0
    w["embed"][:, 1] = 1.0                       # every token has column 1
    w["l0.mix.q"].zero_()
    w["l0.mix.q"][6, 1] = 4.0
    w["l0.mix.k"][6].zero_()
    w["l0.mix.k"][6, 0] = 9.0
    w["l0.mix.o"] *= 3
    return cfg, w


def loud(toks, at):
    """The prompt with token 1, and another one, at position `at`."""
    a, b = list(toks), list(toks)
    a[at], b[at] = 1, 2
    return a, b


CUTS = [[80], [10, 1], [30, 2, 1], [16, 17, 2]]


@pytest.mark.parametrize("cuts", CUTS)
def test_key_leaves_the_window(tmp_path, cuts):
    """Positions 39 and 40 see and do not see the key at 7, in prompts, short
    portions and decoding."""
    cfg, w = loud_key_model()
    a, b = loud([3 + i % 50 for i in range(80)], 7)
    r = replay(U.write(tmp_path, cfg, w))
    got = U.feed(r, "a", a, cuts)
    want, _ = O.forward(cfg, w, a)
    assert U.error(got, want) < TOL
    moved = (O.forward(cfg, w, b)[0] - want).abs().amax(-1)
    assert moved[39] > 0.3 and moved[40] < 1e-9      # the test is sharp
    d = (U.feed(r, "b", b, cuts).double() - got).abs().amax(-1)
    assert d[39] > 0.3 and d[40:].max() == 0


@pytest.mark.parametrize("cuts", CUTS)
def test_first_tokens_are_kept(tmp_path, cuts):
    """The last kept token is seen for good, the next one leaves with the
    window."""
    cfg, w = loud_key_model(size=9, keep=3)
    r = replay(U.write(tmp_path, cfg, w))
    for at, kept in ((2, True), (3, False)):
        a, b = loud([3 + i % 50 for i in range(80)], at)
        got = U.feed(r, f"a{at}", a, cuts)
        assert U.error(got, O.forward(cfg, w, a)[0]) < TOL
        d = (U.feed(r, f"b{at}", b, cuts) - got).abs().amax(-1)
        assert d[at + 8] > 0.3
        assert d[at + 9:].min() > 0.3 if kept else d[at + 9:].max() == 0


def test_latent_layers_see_everything(tmp_path):
    """A key that stands out is seen from any later position."""
    cfg = U.config([U.latent(heads=1, dim=8, rot_dim=4, vdim=16, kv_rank=16,
                             scale=1.0, mlp=None)])
    w = U.weights(cfg, seed=8)
    w["embed"][:, 0] = 0.0
    w["embed"][1, 0] = 8.0
    w["embed"][:, 1] = 1.0
    for n in ("q", "uk"):
        w["l0.mix." + n].zero_()
    w["l0.mix.q"][2, 1] = 4.0
    w["l0.mix.dkv"][0].zero_()
    w["l0.mix.dkv"][0, 0] = 9.0
    w["l0.mix.uk"][2, 0] = 3.0
    w["l0.mix.dkv.norm"][0] = 1.0
    w["l0.mix.g"].zero_()
    w["l0.mix.o"] *= 3
    r = replay(U.write(tmp_path, cfg, w))
    for at in (0, 15, 16, 40):
        a, b = loud([3 + i % 50 for i in range(150)], at)
        for i, cuts in enumerate(([150], [41, 1], [17, 60, 2])):
            got = U.feed(r, f"a{at}{i}", a, cuts)
            assert U.error(got, O.forward(cfg, w, a)[0]) < TOL
            d = (U.feed(r, f"b{at}{i}", b, cuts) - got).abs().amax(-1)
            assert d[:at].sum() == 0 and d[at:].min() > 0.2


def mixed_run(r, cfg, w, lens, seed=0, limits=lambda toks: TOL):
    """Requests of these lengths through random portions, single tokens and
    pauses, at most four live, each checked against itself alone; the largest
    error over its limit."""
    import test_tefezen
    return test_tefezen.mixed_run(r, cfg, w, lens, seed, limits,
                                  forward=O.forward)


def fill_caches(r, value):
    for c in r.engine.runner.kv_caches:
        for t in c:
            t.fill_(value)


LENS = [70, 3, 120, 41, 1, 90, 17, 64, 33, 2]


def test_mixed_batches_and_reused_pages(std):
    """More requests than the pool holds at once, so pages are handed on; the
    pool starts out as garbage."""
    cfg, w, folder = std
    r = replay(folder, 4 * 128)
    fill_caches(r, 5.0)
    bm = r.engine.runner.block_manager
    free, rows = bm.num_free, bm.num_free_rows
    assert free == 32
    assert mixed_run(r, cfg, w, LENS) < 1
    assert bm.num_free == free and bm.num_free_rows == rows


ODD = {
    "ones": U.config([U.window(1, 1, 1, 2, 1, 0, rot=0, mlp=U.dense(1)),
                      U.latent(1, 1, 2, 1, 1, mlp=U.dense(1))],
                     width=3, vocab=11, loop=(0, 1, 2)),
    "odd": U.config([U.window(6, 3, 5, 14, 11, 1, rot=2, mlp=U.dense(5)),
                     U.latent(3, 7, 6, 9, 11, mlp=U.dense(13)),
                     U.window(5, 5, 7, 6, 3, 7, rot=6, mlp=None),
                     U.latent(7, 3, 2, 5, 9, mlp=None)],
                    width=21, vocab=37, loop=(1, 3, 2)),
    "window only": U.config([U.window(size=9, keep=0),
                             U.window(size=300, keep=4)]),
    "latent only": U.config([U.latent(), U.latent(mlp=None)],
                            loop=(0, 2, 2)),
    "all rotated": U.config([U.window(dim=16, rot=16, factor=1.0),
                             U.latent(dim=8, rot_dim=16, factor=1.0)]),
    "negative scale": U.config([U.window(scale=-0.4), U.latent(scale=-0.2)]),
    "many heads": U.config([U.window(20, 1, 8, 8, 12),
                            U.latent(38, 8, 8, 8, 16),
                            U.window(38, 2, 8, 8, 12, 30)]),
    "more kept than seen": U.config([U.window(size=1, keep=40),
                                     U.window(size=3, keep=16)]),
    "equal sizes": U.config([U.window(8, 8, 8, 8, 8, 8, rot=8,
                                      mlp=U.dense(8)),
                             U.latent(8, 8, 8, 8, 8, mlp=U.dense(8))],
                            width=8, vocab=8, loop=(0, 2, 8)),
}


@pytest.mark.parametrize("name", sorted(ODD))
def test_other_sizes(tmp_path, name):
    cfg = ODD[name]
    w = U.weights(cfg, seed=6)
    r = replay(U.write(tmp_path, cfg, w))
    fill_caches(r, 3.0)
    toks = U.tokens(50, cfg["vocab"])
    want = O.forward(cfg, w, toks)[0]
    for i, cuts in enumerate(([50], [20, 1], [2])):
        assert U.error(U.feed(r, f"a{i}", toks, cuts), want) < TOL, cuts
    assert mixed_run(r, cfg, w, [30, 9, 21]) < 1


# ------------------------------------------- engine: generation, scheduling

def engine(folder, **kw):
    base = dict(model=folder, max_num_seqs=4, max_num_batched_tokens=64,
                max_model_len=256, num_gpu_blocks=64)
    base.update(kw)
    return LLMEngine(EngineConfig(**base), device="cpu")


@pytest.fixture(scope="module")
def greedy(std):
    cfg, w, _ = std
    prompts = [U.tokens(n, cfg["vocab"], seed=20 + n) for n in (5, 40, 1, 23)]
    want = [O.greedy(cfg, w, p, 12) for p in prompts]
    assert min(len(set(x)) for x in want) >= 4     # not stuck
    return prompts, want


GREEDY = SamplingParams(temperature=0.0, max_tokens=12)


@pytest.mark.parametrize("kw", [
    {}, {"max_num_batched_tokens": 7}, {"mixed_batches": True},
    {"mixed_batches": True, "max_num_batched_tokens": 6},
    {"max_num_seqs": 2}, {"max_num_seqs": 1, "mixed_batches": True}])
def test_greedy_generation(std, greedy, kw):
    prompts, want = greedy
    assert engine(std[2], **kw).generate(prompts, GREEDY) == want


@pytest.mark.parametrize("mixed", [False, True])
def test_generation_with_preemption(std, greedy, mixed):
    prompts, want = greedy
    eng = engine(std[2], num_gpu_blocks=6, mixed_batches=mixed)
    assert eng.generate(prompts, GREEDY) == want
    assert eng.runner.block_manager.num_free == 6


def test_abort_gives_pages_back(std):
    eng = engine(std[2])
    bm = eng.runner.block_manager
    rid = eng.add_request(U.tokens(100, 272), GREEDY)
    eng.step()
    assert bm.num_free < 64
    eng.abort_request(rid)
    assert bm.num_free == 64


def test_embeddings(std):
    eng = engine(std[2])
    p = [U.tokens(4 + i, 272, seed=i) for i in range(6)]
    v = eng.embed(p)
    assert v.shape == (6, 56)
    assert torch.allclose(v[5], eng.embed([p[5]])[0], atol=1e-5)


def test_prefix_caching(std):
    """Nothing but pages is kept per sequence, so a second prompt shares
    those of the first."""
    cfg, w, folder = std
    head = U.tokens(50, cfg["vocab"])
    prompts = [head + U.tokens(n, cfg["vocab"], seed=n) for n in (3, 9)]
    eng = engine(folder, enable_prefix_caching=True)
    got = [eng.generate([p], GREEDY)[0] for p in prompts]
    assert got == [O.greedy(cfg, w, p, 12) for p in prompts]
    assert eng.runner.block_manager.cache_hits == 1


def test_preset_runs_and_sampling_is_seeded():
    kw = dict(model="tiny-radenex", max_num_seqs=2, max_model_len=64,
              num_gpu_blocks=16)
    sp = SamplingParams(temperature=0.8, top_k=20, max_tokens=6, seed=3)
    a, b = (LLMEngine(EngineConfig(**kw), device="cpu").generate(
        [[4, 5, 6]], sp) for _ in range(2))
    assert a == b and len(a[0]) == 6


def test_fp8_options_are_refused(std):
    with pytest.raises(ValueError):
        engine(std[2], kv_dtype="fp8")
    with pytest.raises(ValueError):
        engine(std[2], quant="fp8")


# -------------------------------------------------------- loading, registry

def test_parameter_count_matches_tensors(std):
    cfg, w, folder = std
    spec = EngineConfig(model=folder).spec()
    assert spec.param_count() == sum(t.numel() for t in w.values())


@pytest.mark.parametrize("name", ["standard", "odd"])
def test_checkpoint_save_and_hot_swap(tmp_path, name):
    """Odd sizes have zero rows between the merged projections, which a
    checkpoint does not hold."""
    cfg = U.standard() if name == "standard" else ODD[name]
    vocab = cfg["vocab"]
    folder, other = (U.write(tmp_path / f"m{s}", cfg, U.weights(cfg, seed=s))
                     for s in (1, 9))
    eng = engine(folder)
    p = [U.tokens(9, vocab)]
    first = eng.generate(p, GREEDY)
    eng.save_checkpoint(str(tmp_path / "a.safetensors"))
    eng.swap_weights(other)
    second = eng.generate(p, GREEDY)
    assert second != first
    eng.swap_weights(str(tmp_path / "a.safetensors"))
    assert eng.generate(p, GREEDY) == first
    eng.swap_weights(folder)
    assert eng.generate(p, GREEDY) == first


@pytest.mark.parametrize("edit", ["missing", "extra", "shape"])
def test_wrong_tensors_are_refused(std, tmp_path, edit):
    cfg, w, _ = std
    v = dict(w)
    if edit == "missing":
        del v["l0.mix.sink"]
    elif edit == "extra":
        v["l5.norm1"] = v["l1.norm1"].clone()     # a later pass has none
    else:
        v["l0.mix.g"] = v["l0.mix.g"][:, :-1]
    with pytest.raises(ValueError):
        engine(U.write(tmp_path, cfg, v))


def test_wrong_configurations_are_refused(std, tmp_path):
    cfg, w, _ = std

    def load(i, edit):
        c = copy.deepcopy(cfg)
        edit(c)
        return engine(U.write(tmp_path / str(i), c, w))

    edits = [lambda c: c["layers"][1].update(type="conv"),
             lambda c: c["layers"][0]["mlp"].update(kind="glu"),
             lambda c: c["layers"][1]["mixer"].update(kv_heads=4),
             lambda c: c["layers"][1]["mixer"].update(vdim=15),
             lambda c: c["layers"][1]["mixer"]["mask"].update(size=0),
             lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1),
             lambda c: c["layers"][1]["mixer"]["rot"].update(dims=26),
             lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(
                 factor=0),
             lambda c: c["layers"][0]["mixer"]["rot"].update(dims=8),
             lambda c: c["layers"][0]["mixer"]["rot"].update(base=1.0),
             lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(
                 slow=0.0),
             lambda c: c["loop"].update(stop=6),
             lambda c: c["loop"].update(start=4, stop=3),
             lambda c: c["loop"].update(times=0)]
    for i, edit in enumerate(edits):
        with pytest.raises(ValueError):
            load(i, edit)


def test_only_a_dense_feed_forward_runs_beside_a_mixer():
    from hyperspot.engine.layer_spec import Experts, WindowAttention
    from hyperspot.models.mixers import KeptWindowAttention
    spec = WindowAttention(1, 1, 8, 8, 1.0, 4, 4, 10.0)
    with pytest.raises(ValueError):
        KeptWindowAttention(spec, 8, 1e-5, torch.float32, 1, Experts(2, 1, 8))


def test_cache_layout(std):
    from hyperspot.engine.layer_spec import (UNBOUNDED, LatentPages, PagedKV)
    spec = EngineConfig(model=std[2]).spec()
    assert not spec.has_state and spec.latent_windows == [UNBOUNDED]
    layout = spec.cache_layout(1)
    assert len(layout) == 11
    assert layout[0] == LatentPages(56) and layout[2] == LatentPages(32)
    assert layout[1] == layout[4] == PagedKV(2, 24, 16, True)
    caches = engine(std[2]).runner.kv_caches
    assert len({t.data_ptr() for c in caches for t in c}) \
        == sum(len(c) for c in caches) == 7 * 2 + 4
    assert EngineConfig(model="tiny-radenex").spec().cache_layout(2)[0] \
        .kv_heads == 1


def _tp_rank(rank, world, folder, prompts, port, results):
    os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT=str(port),
                      RANK=str(rank), WORLD_SIZE=str(world))
    import torch.distributed as dist
    from hyperspot.parallel.state import (destroy_model_parallel,
                                          initialize_model_parallel)
    dist.init_process_group("gloo", rank=rank, world_size=world)
    initialize_model_parallel(tp_size=world)
    eng = engine(folder, tp_size=world)
    out = eng.generate(prompts, GREEDY)
    eng.save_checkpoint(folder + "/saved.safetensors")
    dist.barrier()
    eng.swap_weights(folder + "/saved.safetensors")
    results[rank] = (out, eng.generate(prompts, GREEDY))
    dist.barrier()
    destroy_model_parallel()
    dist.destroy_process_group()


def test_tensor_parallel_matches_single(tmp_path):
    """Heads, sinks, gates and both parts of the joined products divided; a
    checkpoint saved by two ranks loads into one."""
    import torch.multiprocessing as mp
    cfg = U.config([U.window(heads=4, vdim=12, mlp=U.dense(20)),
                    U.latent(heads=6, dim=10, vdim=6, mlp=U.dense(14)),
                    U.window(mlp=None), U.latent(heads=2, mlp=None)],
                   loop=(0, 2, 2))
    w = U.weights(cfg, seed=7)
    folder = U.write(tmp_path, cfg, w)
    prompts = [U.tokens(30, 272), U.tokens(6, 272, seed=1)]
    want = [O.greedy(cfg, w, p, 12) for p in prompts]
    with mp.Manager() as mgr:
        results = mgr.dict()
        mp.spawn(_tp_rank, args=(2, folder, prompts, 29657, results),
                 nprocs=2, join=True)
        for r in (0, 1):
            assert results[r] == (want, want)
    eng = engine(U.write(tmp_path / "other", cfg, U.weights(cfg, seed=3)))
    eng.swap_weights(folder + "/saved.safetensors")
    assert eng.generate(prompts, GREEDY) == want


def test_trace_run_program(std, tmp_path):
    import numpy as np
    cfg, w, folder = std
    toks = U.tokens(40, cfg["vocab"], seed=4)
    want = O.forward(cfg, w, toks)[0]
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": toks[:30],
                                 "want": [3, 29]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": toks[:2], "want": []},
                                {"id": "a", "tokens": toks[30:31],
                                 "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": toks[2:9],
                                 "want": [6]},
                                {"id": "a", "tokens": toks[31:32],
                                 "want": [0]}], "end": ["b", "a"]}]
    out = subprocess.run(
        [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model",
         folder, "--dtype", "float32", "--out", str(tmp_path),
         "--max-tokens", "128", "--device", "cpu"],
        input="".join(json.dumps(s) + "\n" for s in steps), text=True,
        capture_output=True, timeout=120)
    assert out.returncode == 0, out.stderr[-2000:]
    rows = {0: [3, 29], 2: [8, 31]}
    assert sorted(os.listdir(tmp_path)) == [f"{i}.f32" for i in rows]
    for i, r in rows.items():
        got = torch.from_numpy(np.fromfile(tmp_path / f"{i}.f32", "<f4"))
        assert U.error(got.view(len(r), -1), want[r]) < TOL
