"""Tefezen on the CPU: every mechanism against the plain float64
implementation, whole models through portions, mixed batches, reused pages and
slots, and generation through the engine."""

import copy
import json
import os
import subprocess
import sys

import pytest
import torch

import tefezen_oracle as O
import tefezen_util as U
from hyperspot.engine import EngineConfig, LLMEngine, SamplingParams
from hyperspot.engine.kv_cache import RecurrentState
from hyperspot.engine.replay import Replay
from hyperspot.ops import hybrid, torch_ref

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = 2e-4          # float32 against float64, relative to the logits' RMS
SEEN = 5e-3         # what a planted mistake moves at least


@pytest.fixture(scope="module")
def std(tmp_path_factory):
    cfg = U.standard()
    w = U.weights(cfg)
    return cfg, w, U.write(tmp_path_factory.mktemp("std"), cfg, w)


def replay(folder, max_tokens=512):
    return Replay(folder, "float32", max_tokens, device="cpu")


def f64(*shape, seed=0, gain=1.0):
    g = torch.Generator().manual_seed(seed)
    return gain * torch.randn(*shape, generator=g, dtype=torch.float64)


def close(a, b, tol=1e-5):
    err = (a.double() - b).abs().max() / b.abs().max().clamp_min(1e-9)
    assert float(err) < tol, float(err)


# ------------------------------------------------------------- mechanisms

def test_scaled_embedding():
    table = f64(9, 6).float()
    x, res = hybrid.embed_scaled(table, torch.tensor([3, 3, 8]), 2.5)
    close(res, table[[3, 3, 8]].double() * 2.5)
    assert res.dtype == torch.float32 and torch.equal(x, res)


def test_norm_and_add():
    h, res, w = f64(5, 24, gain=3), f64(5, 24, seed=1), f64(24, seed=2)
    want = res + O.rms(h, 0.1) * w
    r = res.float()
    close(hybrid.add_rms(h.float(), r, w.float(), 0.1, torch.float32), want)
    close(r, want)
    close(hybrid.rms_scale(h.float(), w.float(), 0.1, torch.float32),
          O.rms(h, 0.1) * w)


def test_norm_and_gate_over_all_heads():
    o, g, w = f64(4, 18, gain=2), f64(4, 18, seed=1), f64(18, seed=2)
    want = O.rms(o, 1e-3) * w * torch.sigmoid(g)
    close(hybrid.rms_gate(o.float(), g.float(), w.float(), 1e-3, None, 18),
          want)
    ss = o.pow(2).sum(-1).float()          # half of the columns at a time
    for c in (slice(0, 9), slice(9, 18)):
        close(hybrid.rms_gate(o[:, c].float(), g[:, c].float(),
                              w[c].float(), 1e-3, ss, 18), want[:, c])


def test_token_gate():
    z, table = f64(3, 4, gain=2), f64(7, 12, seed=1)
    ids = torch.tensor([6, 0, 6])
    close(hybrid.gelu_gate(z.float(), table.float(), ids, 8),
          O.gelu_tanh(z) * table[ids, 8:12])


def test_rotation_and_append():
    """Only the last part of a query head turns; the latent is normed, the
    shared key part is turned but not normed; slot -1 keeps nothing."""
    H, D, R, rank, T = 3, 5, 6, 7, 9
    q, kv, w = f64(T, H * (D + R)), f64(T, rank + R, seed=1), f64(rank, seed=2)
    pos = torch.tensor([0, 1, 15, 16, 17, 500, 30000, 2, 3])
    slots = torch.tensor([5, 40, 0, 3, 33, 17, -1, 21, 46])
    cache = torch.full((3, 16, rank + R), 9.0)
    qf = q.float()
    torch_ref.latent_rope_append(
        qf, kv.float(), w.float(), pos, 1e3 ** (
            -torch.arange(0, R, 2).double() / R), slots, cache, H, rank, 1e-4)
    for h in range(H):
        a = h * (D + R)
        close(qf[:, a:a + D], q[:, a:a + D])
        close(qf[:, a + D:a + D + R],
              O.rotate_pairs(q[:, a + D:a + D + R], pos, R, 1e3), 1e-4)
    want = torch.cat([O.rms(kv[:, :rank], 1e-4) * w,
                      O.rotate_pairs(kv[:, rank:], pos, R, 1e3)], -1)
    flat = cache.view(-1, rank + R)
    ok = slots >= 0
    close(flat[slots[ok]], want[ok], 1e-4)
    assert (flat[[1, 2, 47]] == 9.0).all() and ok.sum() == 8


@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 33, 500])
def test_attention_pages_and_window_edges(window):
    """A key that stands out just inside and just outside of the window and
    next to a page's border; pages in any order."""
    T, H, D, R, E, rank = 50, 2, 6, 4, 5, 8
    q = f64(T, H, D + R, gain=0.3)
    c, kr = f64(T, rank, seed=1, gain=0.3), f64(T, R, seed=2, gain=0.3)
    uk, uv = f64(H, D, rank, seed=3), f64(H, E, rank, seed=4)
    for at in (0, 15, 16, 31):                  # loud keys
        c[at] = f64(rank, seed=50 + at, gain=4)
    want = []
    for h in range(H):
        want.append(O.window_softmax_attention(
            q[:, h], torch.cat([c @ uk[h].T, kr], -1), c @ uv[h].T, 0.4,
            window))
    table = torch.tensor([[3, 0, 2, 1]])
    cache = torch.full((4, 16, rank + R), float("nan"))
    for t in range(T):
        cache[table[0, t // 16], t % 16] = torch.cat([c[t], kr[t]]).float()
    got = torch_ref.latent_attention(
        q.float().view(T, -1), cache, table, torch.arange(T),
        torch.zeros(T, dtype=torch.int32),
        uk.permute(2, 0, 1).reshape(rank, H * D).float(),
        uv.reshape(H * E, rank).float(), H, window, 0.4)
    close(got, torch.cat(want, -1), 1e-4)


@pytest.mark.parametrize("decay", [0.0, 0.3, 0.999, 1.0])
def test_recurrence_portions_and_state(decay):
    T, H, D, E = 30, 2, 5, 7
    q, k, v = f64(T, H * D), f64(T, H * D, seed=1), f64(T, H * E, seed=2)
    d = torch.tensor([decay, 0.8])
    st = RecurrentState(torch.full((3, H, D, E), 7.0))
    o = torch.cat([torch_ref.lightning_scan(
        q[a:b].float(), k[a:b].float(), v[a:b].float(), d, st,
        torch.tensor([0, b - a]), torch.tensor([1]), torch.arange(a, b))
        for a, b in ((0, 2), (2, 11), (11, 12), (12, 30))])
    for h in range(H):
        part = lambda x, n: O.silu(x[:, h * n:(h + 1) * n])
        close(o[:, h], O.decayed_recurrence(part(q, D), part(k, D),
                                            part(v, E), float(d[h])), 1e-4)
    assert (st.S[[0, 2]] == 7.0).all()


@pytest.mark.parametrize("experts,top,shared", [(6, 2, True), (3, 3, False),
                                                (1, 1, True)])
def test_experts(experts, top, shared):
    W, F, Fs, T = 10, 6, 9, 17
    x, router = f64(T, W), f64(experts + shared, W, seed=1)
    up, down = f64(experts, 2 * F, W, seed=2), f64(experts, W, F, seed=3)
    su, sd = f64(1, 2 * Fs, W, seed=4), f64(1, W, Fs, seed=5)
    w = {"router": router[:experts]}
    for i in range(experts):
        w.update({f"e{i}.gate": up[i, :F], f"e{i}.up": up[i, F:],
                  f"e{i}.down": down[i]})
    m = {"router": {"top": top}}
    if shared:
        m["shared"] = {}
        w.update({"shared.sg": router[experts:], "shared.gate": su[0, :Fs],
                  "shared.up": su[0, Fs:], "shared.down": sd[0]})
    f = lambda t: t.float()
    got = torch_ref.mixture(f(x), f(router), f(up), f(down),
                            f(su) if shared else None,
                            f(sd) if shared else None, top)
    close(got, O.mixture(x, w, m), 1e-4)


@pytest.mark.parametrize("kind", ["latent", "lightning"])
def test_each_mixer_alone_in_a_model(tmp_path, kind):
    cfg = U.config([{"latent": U.latent, "lightning": U.lightning}[kind]()])
    w = U.weights(cfg, seed=3)
    r = replay(U.write(tmp_path, cfg, w))
    toks = U.tokens(45, cfg["vocab"])
    got = U.feed(r, "a", toks, [30, 1])
    assert U.error(got, O.forward(cfg, w, toks)[0]) < TOL


# ------------------------------------------------------------ whole models

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
    assert len(got) == len(trail)
    for a, b in zip(got, trail):
        assert a.dtype == torch.float32
        close(a, b, 1e-4)


def test_planted_mistakes_show(std):
    """The comparison is sharp enough: one wrong detail in the plain
    implementation moves it far past the tolerance."""
    cfg, w, folder = std
    toks = U.tokens(60, cfg["vocab"])
    got = U.feed(replay(folder), "a", toks, [60])

    def changed(edit_cfg=None, edit_w=None):
        c, v = copy.deepcopy(cfg), dict(w)
        if edit_cfg:
            edit_cfg(c)
        if edit_w:
            edit_w(v)
        return U.error(got, O.forward(c, v, toks)[0])

    def mixer(i, **kw):
        return lambda c: c["layers"][i]["mixer"].update(kw)

    def roll(name):
        return lambda v: v.update({name: v[name].roll(1, 0)})

    assert changed() < TOL
    for i, size in ((0, 21), (2, 37), (4, 5)):
        assert changed(mixer(i, mask={"size": size + 1})) > SEEN
        assert changed(mixer(i, mask={"size": size - 1})) > SEEN
    assert changed(mixer(0, rot={"base": 900.0, "dims": 8})) > SEEN
    assert changed(mixer(0, scale=0.2)) > SEEN
    assert changed(mixer(3, decay=[0.96, 0.5])) > SEEN
    assert changed(lambda c: c["embedding"].update(scale=2.1)) > SEEN
    assert changed(lambda c: c["layers"][1]["mlp"]["router"].update(top=2)) \
        > SEEN
    for name in ("l0.mix.dkv.norm", "l2.mix.uk", "l2.mix.uv", "l1.mix.norm",
                 "l0.norm1", "l3.norm2", "l2.side.norm", "side.embed",
                 "l0.mlp.shared.sg", "l1.mlp.router", "final.norm"):
        if name != "l0.mlp.shared.sg":
            assert changed(edit_w=roll(name)) > SEEN, name
    assert changed(edit_w=lambda v: v.update(
        {"l0.mlp.shared.sg": -v["l0.mlp.shared.sg"]})) > SEEN


@pytest.mark.parametrize("cuts", [[1], [2], [3, 2, 7, 64], [16], [17, 15],
                                  [63, 65, 2], [20, 1], [64, 1]])
def test_portions_match_whole(std, cuts):
    cfg, w, folder = std
    toks = U.tokens(140, cfg["vocab"], seed=1)
    want = O.forward(cfg, w, toks)[0]
    assert U.error(U.feed(replay(folder), "a", toks, cuts), want) < TOL


def test_long_decoding(std):
    cfg, w, folder = std
    toks = U.tokens(260, cfg["vocab"], seed=2)
    got = U.feed(replay(folder), "a", toks, [5, 1])
    assert U.error(got, O.forward(cfg, w, toks)[0]) < TOL


def test_single_token_prompt(std):
    cfg, w, folder = std
    assert U.error(U.feed(replay(folder), "a", [5], [1]),
                   O.forward(cfg, w, [5])[0]) < TOL


def loud_key_model():
    """One latent layer whose token 1 has a key that every query asks for:
    from the place where it leaves the window on, logits change."""
    cfg = U.config([U.latent(heads=1, dim=8, rot_dim=2, vdim=16, kv_rank=16,
                             window=33, base=1e6, mlp=None)], scale=4.0)
    w = U.weights(cfg, seed=8)
    x = torch.zeros(56)
    x[0] = 3.0
    w["embed"][1] = x.to(torch.bfloat16)         # only token 1 uses column 0
    w["embed"][:, 1] = 1.0                       # every token has column 1
    w["embed"][2:, 0] = 0.0
    w["l0.mix.q"].zero_()
    w["l0.mix.q"][0, 1] = 4.0                    # q = (16, 0, ...) always
    w["l0.mix.dkv"][0].zero_()
    w["l0.mix.dkv"][0, 0] = 8.0
    w["l0.mix.uk"].zero_()
    w["l0.mix.uk"][0, 0] = 2.0
    return cfg, w


@pytest.mark.parametrize("cuts", [[80], [10, 1], [30, 2, 1], [16, 17, 2]])
def test_key_leaves_the_window_at_its_edge(tmp_path, cuts):
    """Positions 7 + 32 and 7 + 33 see and do not see the key at 7, in
    prompts, short portions and decoding."""
    cfg, w = loud_key_model()
    toks = [3 + i % 50 for i in range(80)]
    toks[7] = 1
    r = replay(U.write(tmp_path, cfg, w))
    got = U.feed(r, "a", toks, cuts)
    want, _ = O.forward(cfg, w, toks)
    assert U.error(got, want) < TOL
    other = list(toks)
    other[7] = 2
    moved = (O.forward(cfg, w, other)[0] - want).abs().amax(-1)
    assert moved[39] > 0.1 and moved[40] < 1e-9      # the test is sharp
    d = (U.feed(r, "b", other, cuts).double() - got).abs().amax(-1)
    assert d[39] > 0.1 and d[40:].max() == 0


def mixed_run(r, cfg, w, lens, seed=0, limits=lambda toks: TOL,
              forward=O.forward):
    """Requests of these lengths through random portions, single tokens and
    pauses, at most four live, each checked against itself alone; the largest
    error over its limit."""
    g = torch.Generator().manual_seed(seed)
    rnd = lambda n: int(torch.randint(0, n, (1,), generator=g))
    todo = [(f"r{i}", U.tokens(n, cfg["vocab"], seed=i))
            for i, n in enumerate(lens)]
    want = {i: forward(cfg, w, t)[0] for i, t in todo}
    lim = {i: torch.as_tensor(limits(t)).expand(len(t)) for i, t in todo}
    live, worst = [], 0.0
    while todo or live:
        if todo and len(live) < 4 and rnd(2) == 0:
            live.append([*todo.pop(0), 0])
        entries, end, rows = [], [], []
        for x in list(live):
            rid, toks, at = x
            if rnd(5) == 0:
                continue                       # sits this step out
            n = min(1 if rnd(2) else 2 + rnd(40), len(toks) - at)
            entries.append({"id": rid, "tokens": toks[at:at + n],
                            "want": list(range(n))})
            rows.append((rid, at, n))
            x[2] += n
            if x[2] == len(toks):
                end.append(rid)
                live.remove(x)
        if entries:
            got = r.step(entries, end)
            assert got.isfinite().all()
            for rid, at, n in rows:
                d, got = got[:n].double() - want[rid][at:at + n], got[n:]
                d = d - d.mean(-1, keepdim=True)
                e = d.pow(2).mean(-1).sqrt() / want[rid].pow(2).mean().sqrt()
                worst = max(worst, float((e / lim[rid][at:at + n]).max()))
    return worst


def fill_caches(r, value):
    for c in r.engine.runner.kv_caches:
        for t in c:
            if t is not None:
                t.fill_(value)


def test_mixed_batches_and_reused_pages_and_slots(std):
    """More requests than the pool holds at once, so pages and state slots
    are handed on; the pool and slots start out as garbage."""
    cfg, w, folder = std
    r = replay(folder, 4 * 128)
    fill_caches(r, 5.0)
    bm = r.engine.runner.block_manager
    free, rows = bm.num_free, bm.num_free_rows
    assert rows == 4
    lens = [70, 3, 120, 41, 1, 90, 17, 64, 33, 2]
    assert mixed_run(r, cfg, w, lens) < 1
    assert bm.num_free == free and bm.num_free_rows == rows


ODD = {
    "ones": U.config([
        U.latent(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, window=1,
                 mlp=U.moe(1, 1, 1, 1)),
        U.lightning(heads=1, dim=1, vdim=1, decay=[0.9])],
        width=3, vocab=11, side=1),
    "odd": U.config([
        U.lightning(heads=3, dim=5, vdim=7, mlp=U.moe(3, 3, 5, 7)),
        U.latent(heads=7, dim=5, rot_dim=6, vdim=9, kv_rank=11, window=13,
                 mlp=None),
        U.latent(heads=3, dim=7, rot_dim=6, vdim=5, kv_rank=11, window=30,
                 kv_from=1, mlp=U.moe(9, 2, 3, None))],
        width=21, vocab=37, side=3),
    "attention only": U.config([U.latent(window=5),
                                U.latent(window=50, kv_from=0),
                                U.latent(heads=1, kv_from=0)]),
    "recurrent only": U.config([U.lightning(decay=[1.0, 0.0]),
                                U.lightning(mlp=None)]),
    "negative scale": U.config([U.latent(scale=-0.3)]),
    "many heads": U.config([U.latent(heads=20, dim=8, vdim=8, window=12),
                            U.latent(heads=37, dim=8, vdim=8, window=12)]),
    "equal sizes": U.config([U.latent(heads=8, dim=8, rot_dim=8, vdim=8,
                                      kv_rank=8, window=8,
                                      mlp=U.moe(8, 8, 8, 8)),
                             U.lightning(heads=8, dim=8, vdim=8)],
                            width=8, vocab=8, side=8),
}


@pytest.mark.parametrize("name", sorted(ODD))
def test_other_sizes(tmp_path, name):
    cfg = ODD[name]
    w = U.weights(cfg, seed=6)
    r = replay(U.write(tmp_path, cfg, w))
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
    bm = eng.runner.block_manager
    assert bm.num_free == 6 and bm.num_free_rows == 4


def test_abort_gives_pages_and_slot_back(std):
    eng = engine(std[2])
    bm = eng.runner.block_manager
    rid = eng.add_request(U.tokens(100, 272), GREEDY)
    eng.step()
    assert bm.num_free_rows == 3
    eng.abort_request(rid)
    assert bm.num_free_rows == 4 and bm.num_free == 64


def test_embeddings(std):
    eng = engine(std[2])
    p = [U.tokens(4 + i, 272, seed=i) for i in range(6)]
    v = eng.embed(p)
    assert v.shape == (6, 56)
    assert torch.allclose(v[5], eng.embed([p[5]])[0], atol=1e-5)


def test_prefix_caching(std, tmp_path):
    """Refused with recurrent state; without, shared latent pages serve a
    second prompt, also through a layer that borrows them."""
    assert not engine(std[2], enable_prefix_caching=True) \
        .config.enable_prefix_caching
    cfg = ODD["attention only"]
    w = U.weights(cfg, seed=6)
    folder = U.write(tmp_path, cfg, w)
    head = U.tokens(50, cfg["vocab"])
    prompts = [head + U.tokens(n, cfg["vocab"], seed=n) for n in (3, 9)]
    eng = engine(folder, enable_prefix_caching=True)
    got = [eng.generate([p], GREEDY)[0] for p in prompts]
    assert got == [O.greedy(cfg, w, p, 12) for p in prompts]
    assert eng.runner.block_manager.cache_hits == 1


def test_preset_runs_and_sampling_is_seeded():
    kw = dict(model="tiny-tefezen", max_num_seqs=2, max_model_len=64,
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


def test_checkpoint_save_and_hot_swap(std, tmp_path):
    cfg, w, folder = std
    eng = engine(folder)
    p = [U.tokens(9, 272)]
    first = eng.generate(p, GREEDY)
    eng.save_checkpoint(str(tmp_path / "a.safetensors"))
    other = U.write(tmp_path / "other", cfg, U.weights(cfg, seed=9))
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
        del v["l1.mlp.e6.up"]
    elif edit == "extra":
        v["l2.mix.dkv"] = v["l0.mix.dkv"].clone()     # a borrowing layer
    else:
        v["l0.mix.uk"] = v["l0.mix.uk"][:-1]
    with pytest.raises(ValueError):
        engine(U.write(tmp_path, cfg, v))


def test_wrong_configurations_are_refused(std, tmp_path):
    cfg, w, _ = std

    def load(i, edit):
        c = copy.deepcopy(cfg)
        edit(c["layers"])
        return engine(U.write(tmp_path / str(i), c, w))

    edits = [lambda x: x[1].update(type="conv"),
             lambda x: x[0]["mlp"].update(kind="dense"),
             lambda x: x[2]["mixer"].update(kv_from=1),
             lambda x: x[2]["mixer"].update(kv_from=4),
             lambda x: x[2]["mixer"].update(kv_rank=32),
             lambda x: x[0]["mixer"]["rot"].update(dims=4),
             lambda x: x[3]["mixer"].update(decay=[0.5]),
             lambda x: x[0]["mlp"]["router"].update(top=6)]
    for i, edit in enumerate(edits):
        with pytest.raises(ValueError):
            load(i, edit)


def test_cache_layout_and_sharing(std):
    from hyperspot.engine.layer_spec import (LatentPages, SharedCache,
                                             StateSlots)
    spec = EngineConfig(model=std[2]).spec()
    layout = spec.cache_layout(1)
    assert [type(c) for c in layout] == [LatentPages, StateSlots, SharedCache,
                                         StateSlots, LatentPages]
    assert layout[0].bytes_per_token(2) == 2 * 48
    assert layout[2].bytes_per_token(2) == 0
    assert spec.latent_windows == [5, 21, 37]
    caches = engine(std[2]).runner.kv_caches
    assert caches[2] is caches[0] and caches[4] is not caches[0]


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
    import torch.multiprocessing as mp
    cfg = U.config([U.latent(heads=4, vdim=12), U.lightning(heads=2),
                    U.latent(heads=2, kv_from=0, mlp=U.moe(3, 2, 6, None)),
                    U.lightning(heads=4, mlp=None)])
    w = U.weights(cfg, seed=7)
    folder = U.write(tmp_path, cfg, w)
    prompts = [U.tokens(30, 272), U.tokens(6, 272, seed=1)]
    want = [O.greedy(cfg, w, p, 12) for p in prompts]
    with mp.Manager() as mgr:
        results = mgr.dict()
        mp.spawn(_tp_rank, args=(2, folder, prompts, 29643, results),
                 nprocs=2, join=True)
        for r in (0, 1):
            assert results[r] == (want, want)


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
