"""Mutusun on the CPU: every mechanism against the plain float64
implementation, whole models through portions, mixed batches, reused pages and
slots, and generation through the engine."""

import copy
import json
import os
import subprocess
import sys

import pytest
import torch

import mutusun_oracle as O
import mutusun_util as U
from hyperspot.engine import EngineConfig, LLMEngine, SamplingParams
from hyperspot.engine.replay import Replay
from hyperspot.models.llama import ForwardMeta
from hyperspot.ops import experts, hybrid, torch_ref

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


def step_meta(starts, lens, slots, decode=False):
    ss = [0]
    for n in lens:
        ss.append(ss[-1] + n)
    pos = [p for a, n in zip(starts, lens) for p in range(a, a + n)]
    return ForwardMeta(
        mode="decode" if decode else "prefill", positions=torch.tensor(pos),
        slot_mapping=torch.arange(len(pos)),
        seq_start=torch.tensor(ss, dtype=torch.int32),
        state_slots=torch.tensor(slots, dtype=torch.int32))


# ------------------------------------------------------------- mechanisms

@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7, 40])
def test_convolution_portions_and_tail(taps):
    """One sequence in portions, down to fewer tokens than taps, beside a
    second one; the slots start out as garbage and slot -1 keeps nothing."""
    W, T = 6, 60
    h, w = f64(T, W), f64(W, taps, seed=1)
    other = f64(T, W, seed=2)
    tail = torch.full((4, taps - 1, W), 7.0)
    out, at = [], 0
    for n in (1, 1, 2, 9, 1, 30, 16):
        x = torch.cat([h[at:at + n], other[:5], other[:3]]).float()
        m = step_meta([at, 0, 0], [n, 5, 3], [2, 1, -1])
        y = hybrid.causal_conv(x, w.t().float().contiguous(), tail, m)
        out.append(y[:n])
        close(y[n:n + 5], O.causal_conv(other[:5], w))
        close(y[n + 5:], O.causal_conv(other[:3], w))
        at += n
    assert at == T
    close(torch.cat(out), O.causal_conv(h, w))
    assert (tail[[0, 3]] == 7.0).all()
    last = torch.cat([torch.zeros(40, W), h.float()])[-(taps - 1):] \
        if taps > 1 else tail[2]
    assert torch.equal(tail[2], last)


def test_first_tokens_decoded_one_by_one():
    """Tokens before the start count as zero whatever the slot holds."""
    w, h = f64(5, 4, seed=1), f64(6, 5)
    tail = torch.full((2, 3, 5), float("nan"))
    got = torch.cat([hybrid.causal_conv(
        h[t:t + 1].float(), w.t().float().contiguous(), tail,
        step_meta([t], [1], [1], decode=True)) for t in range(6)])
    close(got, O.causal_conv(h, w))
    assert tail[0].isnan().all()


def test_between_sublayers():
    y, res = f64(5, 24, gain=3), f64(5, 24, seed=1)
    post, pre, conv = f64(24, seed=2), f64(24, seed=3), f64(24, 3, seed=4)
    want = res + O.rms(y, 0.1) * post
    h = O.rms(want, 0.1) * pre
    m = step_meta([0], [5], [0])
    r = res.float()
    plain = hybrid.NextInput(pre.float(), 0.1)
    close(hybrid.add_rms_next(y.float(), r, post.float(), plain, m), h)
    close(r, want)
    nxt = hybrid.NextInput(pre.float(), 0.1, conv.t().float().contiguous(),
                           torch.zeros(1, 2, 24))
    close(hybrid.next_input(r, nxt, m, torch.float32), O.causal_conv(h, conv))


def test_head_norms_and_append():
    H, G, D, E, T = 4, 2, 6, 5, 9
    q, k, v = f64(T, H * D), f64(T, G * D, seed=1), f64(T, G * E, seed=2)
    qw, kw = f64(D, seed=3), f64(D, seed=4)
    slots = torch.tensor([5, 40, 0, 3, 33, 17, -1, 21, 46])
    kc = torch.full((3, G, 16, D), 9.0)
    vc = torch.full((3, G, E, 16), 9.0)
    qf = q.float()
    torch_ref.norm_append(qf, k.float(), v.float(), qw.float(), kw.float(),
                          slots, kc, vc, 1e-3)
    close(qf.view(T, H, D), O.rms(q.view(T, H, D), 1e-3) * qw)
    ok = slots >= 0
    flat = kc.permute(0, 2, 1, 3).reshape(48, G, D)
    close(flat[slots[ok]], (O.rms(k.view(T, G, D), 1e-3) * kw)[ok])
    vflat = vc.permute(0, 3, 1, 2).reshape(48, G, E)
    close(vflat[slots[ok]], v.view(T, G, E)[ok])
    assert (flat[[1, 2, 47]] == 9.0).all()


@pytest.mark.parametrize("chunk", [1, 2, 15, 16, 17, 33, 500])
def test_attention_pages_and_chunk_edges(chunk):
    """Keys that stand out on both sides of chunk and page borders; pages in
    any order, and what is not the sequence's is not a number."""
    T, H, G, D, E = 50, 4, 2, 6, 5
    q, k = f64(T, H, D, gain=0.5), f64(T, G, D, seed=1, gain=0.5)
    v, bias = f64(T, G, E, seed=2), f64(H, seed=3)
    for at in (0, 14, 15, 16, 31, 32, 33):
        k[at] *= 6
    want = torch.cat([O.sigmoid_attention(
        q[:, h], k[:, h // 2], v[:, h // 2], 1.3, 5.0, bias[h], chunk)
        for h in range(H)], -1)
    table = torch.tensor([[3, 0, 2, 1]])
    kc = torch.full((4, G, 16, D), float("nan"))
    vc = torch.full((4, G, E, 16), float("nan"))
    for t in range(T):
        kc[table[0, t // 16], :, t % 16] = k[t].float()
        vc[table[0, t // 16], :, :, t % 16] = v[t].float()
    got = torch_ref.sigmoid_attention(
        q.float().view(T, -1), kc, vc, table, torch.arange(T),
        torch.zeros(T, dtype=torch.int32), bias.float(), chunk, 1.3, 5.0)
    close(got, want, 1e-4)


def test_squared_relu_and_clamped_unit():
    x = f64(7, 12, gain=2)
    close(hybrid.squared_relu(x.float()), x.clamp(min=0) ** 2)
    w = {"gate": f64(6, 12, seed=1), "up": f64(6, 12, seed=2),
         "down": torch.eye(6, dtype=torch.float64)}
    both = x @ torch.cat([w["gate"], w["up"]]).T
    for limit in (0.3, 1.0, 50.0):
        close(hybrid.clamped_glu(both.float(), limit),
              O.expert(x, w, "", limit))


def expert_weights(E, W, F, seed=2):
    up, down = f64(E, 2 * F, W, seed=seed), f64(E, W, F, seed=seed + 1)
    w = {}
    for i in range(E):
        w.update({f"e{i}.gate": up[i, :F], f"e{i}.up": up[i, F:],
                  f"e{i}.down": down[i]})
    return up, down, w


@pytest.mark.parametrize("E,identity,top", [(6, 3, 2), (3, 0, 3), (1, 1, 1),
                                            (2, 5, 7)])
def test_experts(E, identity, top):
    W, F, T, n = 10, 6, 40, E + identity
    x, router = f64(T, W), f64(n, W, seed=1, gain=0.4)
    corr = f64(n, seed=9, gain=0.3)
    up, down, w = expert_weights(E, W, F)
    w.update({"router": router, "correction": corr})
    m = {"router": {"experts": E, "identity": identity, "top": top},
         "expert": {"limit": 0.8}}
    f = lambda t: t.float()
    rules = experts.Rules(f(corr), identity, 0.8)
    args = (f(x), f(router), f(up), f(down), None, None, top)
    want = O.mixture(x, w, m)
    close(experts.mixture(*args, rules), want, 1e-4)
    # the identity part alone is what another rank leaves out
    ids, weight = O.route(x @ router.T, corr, top)
    part = x * (weight * (ids >= E)).sum(-1, keepdim=True)
    got = experts.mixture(*args, rules._replace(identity_here=False))
    close(got, want - part, 1e-4)
    if n > top:                      # the correction moves some choice
        assert (ids.sort().values != O.route(
            x @ router.T, 0 * corr, top)[0].sort().values).any()


def test_clamped_experts_with_softmax_over_the_chosen_and_a_shared_one():
    """The parts combine freely: the activation of this design under the
    routing of the other one."""
    E, W, F, T, top, lim = 4, 9, 5, 12, 2, 0.6
    x, router = f64(T, W), f64(E + 1 + 1, W, seed=1)
    up, down, w = expert_weights(E, W, F)
    su, sd, s = expert_weights(1, W, F, seed=7)
    f = lambda t: t.float()
    got = experts.mixture(f(x), f(router), f(up), f(down), f(su), f(sd), top,
                          experts.Rules(None, 1, lim))
    z = x @ router.T
    want = torch.sigmoid(z[:, 5:]) * O.expert(x, s, "e0.", lim)
    val, ids = z[:, :5].topk(top, -1)
    p = val.softmax(-1)
    for t in range(T):
        for j in range(top):
            e = int(ids[t, j])
            want[t] += p[t, j] * (x[t] if e == E
                                  else O.expert(x[t], w, f"e{e}.", lim))
    close(got, want, 1e-4)


@pytest.mark.parametrize("mlp", [U.dense(), U.moe(), None])
def test_each_feed_forward_alone_in_a_model(tmp_path, mlp):
    cfg = U.config([U.layer(mlp=mlp)])
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
    assert len(got) == len(trail) == 7
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
    for i, x in enumerate(cfg["layers"]):
        size = x["mixer"]["mask"]["size"]
        assert changed(mixer(i, mask={"size": size + 1})) > SEEN, i
        assert changed(mixer(i, mask={"size": size - 1})) > SEEN, i
    assert changed(mixer(0, scale=0.45)) > SEEN
    assert changed(mixer(1, softcap=5.0)) > SEEN
    assert changed(lambda c: c["layers"][1]["mlp"]["expert"].update(
        limit=0.8)) > SEEN
    assert changed(lambda c: c["layers"][1]["mlp"]["router"].update(top=2)) \
        > SEEN
    assert changed(lambda c: c["layers"][3].update(
        weights_of=1, mlp=None)) > SEEN
    for name in ("l0.mix.q.norm", "l1.mix.k.norm", "l5.mix.pb", "l4.canon1",
                 "l1.canon2", "l0.norm1", "l0.norm1b", "l5.norm2",
                 "l1.norm2b", "l1.mlp.router", "l1.mlp.correction",
                 "final.norm"):
        assert changed(edit_w=roll(name)) > SEEN, name
    for name in ("l0.canon1", "l5.canon2"):        # taps the other way round
        assert changed(edit_w=lambda v: v.update(
            {name: v[name].flip(1)})) > SEEN, name


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


def test_shared_tensors_equal_copies(std, tmp_path):
    """A layer that runs with another one's tensors is a copy of it with a
    cache of its own."""
    cfg, w, folder = std
    c, v = copy.deepcopy(cfg), dict(w)
    for i, x in enumerate(c["layers"]):
        j = x.pop("weights_of", None)
        if j is not None:
            v.update({f"l{i}." + n.split(".", 1)[1]: t.clone()
                      for n, t in w.items() if n.startswith(f"l{j}.")})
    toks = U.tokens(90, cfg["vocab"], seed=5)
    cuts = [40, 7, 1]
    a = U.feed(replay(folder), "a", toks, cuts)
    assert torch.equal(a, U.feed(replay(U.write(tmp_path, c, v)), "a", toks,
                                 cuts))


def loud_key_model():
    """One layer whose token 1 has a key that every query asks for, in chunks
    of 33: from the next chunk on it is gone."""
    cfg = U.config([U.layer(heads=1, kv_heads=1, dim=8, vdim=16, chunk=33,
                            scale=1.0, softcap=9.0, mlp=None)])
    w = U.weights(cfg, seed=8)
    w["l0.canon1"].zero_()
    w["embed"][:, 0] = 0.0
    w["embed"][1, 0] = 3.0                       # only token 1 uses column 0
    w["embed"][:, 1] = 1.0                       # every token has column 1
    w["l0.mix.q"].zero_()
    w["l0.mix.q"][0, 1] = 4.0                    # q = (+-1, 0, ...) always
    w["l0.mix.k"][0].zero_()
    w["l0.mix.k"][0, 0] = 9.0
    w["l0.mix.q.norm"][0] = w["l0.mix.k.norm"][0] = 1.0
    w["l0.mix.pb"][:] = -6.0
    return cfg, w


@pytest.mark.parametrize("cuts", [[80], [10, 1], [30, 2, 1], [16, 17, 2]])
def test_key_is_gone_with_its_chunk(tmp_path, cuts):
    """Positions 32 and 33 see and do not see the key at 7, in prompts, short
    portions and decoding."""
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
    assert moved[32] > 0.3 and moved[33] < 1e-9      # the test is sharp
    d = (U.feed(r, "b", other, cuts).double() - got).abs().amax(-1)
    assert d[32] > 0.3 and d[33:].max() == 0


def test_convolution_reaches_across_chunks(tmp_path):
    """What a token was matters taps - 1 tokens on, whatever the chunks, and
    no further in one layer."""
    cfg = U.config([U.layer(chunk=1, mlp=None)], taps=4)
    w = U.weights(cfg, seed=2)
    r = replay(U.write(tmp_path, cfg, w))
    toks = U.tokens(20, cfg["vocab"])
    other = list(toks)
    other[9] = (toks[9] + 1) % cfg["vocab"]
    for i, cuts in enumerate(([20], [10, 1], [11, 2], [1])):
        a, b = (U.feed(r, f"{i}{n}", t, cuts)
                for n, t in enumerate((toks, other)))
        d = (a - b).abs().amax(-1)
        assert (d[9:13] > 1e-2).all() and d[13:].max() == d[:9].max() == 0


def mixed_run(r, cfg, w, lens, seed=0, limits=lambda toks: TOL):
    """Requests of these lengths through random portions, single tokens and
    pauses, at most four live, each checked against itself alone; the largest
    error over its limit."""
    import test_tefezen
    return test_tefezen.mixed_run(r, cfg, w, lens, seed, limits,
                                  forward=O.forward)


def fill_caches(r, value):
    for c in r.engine.runner.kv_caches:
        for t in (*c.mixer, *c.tails):
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


_PAIR = [U.layer(chunk=7, mlp=U.dense(8)), U.layer(chunk=300)]
ODD = {
    "ones": U.config([U.layer(1, 1, 1, 1, 1, mlp=U.moe(1, 0, 1, 1)),
                      U.layer(1, 1, 1, 1, 2, mlp=U.dense(1))],
                     width=3, vocab=11, taps=1),
    "odd": U.config([U.layer(6, 3, 5, 7, 11, mlp=U.moe(3, 4, 5, 5)),
                     U.layer(7, 1, 9, 3, 29, mlp=U.dense(13)),
                     U.layer(5, 5, 7, 9, 3, mlp=None)],
                    width=21, vocab=37, taps=3),
    "many taps": U.config([U.layer(chunk=9), U.layer(mlp=None)], taps=12),
    "two taps": U.config([U.layer(chunk=17)], taps=2),
    "one of each run thrice": U.config(
        _PAIR + [U.again(_PAIR, i) for i in (1, 0, 0, 1)]),
    "negative scale, tight cap": U.config(
        [U.layer(scale=-0.8, softcap=0.6), U.layer(softcap=200.0)]),
    "many heads": U.config([U.layer(20, 1, 8, 8, 12),
                            U.layer(38, 2, 8, 8, 12)]),
    "identity mostly": U.config([U.layer(mlp=U.moe(2, 9, 1, 8)),
                                 U.layer(mlp=U.moe(1, 3, 4, 8))]),
    "equal sizes": U.config([U.layer(8, 8, 8, 8, 8,
                                     mlp=U.moe(8, 8, 8, 8, 8.0)),
                             U.layer(8, 1, 8, 8, 8, mlp=U.dense(8))],
                            width=8, vocab=8, taps=8),
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


def test_prefix_caching_is_refused_but_with_one_tap(std, tmp_path):
    """Shared pages do not restore the inputs of a convolution; with one tap
    there are none to keep, and shared pages serve a second prompt."""
    assert not engine(std[2], enable_prefix_caching=True) \
        .config.enable_prefix_caching
    cfg = U.config([U.layer(chunk=40), U.layer(mlp=U.dense())], taps=1)
    w = U.weights(cfg, seed=6)
    folder = U.write(tmp_path, cfg, w)
    head = U.tokens(50, cfg["vocab"])
    prompts = [head + U.tokens(n, cfg["vocab"], seed=n) for n in (3, 9)]
    eng = engine(folder, enable_prefix_caching=True)
    got = [eng.generate([p], GREEDY)[0] for p in prompts]
    assert got == [O.greedy(cfg, w, p, 12) for p in prompts]
    assert eng.runner.block_manager.cache_hits == 1


def test_preset_runs_and_sampling_is_seeded():
    kw = dict(model="tiny-mutusun", max_num_seqs=2, max_model_len=64,
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
        del v["l1.mlp.e4.up"]
    elif edit == "extra":
        v["l3.norm1"] = v["l1.norm1"].clone()     # a layer without tensors
    else:
        v["l0.canon1"] = v["l0.canon1"][:, :-1]
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
             lambda c: c["layers"][3].update(weights_of=2),
             lambda c: c["layers"][3].update(weights_of=9),
             lambda c: c["layers"][3].update(weights_of=0),
             lambda c: c["layers"][0]["mixer"].update(kv_heads=4),
             lambda c: c["layers"][0]["mixer"].update(softcap=0.0),
             lambda c: c["layers"][5]["mlp"]["router"].update(top=5),
             lambda c: c["canon"].update(taps=0)]
    for i, edit in enumerate(edits):
        with pytest.raises(ValueError):
            load(i, edit)


def test_cache_layout(std):
    from hyperspot.engine.layer_spec import (ConvTail, PagedKV, cache_parts)
    spec = EngineConfig(model=std[2]).spec()
    assert spec.has_state
    layout = spec.cache_layout(1)
    assert [len(c.tails) for c in layout] == [2, 2, 1, 2, 1, 2, 2]
    assert layout[0].mixer == PagedKV(2, 24, 16, True)
    assert layout[0].tails[0] == ConvTail(3, 56)
    assert layout[0].tails[0].bytes_per_slot(2) == 2 * 3 * 56
    assert len(cache_parts(layout)) == 7 + 12
    caches = engine(std[2]).runner.kv_caches
    at = {t.data_ptr() for c in caches for t in (*c.mixer, *c.tails)}
    assert len(at) == 2 * 7 + 12            # every run has its own
    assert EngineConfig(model="tiny-mutusun").spec().cache_layout(2)[0] \
        .mixer.kv_heads == 1


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
    own = [U.layer(heads=4, vdim=12, mlp=U.dense(20)),
           U.layer(heads=8, mlp=U.moe(3, 2, 3, 6))]
    cfg = U.config(own + [U.again(own, 1), U.layer(mlp=None)])
    w = U.weights(cfg, seed=7)
    folder = U.write(tmp_path, cfg, w)
    prompts = [U.tokens(30, 272), U.tokens(6, 272, seed=1)]
    want = [O.greedy(cfg, w, p, 12) for p in prompts]
    with mp.Manager() as mgr:
        results = mgr.dict()
        mp.spawn(_tp_rank, args=(2, folder, prompts, 29653, results),
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
