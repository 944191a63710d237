"""Nudadra through the framework (config registry, weight images, sequence state cache, step scheduler,
kernels) against the plain float64 oracle in ``nudadra_oracle.py``.

Every test runs on the CPU backend (plain PyTorch ops) and, marked ``gpu``, on the HIP kernels.  The models
are tiny and random; fp32 matrix products make the comparison sharp (a window one token off, a block seen one
row early, a mean over the wrong rows, a lost recurrent state, a pass that reads another pass's pages or misses
its step vector shows as an error thousands of times the tolerance), and some tests run the bf16 mode.  Where
random weights would hide a fault, the weights are set so that one token dominates."""
import json
import math
import os
import pickle
import subprocess
import sys

import numpy as np
import pytest
import torch

import nudadra_oracle as oracle
import nudadra_util as nu
from conftest import gpu_available
from flexible_llm_sharding_amd.runtime.batch import StepEntry, pack_step
from flexible_llm_sharding_amd.serve import generate, load_runner

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
TOL = 2e-4          # fp32 products against float64, relative to a logit row's spread
F = torch.float64


@pytest.fixture(autouse=True)
def _need_gpu(request):
    params = getattr(getattr(request.node, "callspec", None), "params", {})
    if "cuda" in str(params.get("device", "")) and not gpu_available():
        pytest.skip("no GPU")


def build(tmp_path, layers, seed=0, dtype=torch.float32, device="cpu", **kw):
    cfg = nu.config(layers, **{k: v for k, v in kw.items() if k in ("width", "vocab", "eps", "emb", "loop")})
    sd = nu.random_weights(cfg, seed, **({"std": kw["std"]} if "std" in kw else {}))
    path = nu.write_model(str(tmp_path / f"m{seed}"), cfg, sd)
    runner = load_runner(path, dtype, device, max_tokens=kw.get("max_tokens", 64), max_seqs=kw.get("max_seqs", 2),
                         layer_num_per_shard=kw.get("lnps"), token_budget=kw.get("token_budget", 16384),
                         resident=kw.get("resident", True))
    return cfg, sd, runner, path


def run_cut(runner, rid, toks, cuts, end=True):
    """Feed ``toks`` in portions of the sizes ``cuts`` (the rest one by one) -> logits of every position."""
    out, at = [], 0
    sizes = list(cuts) + [1] * (len(toks) - sum(cuts))
    for n in sizes:
        last = at + n == len(toks)
        r = runner.step([StepEntry(rid, toks[at:at + n], range(n))], [rid] if (last and end) else [])
        out.append(r[0][0])
        at += n
    return np.concatenate(out, 0)


# windows and blocks: 11 / 6, 3 / 8 (a block longer than the window), 20 / 5; blocks of 6, 8 and 5 tokens give the
# stack three lists of block pages; layers 1 and 2 run three times
STACK = [nu.layer(),
         nu.layer(nu.left(heads=3, kv_heads=3, dim=8, vdim=5, rot_dims=8, base=1000.0, scale=0.7, size=3, pool=8, scaling=None),
                  nu.right(heads=3, vdim=5, state=20, groups=1, norm_groups=1, conv=2)),
         nu.layer(nu.left(heads=4, kv_heads=1, dim=6, vdim=12, rot_dims=2, size=20, pool=5), nu.right(heads=6, vdim=4, state=3, groups=3, norm_groups=8), None),
         nu.layer(nu.left(size=7, pool=6), nu.right(conv=6), 33)]
LOOP = (1, 3, 3)


# ------------------------------------------------------------------ each mechanism alone
def _only(sd, n_layers, side):
    """Weights with one side of every mixer silenced (its output norm's weight set to zero)."""
    for i in range(n_layers):
        for s in ("left", "right"):
            if s != side:
                sd[f"l{i}.mix.{s}.out"] = torch.zeros_like(sd[f"l{i}.mix.{s}.out"])
    return sd


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name,layers,side,kw", [
    ("pooled-window", [nu.layer(nu.left(scale=1.5), ff=None)], "left", {}),
    ("window-of-one-blocks-of-one", [nu.layer(nu.left(size=1, pool=1), ff=None)], "left", {}),
    ("blocks-of-one-are-full-attention", [nu.layer(nu.left(size=9, pool=1), ff=None)], "left", {}),
    ("window-shorter-than-a-block", [nu.layer(nu.left(size=2, pool=13), ff=None)], "left", {}),
    ("window-longer-than-the-sequence", [nu.layer(nu.left(size=64, pool=4), ff=None)], "left", {}),
    ("window-and-block-of-a-page", [nu.layer(nu.left(size=16, pool=16), ff=None)], "left", {}),
    ("window-a-multiple-of-the-block", [nu.layer(nu.left(size=12, pool=4), ff=None)], "left", {}),
    ("no-rotation-one-head", [nu.layer(nu.left(heads=1, kv_heads=1, dim=4, vdim=3, rot_dims=0), ff=None)], "left", {}),
    ("unscaled-rotation-of-the-whole-head", [nu.layer(nu.left(rot_dims=10, scaling=None), ff=None)], "left", {}),
    ("every-pair-slowed", [nu.layer(nu.left(scaling={"factor": 2.0, "original": 8, "fast": 64.0, "slow": 32.0}), ff=None)], "left", {}),
    ("no-pair-slowed", [nu.layer(nu.left(scaling={"factor": 5.0, "original": 4000, "fast": 0.01, "slow": 0.001}), ff=None)], "left", {}),
    ("factor-one", [nu.layer(nu.left(scaling={"factor": 1.0, "original": 24, "fast": 4.0, "slow": 0.5}), ff=None)], "left", {}),
    ("wide-heads", [nu.layer(nu.left(heads=2, kv_heads=1, dim=150, vdim=130, rot_dims=140, scale=0.1, size=9, pool=4), ff=None)], "left", {"std": 0.15}),
    ("state-space", [nu.layer(ff=None)], "right", {}),
    ("state-space-one-head-one-state-row-one-tap", [nu.layer(rm=nu.right(heads=1, vdim=1, state=1, groups=1, norm_groups=1, conv=1), ff=None)], "right", {}),
    ("state-space-wide", [nu.layer(rm=nu.right(heads=2, vdim=70, state=37, groups=2, norm_groups=7, conv=9), ff=None)], "right", {}),
    ("state-space-a-group-for-all", [nu.layer(rm=nu.right(heads=5, groups=1, norm_groups=15), ff=None)], "right", {}),
    ("feed-forward-alone", [nu.layer(ff=41)], "none", {}),
    ("both-sides-and-feed-forward", [nu.layer(ff=41), nu.layer(ff=7)], "both", {}),
    ("loop-of-one-layer", [nu.layer(), nu.layer(ff=None), nu.layer()], "both", {"loop": (1, 2, 4)}),
    ("loop-over-all", [nu.layer(), nu.layer(ff=None)], "both", {"loop": (0, 2, 2)}),
    ("loop-once-still-enters", [nu.layer(), nu.layer()], "both", {"loop": (1, 2, 1)}),
    ("unit-embedding-scale-width-not-a-multiple-of-four", [nu.layer(), nu.layer()], "both", {"emb": 1.0, "width": 35, "loop": (0, 1, 2)}),
    ("width-of-one", [nu.layer()], "both", {"width": 1, "std": 1.0}),
])
def test_mechanism_alone(tmp_path, device, name, layers, side, kw):
    cfg = nu.config(layers, **{k: v for k, v in kw.items() if k != "std"})
    sd = nu.random_weights(cfg, 3, std=kw.get("std", 0.3))
    if side != "both":
        sd = _only(sd, len(layers), side)
    runner = load_runner(nu.write_model(str(tmp_path / "m"), cfg, sd), torch.float32, device, max_tokens=64)
    toks = nu.tokens(45, cfg["vocab"], 1)
    want = nu.oracle_logits(cfg, sd, toks)
    assert nu.rel_err(run_cut(runner, "a", toks, [len(toks)]), want) < TOL
    assert nu.rel_err(run_cut(runner, "b", toks, [30, 2]), want) < TOL
    assert nu.rel_err(run_cut(runner, "c", toks, [3, 20]), want) < TOL
    runner.close()


def test_oracle_parts_agree_with_their_definitions():
    """The oracle's own pieces on hand-made inputs: the pair layout, the rescaled frequencies and their amplitude,
    what a row sees, the means, the recurrence and its convolution by hand, the order of a loop."""
    x = torch.tensor([[[0.0, 0.0, 5.0, 6.0, 7.0]], [[1.0, 0.0, 0.0, 2.0, 7.0]]], dtype=F)
    r = oracle.rotate(x, {"dims": 4, "base": 100.0})                   # pairs (0, 2) and (1, 3); f = 1, 0.1
    assert torch.allclose(r[1, 0], torch.tensor([math.cos(1.0), -2 * math.sin(0.1), math.sin(1.0), 2 * math.cos(0.1), 7.0], dtype=F))
    assert torch.equal(r[0], x[0])
    rot = {"dims": 16, "base": 100.0, "scaling": {"factor": 8.0, "original": 64, "fast": 4.0, "slow": 1.0}}
    f, amp = oracle.rot_freqs(rot)
    f0, one = oracle.rot_freqs({"dims": 16, "base": 100.0})
    ratio = [a / b for a, b in zip(f, f0)]                              # the ramp runs from entry 1 to entry 5
    assert one == 1.0 and abs(amp - (0.1 * math.log(8.0) + 1.0)) < 1e-15
    assert ratio[0] == 1.0 and ratio[1] == 1.0 and abs(ratio[3] - (0.5 + 0.5 / 8)) < 1e-12 and all(abs(q - 1 / 8) < 1e-12 for q in ratio[5:])
    # window 5, blocks of 4: at position 12 the tokens 8 .. 12 and the blocks that end at 7 or earlier
    assert oracle.visible(12, 5, 4) == ([8, 9, 10, 11, 12], [0, 1])
    assert oracle.visible(11, 5, 4) == ([7, 8, 9, 10, 11], [0]) and oracle.visible(7, 5, 4) == ([3, 4, 5, 6, 7], [])
    assert oracle.visible(8, 5, 4) == ([4, 5, 6, 7, 8], [0]) and oracle.visible(0, 5, 4) == ([0], [])
    # equal scores: the weights are equal, a block counts as one key and carries its mean value
    v = torch.arange(9, dtype=F)[:, None]
    o = oracle.pooled_window_attention(torch.zeros(9, 2, dtype=F), torch.randn(9, 2, dtype=F), v, 1.0, 5, 4)
    assert abs(float(o[8]) - (1.5 + 4 + 5 + 6 + 7 + 8) / 6) < 1e-12 and abs(float(o[7]) - 5.0) < 1e-12
    u = torch.tensor([[1.0], [10.0], [100.0]], dtype=F)
    assert oracle.short_conv(u, torch.tensor([[3.0, 2.0]], dtype=F), torch.tensor([0.5], dtype=F)).flatten().tolist() == [2.5, 23.5, 230.5]
    assert oracle.schedule({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert oracle.schedule({"layers": [0] * 2}) == [(0, None), (1, None)]
    # the recurrence by hand: one head, one group, N = P = 1, no history in the convolution, dt = ln 2, A = 1 -> decay 1/2
    big = 40.0                                                          # silu(40) = 40 up to e^-40
    sd = {"in": torch.tensor([[big], [big], [big], [big], [0.0]], dtype=F), "conv": torch.tensor([[1.0]] * 3, dtype=F),
          "conv.b": torch.zeros(3, dtype=F), "dt_bias": torch.zeros(1, dtype=F), "A_log": torch.zeros(1, dtype=F),
          "D": torch.tensor([3.0], dtype=F), "norm": torch.ones(1, dtype=F), "o": torch.ones(1, 1, dtype=F)}
    m = {"heads": 1, "vdim": 1, "state": 1, "groups": 1, "norm_groups": 1, "conv": 1}
    eps = 1e15                                                          # (next to y^2 ~ 1e13: the norm keeps magnitudes apart)
    got = oracle.state_space(sd, "", m, torch.ones(2, 1, dtype=F), eps).flatten()
    s0 = math.log(2) * big * big
    y = [(s0 * big + 3 * big) * big, ((s0 / 2 + s0) * big + 3 * big) * big]
    assert np.allclose(got.numpy(), [v / math.sqrt(v * v + eps) for v in y], rtol=1e-12)


# ----------------------------------------------- prompts, portions, decoding, first tokens
@pytest.mark.parametrize("device", DEVICES)
def test_prefill_portions_and_decode(tmp_path, device):
    """The same sequence whole, token by token, and in portions of 2, 3, 7, 16 and 17 tokens: windows, half-filled
    blocks, convolution inputs and states of all passes cross the cuts."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=5, device=device, loop=LOOP)
    toks = nu.tokens(50, cfg["vocab"], 2)
    want = nu.oracle_logits(cfg, sd, toks)
    for cuts in ([50], [], [2, 2, 3, 7, 16, 17], [17, 16, 2], [2] * 25, [1, 2, 40]):
        assert nu.rel_err(run_cut(runner, "r", toks, cuts), want) < TOL, cuts
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_residual_rows_after_every_layer_run(tmp_path, device):
    """What leaves every layer run (a looped layer counts each time) against the oracle, through the layer
    functions on the runner's own weights and cache; the embedding rows beside them stay as they were."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=4, device=device, loop=LOOP)
    toks = nu.tokens(21, cfg["vocab"], 8)
    trace = []
    nu.oracle_logits(cfg, sd, toks, trace)
    batch = pack_step([StepEntry("t", toks, [len(toks) - 1])], runner.seq_cache)
    meta = batch.device_tensors(runner.dev)
    W = {}
    for k in range(len(runner.my_shards)):
        W.update(runner.prefetcher.acquire(k))
    state, n = None, 0
    x0 = (sd["embed"].double()[toks] * 1.7)
    for name in runner.names:
        state = runner.family.run_layer(runner.ctx, name, W[name], state, batch, meta)
        if name[0] == "l":
            got = state.cpu().double()
            assert (got[:, :36] - trace[n]).abs().max() < 1e-4 * trace[n].abs().max(), name
            assert (got[:, 36:] - x0).abs().max() < 1e-5
            n += 1
    assert n == len(trace) == 8
    runner.seq_cache.release("t")
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_over_pages_and_blocks(tmp_path, device):
    """A short prompt, then 150 decoded tokens: pages fill and are given back behind the windows, blocks complete
    and stay, block pages fill (16 blocks of 5 tokens a page)."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=6, device=device, loop=LOOP)
    toks = nu.tokens(155, cfg["vocab"], 7)
    got = run_cut(runner, "r", toks, [5], end=False)
    assert nu.rel_err(got, nu.oracle_logits(cfg, sd, toks)) < TOL
    cache, r = runner.seq_cache, runner.seq_cache.requests["r"]
    # window 20: the next token (155) still reads 136 ..; pages 0 .. 7 are back in the pool
    assert cache.pages_trimmed == 8 and [p >= 0 for p in r.pages] == [False] * 8 + [True] * 2
    assert {P: len(v) for P, v in r.block_pages.items()} == {5: 2, 6: 2, 8: 2}
    free = {P: len(cache.free_block_pages[P]) for P in cache.block_sizes}
    cache.release("r")
    assert all(len(cache.free_block_pages[P]) == free[P] + 2 for P in cache.block_sizes)
    assert len(cache.free_pages) == cache.n_pages
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_unfinished_blocks_survive_behind_the_window(tmp_path, device):
    """A window of two tokens and blocks of 40: while a block fills, its tokens lie many pages behind the window
    and must not be given back; once it is complete they are."""
    cfg, sd, runner, _ = build(tmp_path, [nu.layer(nu.left(size=2, pool=40, scale=1.2))], seed=16, device=device)
    toks = nu.tokens(100, cfg["vocab"], 9)
    want = nu.oracle_logits(cfg, sd, toks)
    assert nu.rel_err(run_cut(runner, "d", toks[:39], [10], end=False), want[:39]) < TOL
    assert runner.seq_cache.pages_trimmed == 0
    got = np.concatenate([runner.step([StepEntry("d", [t], [0])])[0][0] for t in toks[39:]])
    assert nu.rel_err(got, want[39:]) < TOL
    assert runner.seq_cache.pages_trimmed == 5                     # position 80 opens the third block
    runner.seq_cache.release("d")
    for cuts in ([38, 2, 2, 58], [39, 1, 40, 20], [100]):
        assert nu.rel_err(run_cut(runner, "p", toks, cuts), want) < TOL, cuts
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(tmp_path, device):
    """Sequences of one, two and three tokens, whole and decoded."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=8, device=device, loop=LOOP)
    for n in (1, 2, 3):
        toks = nu.tokens(n, cfg["vocab"], 20 + n)
        want = nu.oracle_logits(cfg, sd, toks)
        assert nu.rel_err(run_cut(runner, "w", toks, [n]), want) < TOL
        assert nu.rel_err(run_cut(runner, "d", toks, []), want) < TOL
    runner.close()


# ------------------------------------------------------------ batches, pages and slots
@pytest.mark.parametrize("device", DEVICES)
def test_unequal_batch_equals_each_alone(tmp_path, device):
    """Requests of 1, 9, 33 and 50 tokens in one step, then decoded together while the short ones
    finish first; also cut into two micro-batches by a small token budget."""
    for budget in (16384, 40):
        cfg, sd, runner, _ = build(tmp_path, STACK, seed=9, device=device, token_budget=budget, loop=LOOP)
        lens, extra = [1, 9, 33, 50], [3, 12, 0, 6]
        seqs = [nu.tokens(n + e, cfg["vocab"], 30 + i) for i, (n, e) in enumerate(zip(lens, extra))]
        want = [nu.oracle_logits(cfg, sd, s) for s in seqs]
        got = [[] for _ in seqs]
        live = list(range(4))
        res = runner.step([StepEntry(i, seqs[i][:lens[i]], range(lens[i])) for i in live], [i for i in live if extra[i] == 0])
        for i, r in zip(live, res):
            got[i].append(r[0])
        for t in range(max(extra)):
            live = [i for i in range(4) if extra[i] > t]
            res = runner.step([StepEntry(i, [seqs[i][lens[i] + t]], [0]) for i in live], [i for i in live if extra[i] == t + 1])
            for i, r in zip(live, res):
                got[i].append(r[0])
        for i in range(4):
            assert nu.rel_err(np.concatenate(got[i], 0), want[i]) < TOL, (budget, i)
        assert not runner.seq_cache.requests
        runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_portions_and_decoded_rows_in_one_step(tmp_path, device):
    """One step that starts a request, continues another by a portion that completes several blocks, and decodes a
    third whose row completes a block: each equals itself alone."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=10, device=device, loop=LOOP)
    a, b, c = nu.tokens(30, cfg["vocab"], 1), nu.tokens(60, cfg["vocab"], 2), nu.tokens(24, cfg["vocab"], 3)
    wa, wb, wc = (nu.oracle_logits(cfg, sd, s) for s in (a, b, c))
    runner.step([StepEntry("b", b[:21], []), StepEntry("c", c[:23], [])])
    res = runner.step([StepEntry("a", a[:29], range(29)), StepEntry("b", b[21:59], range(38)), StepEntry("c", c[23:], [0])])
    for r, w in zip(res, (wa[:29], wb[21:59], wc[23:])):
        assert nu.rel_err(r[0], w) < TOL
    res = runner.step([StepEntry("a", a[29:], [0]), StepEntry("b", b[59:], [0])], ["a", "b", "c"])
    assert nu.rel_err(res[0][0], wa[29:]) < TOL and nu.rel_err(res[1][0], wb[59:]) < TOL
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_pages_blocks_and_slots_used_again(tmp_path, device):
    """Requests come and go through pools of two slots and a few pages: whoever inherits a page, a block page or a
    slot (with the last owner's keys, means and states still in it) computes what it computes alone, and pools
    that run out grow without disturbing the live request."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=11, device=device, max_tokens=40, max_seqs=2, loop=LOOP)
    cache = runner.seq_cache
    a, b, c = (nu.tokens(n, cfg["vocab"], 40 + n) for n in (37, 22, 130))
    wa, wb, wc = (nu.oracle_logits(cfg, sd, s) for s in (a, b, c))
    assert nu.rel_err(run_cut(runner, "a", a, [30]), wa) < TOL
    ga = run_cut(runner, "a2", a, [10, 2], end=False)                       # stays alive
    gb = run_cut(runner, "b", b, [22])                                      # inherits a's first slot
    assert cache.slots_reused > 0 and cache.pages_reused > 0 and cache.block_pages_reused > 0
    nb = dict(cache.n_block_pages)
    gc = run_cut(runner, "c", c, [3, 120])
    assert any(cache.n_block_pages[P] > nb[P] for P in nb)                  # (the block pools ran out and grew)
    n0 = cache.n_slots
    others = [run_cut(runner, f"x{i}", b, [5], end=False) for i in range(3)]    # more requests than slots
    assert cache.n_slots > n0
    tail = runner.step([StepEntry("a2", [a[0]], [0])], ["a2"])[0][0]         # a2's state survived the growth
    assert nu.rel_err(tail, nu.oracle_logits(cfg, sd, a + [a[0]])[-1:]) < TOL
    for g, w in ((ga, wa), (gb, wb), (gc, wc)) + tuple((o, wb) for o in others):
        assert nu.rel_err(g, w) < TOL
    runner.close()


# ------------------------------------------- one token that stands out, at every edge of a window and a block
def _marked_model(tmp_path, size, pool, side="left", heads=2, dim=8, vdim=6):
    """One layer whose weights make one marked token decide every row that sees it.  Channel 0 of the embedding is
    the same for every token, channel 1 is zero except for the marked token.  ``left``: every query is u, a
    plain token's key next to nothing, the marked token's a large multiple of u: its score stands out among
    hundreds even divided by the block length, its value is large, and as part of a block it counts 1 / pool.
    ``right``: the state forgets next to nothing, and only the marked token writes much.  The other side is silenced."""
    D, vocab, mark = 24, 40, 7
    cfg = nu.config([nu.layer(nu.left(heads=heads, kv_heads=1, dim=dim, vdim=vdim, rot_dims=2, base=1e6, scale=1.0, size=size,
                                      pool=pool, scaling=None),
                              nu.right(heads=2, vdim=6, state=4, groups=1, norm_groups=1, conv=3), ff=None)],
                    width=D, vocab=vocab, emb=1.0)
    sd = {k: v.float() for k, v in nu.random_weights(cfg, 12, std=0.05).items()}
    sd["embed"] *= 0.05
    sd["embed"][:, 0] = 4.0
    sd["embed"][:, 1] = 0.0
    sd["embed"][mark, 1] = 4.0
    sd["l0.norm1"] = torch.ones(())
    x, y = "l0.mix.left.", "l0.mix.right."
    if side == "left":
        sd[y + "out"][:] = 0.0
        u = torch.zeros(dim)
        u[2:] = 1.0 / math.sqrt(dim - 2)                                # (entries 0, 1 are a rotated pair: left out)
        n = math.sqrt(D)                                                # channel 0 of a plain normed row
        for hh in range(heads):
            sd[x + "q"][hh * dim:(hh + 1) * dim] = 0.0
            sd[x + "q"][hh * dim:(hh + 1) * dim, 0] = u * (9.0 / n)
        sd[x + "k"][:] = 0.0
        sd[x + "k"][:, 1] = u * (1.4 * max(pool, 1) / n * math.sqrt(2))
        sd[x + "v"][:, 1] = 3.0
        sd[x + "g"][:] = 0.0
    else:
        sd[x + "out"][:] = 0.0
        inner, gn = 12, 4
        sd[y + "A_log"][:] = -8.0
        sd[y + "dt_bias"][:] = -1.0
        sd[y + "in"][inner:2 * inner, 1] = 3.0                          # x: the mark's
        sd[y + "in"][2 * inner:2 * inner + gn, 1] = 2.0                 # B: the mark's
        sd[y + "in"][2 * inner + gn:2 * inner + 2 * gn, 0] = 1.0        # C and z: everyone's
        sd[y + "in"][:inner, 0] = 1.0
    sd = {k: v.to(torch.bfloat16) for k, v in sd.items()}
    return cfg, sd, nu.write_model(str(tmp_path / f"mark_{side}_{size}_{pool}"), cfg, sd), mark, vocab


def _sees(place, i, size, pool):
    """How row i sees position ``place``: "token", "block" or "" (not at all)."""
    if i < place:
        return ""
    if i - place < size:
        return "token"
    return "block" if (place // pool + 1) * pool - 1 <= i - size else ""


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,pool", [(11, 6), (16, 16), (5, 12), (40, 3)])
def test_one_token_stands_out_at_window_and_block_edges(tmp_path, device, size, pool):
    """The marked token at the start, on both sides of page and block borders and hundreds of places back: the rows
    that see it (as a token, in a block) and those that do not (before it; after it left the window while its
    block is not yet seen) are exactly the design's, in prompts, in portions cut right behind it and where its
    visibility changes, and in decoding."""
    cfg, sd, path, mark, vocab = _marked_model(tmp_path, size, pool)
    runner = load_runner(path, torch.float32, device, max_tokens=320, max_seqs=2)
    rng = np.random.default_rng(0)
    n = 96
    base = [int(t) for t in rng.integers(8, vocab, n)]
    kinds = set()
    plain = nu.oracle_logits(cfg, sd, base)
    for place in (0, pool - 1, pool, 15, 16, 2 * pool - 1, 33):
        toks = list(base)
        toks[place] = mark
        want = nu.oracle_logits(cfg, sd, toks)
        diff = np.array([nu.rel_err(plain[i:i + 1], want[i:i + 1]) for i in range(n)])      # (per row, relative to the row's spread)
        for i in range(n):
            how = _sees(place, i, size, pool)
            kinds.add(how)
            assert (diff[i] > 1000 * TOL) if how else (diff[i] == 0.0), (place, i, how, diff[i])
        gone, back = place + size, (place // pool + 1) * pool - 1 + size                     # first rows of the next two states
        assert nu.rel_err(run_cut(runner, "p", toks, [n]), want) < TOL, place
        cuts, at = [], 0
        for edge in sorted({place + 1, gone, back, back + 1}):
            if at < edge < n:
                cuts.append(edge - at)
                at = edge
        assert nu.rel_err(run_cut(runner, "e", toks, cuts), want) < TOL, place
        assert nu.rel_err(run_cut(runner, "d", toks, [max(1, place - 1)]), want) < TOL, place
    assert kinds == ({"", "token", "block"})
    # hundreds of places back
    toks = [int(t) for t in rng.integers(8, vocab, 300)]
    toks[1] = mark
    want = nu.oracle_logits(cfg, sd, toks)
    other = nu.oracle_logits(cfg, sd, [t if t != mark else 9 for t in toks])
    assert nu.rel_err(other[-1:], want[-1:]) > 100 * TOL
    assert nu.rel_err(run_cut(runner, "p", toks, [300]), want) < TOL
    assert nu.rel_err(run_cut(runner, "d", toks, [200, 70]), want) < TOL
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_one_token_stays_in_the_recurrent_state(tmp_path, device):
    """A marked token that the state-space side keeps for hundreds of rows: seen from every later row and no earlier
    one, through prompts, portions cut right behind it (the convolution's carried inputs) and decoding."""
    cfg, sd, path, mark, vocab = _marked_model(tmp_path, 11, 6, "right")
    runner = load_runner(path, torch.float32, device, max_tokens=320, max_seqs=2)
    rng = np.random.default_rng(1)
    n = 200
    for place in (0, 15, 60, n - 2):
        toks = [int(t) for t in rng.integers(8, vocab, n)]
        toks[place] = mark
        want = nu.oracle_logits(cfg, sd, toks)
        plain = nu.oracle_logits(cfg, sd, [t if t != mark else 9 for t in toks])
        diff = np.array([nu.rel_err(plain[i:i + 1], want[i:i + 1]) for i in range(n)])
        assert diff[:place].max(initial=0.0) == 0.0 and diff[place + 1:].min() > 50 * TOL
        assert nu.rel_err(run_cut(runner, "p", toks, [n]), want) < TOL, place
        cuts = [place + 1] + ([n - 20 - place - 1] if n - 20 - place - 1 > 0 else [])
        assert nu.rel_err(run_cut(runner, "d", toks, cuts), want) < TOL, place
    runner.close()


# ----------------------------------------------------- shards, bf16, generation
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("lnps", [1, 3])
def test_few_layers_per_shard_stream_weights(tmp_path, device, lnps):
    """Weights streamed shard by shard: the passes of a looped layer land in different shards (its image is
    loaded again) or in one (loaded once, shared); the embedding rows travel with the residual rows."""
    cfg = nu.config(STACK, loop=LOOP)
    sd = nu.random_weights(cfg, 13)
    path = nu.write_model(str(tmp_path / "s"), cfg, sd)
    runner = load_runner(path, torch.float32, device, max_tokens=64, layer_num_per_shard=lnps, resident=False)
    toks = nu.tokens(40, cfg["vocab"], 3)
    assert nu.rel_err(run_cut(runner, "r", toks, [20, 2]), nu.oracle_logits(cfg, sd, toks)) < TOL
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_bf16_products_stay_close(tmp_path, device):
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=14, device=device, dtype=torch.bfloat16, loop=LOOP)
    toks = nu.tokens(60, cfg["vocab"], 4)
    want = nu.oracle_logits(cfg, sd, toks)
    whole, cut = run_cut(runner, "a", toks, [60]), run_cut(runner, "b", toks, [9, 2, 20])
    assert nu.rel_err(whole, want) < 0.1 and nu.rel_err(cut, want) < 0.1      # (the worst row)
    assert nu.rel_err(cut, whole) < 0.1
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dim,vdim,size,pool", [(128, 128, 50, 8), (32, 32, 130, 5), (64, 128, 33, 32), (96, 96, 64, 3), (128, 64, 20, 1)])
def test_head_sizes_of_the_matrix_core_kernels(tmp_path, device, dim, vdim, size, pool):
    """bf16 with head sizes that the matrix-core prompt attention serves on the GPU: a prompt of several row tiles
    whose blocks fill several key tiles, a portion that continues it, then decoding; a marked token far back
    must not drown in the rounding."""
    cfg, sd, path, mark, vocab = _marked_model(tmp_path, size, pool, heads=3, dim=dim, vdim=vdim)
    runner = load_runner(path, torch.bfloat16, device, max_tokens=512)
    toks = [int(t) for t in np.random.default_rng(5).integers(8, vocab, 260)]
    toks[21] = mark
    want = nu.oracle_logits(cfg, sd, toks)
    whole = run_cut(runner, "a", toks, [260])
    cut = run_cut(runner, "b", toks, [150, 70])
    for got, ref in ((whole, want), (cut, want), (cut, whole)):
        e = nu.row_errs(got, ref)
        assert e.max() < 0.08 and e.mean() < 0.03, (e.max(), e.mean())
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(tmp_path, device):
    """serve.generate: prompts of unequal length, 12 new tokens each; the tokens are the oracle's
    greedy continuation (recomputed from scratch at every step)."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=15, device=device, loop=LOOP)
    prompts = [nu.tokens(n, cfg["vocab"], 50 + n) for n in (3, 17, 26)]
    got = generate(runner, prompts, 12)
    for p, g in zip(prompts, got):
        z = nu.oracle_logits(cfg, sd, list(p) + list(g))
        for k, t in enumerate(g):
            row = z[len(p) + k - 1]
            top2 = np.sort(row)[-2:]
            if top2[1] - top2[0] > 1e-3:              # (a tie within rounding may go either way)
                assert t == int(row.argmax())
    assert not runner.seq_cache.requests
    runner.close()


# ----------------------------------------------------- command line, configuration, graphs, trace replay
def test_command_line_serves_the_model(tmp_path):
    from flexible_llm_sharding_amd import api
    from flexible_llm_sharding_amd.utils.tokenizer import write_synthetic_tokenizer
    cfg = nu.config(STACK, vocab=64, loop=LOOP)
    path = nu.write_model(str(tmp_path / "cli"), cfg, nu.random_weights(cfg, 16))
    write_synthetic_tokenizer(path, 64)
    prompts = [("w1 w2 w3", ("w4", "w5 w6")), ("w7", ("w8 w9 w10",))]
    pk = str(tmp_path / "p.pkl")
    with open(pk, "wb") as f:
        pickle.dump(prompts, f)
    out = str(tmp_path / "o.pkl")
    api.main(["--model_path", path, "--prompt_pickle", pk, "--output_file", out, "--num_gen_token", "3",
              "--num_gpus", "0" if not gpu_available() else "1", "--dtype", "float32", "--layer_num_per_shard", "2"])
    with open(out, "rb") as f:
        scores = pickle.load(f)
    assert [s.shape for s in scores] == [(2, 3, 64), (1, 3, 64)]
    assert all(abs(float(s[i, j].astype(np.float32).sum()) - 1) < 2e-2 for s in scores for i in range(s.shape[0]) for j in range(3))


def test_config_is_read_not_assumed(tmp_path):
    """The registry picks the family by config.json's architecture; every pass of a looped layer has a state of its
    own and shares its layer's weight image; every tensor of the checkpoint lands, none is invented; a
    checkpoint that contradicts the config is refused at load."""
    from flexible_llm_sharding_amd.config import NudadraConfig, load_config
    from flexible_llm_sharding_amd.models import hybrid_family, nudadra
    from flexible_llm_sharding_amd.runtime.weights import CheckpointSource, HostStore
    cfg = nu.config(STACK, loop=LOOP)
    sd = nu.random_weights(cfg, 18)
    path = nu.write_model(str(tmp_path / "c"), cfg, sd)
    c = load_config(path)
    assert isinstance(c, NudadraConfig) and hybrid_family(c) is nudadra
    assert c.layer_names() == ["embed", "l0", "l1", "l2", "l1@1", "l2@1", "l1@2", "l2@2", "l3", "final.norm", "head"]
    assert c.state_width == 2 * 36 and c.embedding_scale == 1.7
    assert [c.loop_pass(n) for n in c.layer_names()[1:-2]] == [None, 0, None, 1, None, 2, None, None]
    spec = nudadra.state_spec(c)
    assert spec["paged"]["l0"] == spec["blocks"]["l0"][1] == {"k": 2 * 10, "v": 2 * 14} and spec["blocks"]["l1@2"] == (8, {"k": 24, "v": 15})
    assert set(spec["paged"]) == set(spec["slots"]) == set(spec["blocks"]) == set(c.layer_names()[1:-2])
    assert spec["slots"]["l2@1"] == {"conv": (3, 6 * 4 + 2 * 9), "state": (6, 3, 4)}
    names = {pl.hf_name for n in c.layer_names() for pl in nudadra.placements(c, n)}
    assert names == set(sd)
    assert json.loads(json.dumps(NudadraConfig.from_dict(c.to_dict()).to_dict())) == c.to_dict()
    store = HostStore.from_source(CheckpointSource(c, path, torch.float32), pinned=False)
    assert store.host_buffer("l2@1") is store.host_buffer("l2") and store.host_buffer("l3") is not store.host_buffer("l2")
    flat = NudadraConfig.from_dict(nu.config(STACK))
    assert flat.state_width == 36 and "loop_in" not in [s[0] for s in nudadra._specs(flat, "l1")]
    for edit in (lambda d: d["layers"][0].update(type="attention"),
                 lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=4),
                 lambda d: d["layers"][0]["mixer"]["left"]["rot"].update(dims=7),
                 lambda d: d["layers"][0]["mixer"]["left"]["rot"].update(dims=12),
                 lambda d: d["layers"][0]["mixer"]["left"]["mask"].update(size=0),
                 lambda d: d["layers"][0]["mixer"]["left"]["mask"].update(pool=0),
                 lambda d: d["layers"][0]["mixer"]["left"].update(vdim=600),
                 lambda d: d["layers"][0]["mixer"]["right"].update(groups=3),
                 lambda d: d["layers"][0]["mixer"]["right"].update(norm_groups=5),
                 lambda d: d["layers"][0]["mixer"]["right"].update(state=300),
                 lambda d: d["layers"][0]["mlp"].update(kind="moe"),
                 lambda d: d.update(loop={"start": 2, "stop": 9, "times": 2}),
                 lambda d: d.update(loop={"start": 2, "stop": 2, "times": 2})):
        bad = json.loads(json.dumps(cfg))
        edit(bad)
        with pytest.raises((NotImplementedError, ValueError)):
            NudadraConfig.from_dict(bad)
    wrong = json.loads(json.dumps(cfg))
    wrong["layers"][0]["mixer"]["left"]["vdim"] = 15
    nu.write_model(str(tmp_path / "w"), wrong, sd)
    with pytest.raises(ValueError):
        load_runner(str(tmp_path / "w"), torch.float32, "cpu")


@pytest.mark.gpu
def test_captured_decode_steps_equal_eager(tmp_path, monkeypatch):
    """Decode steps replay as captured HIP graphs; every replay is checked against the same steps run
    eagerly, with eager prompt steps of other requests and batch-size changes between the replays.  Blocks
    complete inside the captured steps."""
    if not gpu_available():
        pytest.skip("no GPU")

    def run(graphs: bool):
        monkeypatch.setenv("FLS_DECODE_GRAPHS", "1" if graphs else "0")
        cfg, sd, runner, _ = build(tmp_path, STACK, seed=21, device="cuda:0", dtype=torch.bfloat16, max_tokens=256, max_seqs=4, loop=LOOP)
        a, b, c = (nu.tokens(n, cfg["vocab"], 60 + n) for n in (60, 53, 45))
        outs = []
        runner.step([StepEntry("a", a[:10], [9]), StepEntry("b", b[:12], [11])])
        for t in range(40):
            live = [("a", a[10 + t]), ("b", b[12 + t])] + ([("c", c[9 + t - 8])] if t >= 8 else [])
            r = runner.step([StepEntry(i, [tok], [0]) for i, tok in live])
            outs += [x[0] for x in r]
            if t == 7:
                outs.append(runner.step([StepEntry("c", c[:9], [8])])[0][0])
            if t % 5 == 0:
                torch.cuda.synchronize()
        replays = runner._decode_graphs.replays if runner._decode_graphs is not None else 0
        runner.close()
        return np.concatenate(outs, 0), replays

    eager, n0 = run(False)
    graphed, n1 = run(True)
    assert n0 == 0 and n1 >= 30
    assert np.array_equal(eager, graphed)


def test_trace_run_program_replays_steps(tmp_path):
    """bin/trace_run as a process on a two-request schedule: prompts of unequal length in one step,
    then one token each; a flushed 'done <step>' after each step, logits files for the steps that
    want some, exit code 0 at end of input."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = nu.config(STACK[:3], vocab=37, loop=(1, 3, 2))
    sd = nu.random_weights(cfg, 19)
    path = nu.write_model(str(tmp_path / "t"), cfg, sd)
    out = tmp_path / "logits"
    a, b = nu.tokens(19, 37, 4), nu.tokens(3, 37, 5)
    p = subprocess.Popen([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32",
                          "--out", str(out), "--max-tokens", "32", "--device", "cpu"], stdin=subprocess.PIPE,
                         stdout=subprocess.PIPE, text=True, cwd=root)
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": a[:17], "want": [0, 16]}, {"id": "s", "tokens": b[:1], "want": [0]}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": a[17:18], "want": []}, {"id": "s", "tokens": b[1:2], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "q", "tokens": a[18:], "want": [0]}, {"id": "s", "tokens": b[2:], "want": [0]}], "end": ["q", "s"]}]
    for st in steps:
        p.stdin.write(json.dumps(st) + "\n")
        p.stdin.flush()
        while True:
            line = p.stdout.readline()
            assert line, "trace_run ended early"
            if line.strip() == f"done {st['step']}":
                break
    p.stdin.close()
    assert p.wait(timeout=60) == 0
    wa, wb = nu.oracle_logits(cfg, sd, a), nu.oracle_logits(cfg, sd, b)
    got = np.concatenate([np.fromfile(out / "0.f32", dtype="<f4").reshape(3, -1), np.fromfile(out / "2.f32", dtype="<f4").reshape(2, -1)])
    assert not (out / "1.f32").exists()
    assert nu.rel_err(got, np.concatenate([wa[[0, 16]], wb[[0]], wa[[18]], wb[[2]]])) < TOL


def test_bench_model_builder_runs_on_cpu():
    """The benchmark's synthetic stack (bench.py --hybrid --hybrid-family nudadra) at a toy size: random layer
    images straight into a host store, a prompt step and a decode step through the runner; and the stack beside it."""
    from flexible_llm_sharding_amd.engine import ShardedRunner
    from flexible_llm_sharding_amd.utils.hybrid_bench import FAMILIES, nudadra_config, synthetic_hybrid_store
    z = dict(width=64, heads=4, kv=2, dim=16, ff=96, experts=4, top=2, eff=16, blocks=2, mh=2, mp=8, state=8, chunk=12, vocab=50)
    cfg = nudadra_config(z)
    assert len(cfg.layer_names()) == 9 and FAMILIES["nudadra"][1](z).num_hidden_layers == 12
    src = synthetic_hybrid_store(cfg, "cpu", torch.float32)
    r = ShardedRunner(cfg, src, device="cpu", layer_num_per_shard=2, storage_location="cpu", compute_dtype=torch.float32,
                      state_tokens=64, state_seqs=2)
    out = r.step([StepEntry("a", list(range(20)), [19]), StepEntry("b", [1, 2, 3], [2])])
    assert out[0][0].shape == (1, 50) and np.isfinite(out[0][0]).all() and np.isfinite(out[1][0]).all()
    out = r.step([StepEntry("a", [5], [0]), StepEntry("b", [6], [])], ["a", "b"])
    assert out[1] is None and np.isfinite(out[0][0]).all() and not r.seq_cache.requests
    r.close()
