"""Numolorn through the framework (config registry, weight images, sequence state cache, step scheduler, kernels) against
the plain float64 oracle in ``numolorn_oracle.py``.

Every test runs on the CPU backend (plain PyTorch ops) and, marked ``gpu``, on the HIP kernels.  The models are tiny and
random; fp32 matrix products make the comparison sharp (a window one token off, a sink left out, a wrong previous token, a
lost recurrent state, an expert of a closed group or a pass that reads another pass's rows shows as an error thousands of
times the tolerance), and some tests run the bf16 mode.  Where random weights would hide a fault, the weights are set so
that one token dominates."""
import json
import math
import os
import pickle
import subprocess
import sys

import numpy as np
import pytest
import torch

import numolorn_oracle as oracle
import numolorn_util as nu
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
    cfg = nu.config(layers, **{k: v for k, v in kw.items() if k in ("width", "vocab", "eps", "logit_scale", "loop", "bigram")})
    sd = nu.random_weights(cfg, seed, **{k: v for k, v in kw.items() if k in ("std", "ranks")})
    if kw.get("edit"):
        kw["edit"](sd)
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


# every mixer with every kind of feed-forward, one without; layers 1 .. 3 run twice
STACK = [(nu.window(), nu.dense()),
         (nu.latent(), nu.moe()),
         (nu.delta(), nu.moe(experts=5, identity=1, top=2, ff=9, groups=None, scale=0.8, limit=2.0)),
         (nu.window(heads=3, dim=12, vdim=4, kv_rank=6, size=5, scale=0.5), None),
         (nu.delta(heads=3, kv_heads=3, dim=20, vdim=6, conv=2), nu.dense(33)),
         (nu.latent(heads=2, dim=10, rot_dim=4, vdim=12, kv_rank=7, q_rank=16, base=1000.0), nu.moe(experts=6, identity=6, top=5, groups=(4, 3), limit=0.3))]
LOOP = (1, 4, 2)


# ------------------------------------------------------------------ each mechanism alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name,layers,kw", [
    ("latent-attention", [(nu.latent(scale=0.9), None)], {}),
    ("latent-attention-one-head", [(nu.latent(heads=1, dim=3, rot_dim=2, vdim=13, kv_rank=3, q_rank=1), None)], {}),
    ("latent-attention-loud-sinks", [(nu.latent(), None)], {"edit": lambda sd: sd["l0.mix.sink"].add_(3.0)}),
    ("latent-attention-silent-sinks", [(nu.latent(), None)], {"edit": lambda sd: sd["l0.mix.sink"].sub_(60.0)}),
    ("latent-attention-wide", [(nu.latent(heads=2, dim=70, rot_dim=34, vdim=130, kv_rank=150, q_rank=90, scale=0.05), None)], {"std": 0.15}),
    ("window", [(nu.window(scale=1.1), None)], {}),
    ("window-of-one", [(nu.window(size=1), None)], {}),
    ("window-longer-than-the-sequence", [(nu.window(size=500), None)], {}),
    ("window-of-a-page", [(nu.window(size=16), None)], {}),
    ("window-wide", [(nu.window(heads=2, dim=130, vdim=70, kv_rank=200, size=20, scale=0.05), None)], {"std": 0.15}),
    ("delta", [(nu.delta(), None)], {}),
    ("delta-one-value-head-per-key-head", [(nu.delta(heads=2, kv_heads=2, dim=16, vdim=24), None)], {}),
    ("delta-four-value-heads-per-key-head", [(nu.delta(heads=4, kv_heads=1, dim=5, vdim=3), None)], {}),
    ("delta-of-single-numbers", [(nu.delta(heads=3, kv_heads=3, dim=1, vdim=1, conv=1), None)], {}),
    ("delta-wide", [(nu.delta(heads=2, kv_heads=1, dim=70, vdim=150, conv=9), None)], {"ranks": (13, 1)}),
    ("delta-more-than-one-register-tile", [(nu.delta(heads=1, kv_heads=1, dim=140, vdim=36), None)], {"ranks": (1, 8)}),
    ("delta-strong-decays", [(nu.delta(), None)], {"edit": lambda sd: (sd["l0.mix.A_log"].add_(3.0), sd["l0.mix.dt_bias"].add_(2.0))}),
    ("dense", [(nu.window(), nu.dense(ff=41))], {}),
    ("experts", [(nu.window(), nu.moe())], {}),
    ("experts-closed-groups-and-negative-scores", [(nu.window(), nu.moe(experts=10, identity=2, top=2, groups=(4, 1)))],
     {"edit": lambda sd: sd["l0.mlp.correction"].sub_(1.5)}),
    ("experts-groups-of-one", [(nu.window(), nu.moe(experts=5, identity=2, top=2, groups=(7, 3)))], {}),
    ("experts-all-groups-all-chosen", [(nu.window(), nu.moe(experts=3, identity=1, top=4, groups=(2, 2), scale=1.0))], {}),
    ("experts-without-groups", [(nu.window(), nu.moe(groups=None))], {}),
    ("experts-without-identities", [(nu.window(), nu.moe(experts=6, identity=0, groups=(2, 1)))], {}),
    ("mostly-identities", [(nu.window(), nu.moe(experts=1, identity=8, top=3, groups=(3, 2)))], {}),
    ("experts-top-1", [(nu.window(), nu.moe(top=1))], {}),
    ("experts-never-clamped", [(nu.window(), nu.moe(limit=1e4))], {}),
    ("experts-always-clamped", [(nu.window(), nu.moe(limit=0.01))], {}),
    ("many-experts", [(nu.window(), nu.moe(experts=130, identity=20, top=8, ff=3, groups=(10, 4)))], {}),
    ("loop-of-one-layer", [(nu.window(), nu.dense()), (nu.delta(), None), (nu.latent(), None)], {"loop": (1, 2, 4)}),
    ("loop-over-all", [(nu.latent(), nu.dense()), (nu.delta(), nu.moe())], {"loop": (0, 2, 3)}),
    ("loop-once", [(nu.latent(), nu.dense()), (nu.delta(), nu.moe())], {"loop": (0, 1, 1)}),
    ("empty-loop", [(nu.latent(), nu.dense()), (nu.delta(), nu.moe())], {"loop": (1, 1, 3)}),
    ("unit-logit-scale-odd-width", [(nu.latent(), nu.moe()), (nu.delta(), nu.dense())], {"logit_scale": 1.0, "width": 35, "loop": (0, 1, 2)}),
    ("width-of-one", [(nu.delta(), nu.moe()), (nu.window(), nu.dense())], {"width": 1, "std": 1.0}),
    ("one-bigram-bucket", [(nu.window(), None)], {"bigram": {"buckets": 1, "mul_prev": 5, "mul_cur": 9}}),
    ("bigram-of-large-multipliers", [(nu.window(), None)], {"bigram": {"buckets": 997, "mul_prev": 1000003, "mul_cur": 999983}}),
    ("bigram-blind-to-the-token-itself", [(nu.window(), None)], {"bigram": {"buckets": 50, "mul_prev": 1, "mul_cur": 0}}),
])
def test_mechanism_alone(tmp_path, device, name, layers, kw):
    cfg, sd, runner, _ = build(tmp_path, layers, seed=3, device=device, **kw)
    toks = nu.tokens(45, cfg["vocab"], 1)
    want = nu.oracle_logits(cfg, sd, toks)
    assert nu.rel_err(run_cut(runner, "a", toks, [len(toks)]), want) < TOL
    assert nu.rel_err(run_cut(runner, "b", toks, [30, 2]), want) < TOL
    assert nu.rel_err(run_cut(runner, "c", toks, [3, 20]), want) < TOL
    runner.close()


def test_oracle_parts_agree_with_their_definitions():
    """The oracle's own pieces on hand-made inputs: the pair layout, what a window sees, the sink in the denominator, the
    bigram rows, the convolution, one write and read of the delta rule, the clamps of an expert, routing, the layer order."""
    x = torch.tensor([[0.0, 0.0, 5.0, 6.0, 7.0], [1.0, 0.0, 0.0, 2.0, 7.0]], dtype=F)
    r = oracle.rotate(x, 4, 100.0)                                      # pairs (0, 2) and (1, 3); f = 1, 0.1
    assert torch.allclose(r[1], torch.tensor([math.cos(1.0), -2 * math.sin(0.1), math.sin(1.0), 2 * math.cos(0.1), 7.0], dtype=F))
    assert torch.equal(r[0], x[0])
    assert [j for j in range(9) if oracle.sees(6, j, 3)] == [4, 5, 6] and [j for j in range(9) if oracle.sees(2, j)] == [0, 1, 2]
    v = torch.arange(1.0, 5.0, dtype=F)[:, None]
    z = torch.zeros(4, 2, dtype=F)
    assert oracle.softmax_attention(z, z, v, 1.0, size=2).flatten().tolist() == [1.0, 1.5, 2.5, 3.5]
    o = oracle.softmax_attention(z, z, v, 7.0, sink=torch.tensor(math.log(2.0), dtype=F))       # (the sink is not scaled)
    assert torch.allclose(o.flatten(), torch.tensor([1 / 3, 3 / 4, 6 / 5, 10 / 6], dtype=F))
    b = {"buckets": 10, "mul_prev": 7, "mul_cur": 3}
    assert oracle.bigram_row(None, 5, b) == 10 and oracle.bigram_row(4, 5, b) == 3 and oracle.bigram_row(0, 0, b) == 0
    u = torch.tensor([[1.0], [10.0], [100.0]], dtype=F)
    assert oracle.short_conv(u, torch.tensor([[3.0, 2.0]], dtype=F)).flatten().tolist() == [2.0, 23.0, 230.0]
    # S = [[1, 2], [3, 4]], rows decay by 1/2 and 1/4; k = e0, v = (5, 5), beta = 1/2: row 0 moves halfway to v
    S, o = oracle.delta_step(torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=F), torch.tensor([1.0, 1.0], dtype=F), torch.tensor([1.0, 0.0], dtype=F),
                             torch.tensor([5.0, 5.0], dtype=F), torch.tensor([0.5, 0.25], dtype=F), 0.5)
    assert torch.equal(S, torch.tensor([[2.75, 3.0], [0.75, 1.0]], dtype=F)) and o.tolist() == [3.5, 4.0]
    sd = {"gate": torch.tensor([[3.0]], dtype=F), "up": torch.tensor([[-9.0]], dtype=F), "down": torch.tensor([[1.0]], dtype=F)}
    y = oracle.expert(sd, "", torch.ones(1, 1, dtype=F), 2.0)
    assert abs(float(y) + 2.0 / (1 + math.exp(-3.404))) < 1e-12         # g = 2, u = -2
    assert abs(float(oracle.expert(dict(sd, gate=-sd["gate"] * 3), "", torch.ones(1, 1, dtype=F), 2.0)) - 9.0 / (1 + math.exp(1.702 * 9))) < 1e-12
    # all choice scores negative: the group of the best one stays open, the others are closed however close they come
    zz, corr = torch.zeros(6, dtype=F), torch.tensor([-2.0, -0.9, -0.8, -0.85, -3.0, -0.82], dtype=F)
    r = {"experts": 5, "identity": 1, "top": 2, "scale": 3.0, "groups": {"count": 3, "keep": 1}}
    assert [e for e, _ in oracle.route(zz, corr, r)] == [2, 3] and all(abs(w - 1.5) < 1e-12 for _, w in oracle.route(zz, corr, r))
    assert [e for e, _ in oracle.route(zz, corr, dict(r, groups=None))] == [2, 5]
    assert oracle.schedule({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == \
        [(0, False), (1, False), (2, False), (1, True), (2, False), (3, False)]
    assert oracle.schedule({"layers": [0] * 2}) == [(0, False), (1, False)]


def test_planted_mistakes_show(tmp_path):
    """The comparison sees what it is meant to see: each of these mistakes, made in the oracle, moves some row by many
    times the tolerance."""
    cfg = nu.config(STACK, loop=LOOP)
    sd = nu.random_weights(cfg, 5)
    toks = nu.tokens(40, cfg["vocab"], 2)
    want = nu.oracle_logits(cfg, sd, toks)

    def differs(c=None, s=None):
        return nu.rel_err(nu.oracle_logits(c or cfg, s or sd, toks), want)

    def with_cfg(edit):
        c = json.loads(json.dumps(cfg))
        edit(c)
        return c

    def with_sd(**kw):
        return dict(sd, **kw)

    assert differs(with_cfg(lambda c: c["layers"][0]["mixer"]["mask"].update(size=13))) > 20 * TOL
    assert differs(with_cfg(lambda c: c["layers"][3]["mixer"]["mask"].update(size=4))) > 20 * TOL
    assert differs(with_cfg(lambda c: c["loop"].update(times=1))) > 20 * TOL
    assert differs(with_cfg(lambda c: c["embedding"]["bigram"].update(mul_prev=12))) > 20 * TOL
    assert differs(with_cfg(lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=3))) > 20 * TOL
    assert differs(with_cfg(lambda c: c["layers"][1]["mlp"]["expert"].update(limit=1e9))) > 20 * TOL
    assert differs(s=with_sd(**{"l1.mix.sink": sd["l1.mix.sink"] - 90})) > 20 * TOL
    assert differs(s=with_sd(**{"l2.mlp.correction": torch.zeros_like(sd["l2.mlp.correction"])})) > 20 * TOL
    assert differs(s=with_sd(**{"l2.mix.A_log": sd["l2.mix.A_log"] - 90})) > 20 * TOL
    assert differs(s=with_sd(**{"bigram": torch.cat([sd["bigram"][:-1], sd["bigram"][:1]])})) > 20 * TOL


# ----------------------------------------------- prompts, portions, decoding, first tokens
@pytest.mark.parametrize("device", DEVICES)
def test_prefill_portions_and_decode(tmp_path, device):
    """The same sequence whole, token by token, and in portions of 2, 3, 7, 16 and 17 tokens: windows, convolution inputs,
    recurrent states of all passes and the previous token cross the cuts."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=5, device=device, loop=LOOP)
    toks = nu.tokens(50, cfg["vocab"], 2)
    want = nu.oracle_logits(cfg, sd, toks)
    for cuts in ([50], [], [2, 2, 3, 7, 16, 17], [17, 16, 2], [2] * 25, [1, 2, 40]):
        assert nu.rel_err(run_cut(runner, "r", toks, cuts), want) < TOL, cuts
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_residual_rows_after_every_layer_run(tmp_path, device):
    """What leaves every layer run (a looped layer counts each time) against the oracle, through the layer functions on the
    runner's own weights and cache; the embedding rows beside them stay as they were."""
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
    x0 = oracle.embed(nu.f64(sd), cfg, toks)
    for name in runner.names:
        state = runner.family.run_layer(runner.ctx, name, W[name], state, batch, meta)
        if name[0] == "l":
            got = state.cpu().double()
            assert (got[:, :36] - trace[n]).abs().max() < 1e-4 * trace[n].abs().max(), name
            assert (got[:, 36:] - x0).abs().max() < 1e-5
            n += 1
    assert n == len(trace) == 9
    runner.seq_cache.release("t")
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_over_pages(tmp_path, device):
    """A short prompt, then 150 decoded tokens over many pages, beside a stack of windows alone whose pages go back."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=6, device=device, loop=LOOP)
    toks = nu.tokens(155, cfg["vocab"], 7)
    assert nu.rel_err(run_cut(runner, "r", toks, [5], end=False), nu.oracle_logits(cfg, sd, toks)) < TOL
    assert runner.seq_cache.pages_trimmed == 0                     # (a latent attention without a window reads every key)
    runner.close()
    cfg, sd, runner, _ = build(tmp_path, [(nu.window(size=20), nu.moe()), (nu.delta(), nu.dense()), (nu.window(size=7), None)], seed=7,
                               device=device, loop=(0, 2, 2))
    assert nu.rel_err(run_cut(runner, "r", toks, [5], end=False), nu.oracle_logits(cfg, sd, toks)) < TOL
    # window 20: the next token (155) still reads 136 ..; pages 0 .. 7 are back in the pool
    cache, r = runner.seq_cache, runner.seq_cache.requests["r"]
    assert cache.pages_trimmed == 8 and [p >= 0 for p in r.pages] == [False] * 8 + [True] * 2
    cache.release("r")
    assert len(cache.free_pages) == cache.n_pages
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
    """Requests of 1, 9, 33 and 50 tokens in one step, then decoded together while the short ones finish first; also cut
    into two micro-batches by a small token budget."""
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
    """One step that starts a request, continues another by a portion, and decodes a third: each equals itself alone."""
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
def test_pages_and_slots_used_again(tmp_path, device):
    """Requests come and go through pools of two slots and a few pages: whoever inherits a page or a slot (with the last
    owner's rows, states and last token still in it) computes what it computes alone, and pools that run out grow without
    disturbing the live request."""
    cfg, sd, runner, _ = build(tmp_path, STACK, seed=11, device=device, max_tokens=40, max_seqs=2, loop=LOOP)
    cache = runner.seq_cache
    a, b, c = (nu.tokens(n, cfg["vocab"], 40 + n) for n in (37, 22, 130))
    wa, wb, wc = (nu.oracle_logits(cfg, sd, s) for s in (a, b, c))
    assert nu.rel_err(run_cut(runner, "a", a, [30]), wa) < TOL
    ga = run_cut(runner, "a", a, [10, 2], end=False)                        # the same name again: its last token is forgotten
    gb = run_cut(runner, "b", b, [22])                                      # inherits a's first slot
    assert cache.slots_reused > 0 and cache.pages_reused > 0
    gc = run_cut(runner, "c", c, [3, 120])
    n0 = cache.n_slots
    others = [run_cut(runner, f"x{i}", b, [5], end=False) for i in range(3)]    # more requests than slots
    assert cache.n_slots > n0
    tail = runner.step([StepEntry("a", [a[0]], [0])], ["a"])[0][0]           # its state survived the growth
    assert nu.rel_err(tail, nu.oracle_logits(cfg, sd, a + [a[0]])[-1:]) < TOL
    for g, w in ((ga, wa), (gb, wb), (gc, wc)) + tuple((o, wb) for o in others):
        assert nu.rel_err(g, w) < TOL
    runner.close()


# ------------------------------------------- one token that stands out: far back, at page borders, at a window's edges
def _marked_model(tmp_path, kind, size=11, **sizes):
    """One layer whose weights make one marked token decide every row that sees it.  Channel 0 of the embedding is the same
    for every token, channel 1 is zero except for the marked token, where it is large; bigrams add nothing.  ``latent`` and
    ``window``: the latent's first entry is negative for plain tokens and positive for the marked one, W_uk turns it into -u and
    +u, every query is u: the marked score stands out however many keys there are.  ``delta``: the state forgets next to
    nothing; plain tokens write along key channel 0, the marked one along channel 1, and every query asks for channel 1."""
    D, vocab, mark = 24, 40, 7
    make, small = {"latent": (nu.latent, dict(heads=2, dim=8, rot_dim=4, vdim=6, kv_rank=5, q_rank=4, base=1e6, scale=0.4)),
                   "window": (nu.window, dict(heads=2, dim=8, vdim=6, kv_rank=5, size=size, scale=0.4)),
                   "delta": (nu.delta, dict(heads=2, kv_heads=1, dim=6, vdim=5, conv=3))}[kind]
    mixer = make(**{**small, **sizes})
    cfg = nu.config([(mixer, None)], width=D, vocab=vocab, logit_scale=1.0)
    sd = {k: v.float() for k, v in nu.random_weights(cfg, 12, std=0.05).items()}
    sd["embed"] *= 0.05
    sd["bigram"][:] = 0.0
    sd["embed"][:, 0] = 4.0
    sd["embed"][:, 1] = 0.0
    sd["embed"][mark, 1] = 12.0
    sd["l0.norm1"][:] = 1.0
    x, m = "l0.mix.", mixer[1]
    if kind == "delta":
        d = m["dim"]
        for n in ("q", "k", "v"):
            sd[x + n] *= 0.0
            sd[x + n + ".conv"][:] = 0.05
            sd[x + n + ".conv"][:, -1] = 1.0
        sd[x + "A_log"][:] = -9.0
        sd[x + "q"][1, 0] = 1.0
        sd[x + "k"][0, 0], sd[x + "k"][1, 1], sd[x + "k"][0, 1] = 1.0, 1.0, -1.0
        sd[x + "v"][::2, 1] = 1.5
        sd[x + "v"][:, 0] = 0.2
        assert d >= 2
    else:
        H, d, dr, dv, r = m["heads"], m["dim"], m.get("rot_dim", 0), m["vdim"], m["kv_rank"]
        u = torch.tensor([(-1.0) ** (i // 2) for i in range(d)]) * math.sqrt(8.0 / d)
        sd[x + "dkv"][0, 0], sd[x + "dkv"][0, 1] = -1.0, 1.0
        sd[x + "dkv.norm"][:] = 1.0
        sd[x + "uk"][:, 0] = u.repeat(H) / math.sqrt(r)
        sd[x + "dkv"][1, 0], sd[x + "dkv"][1, 1] = 0.0, 0.3                 # the latent's second entry: the marked token's value
        sd[x + "uv"][:, 1] = 8.0 / (H * math.sqrt(r))
        if kind == "latent":
            sd[x + "dq.norm"][:] = 1.0
            sd[x + "dq"][0, 0] = 1.0
            for hh in range(H):
                sd[x + "uq"][hh * (d + dr):hh * (d + dr) + d, 0] = u / math.sqrt(m["q_rank"])
        else:
            sd[x + "q"][:, 0] = u.repeat(H) / math.sqrt(D)
    sd = {k: v.to(torch.bfloat16) for k, v in sd.items()}
    return cfg, sd, nu.write_model(str(tmp_path / f"mark_{kind}_{size}"), cfg, sd), mark, vocab


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["latent", "delta"])
def test_one_token_stands_out_far_back_and_at_page_borders(tmp_path, device, kind):
    """The marked token at the start, on both sides of page borders and hundreds of places (many pages) back: every later
    row still depends on it, no earlier one does; seen from prompt rows, from decoded rows, and from the first row after a
    cut right behind the mark."""
    cfg, sd, path, mark, vocab = _marked_model(tmp_path, kind)
    runner = load_runner(path, torch.float32, device, max_tokens=640, max_seqs=2)
    rng = np.random.default_rng(0)
    n = 260
    for place in (0, 15, 16, 143, n - 2):
        toks = [int(t) for t in rng.integers(8, vocab, n)]
        toks[place] = mark
        want = nu.oracle_logits(cfg, sd, toks)
        plain = nu.oracle_logits(cfg, sd, [t if t != mark else 9 for t in toks])
        seen = np.array([nu.rel_err(plain[i:i + 1], want[i:i + 1]) for i in range(n)])      # (per row, relative to the row's spread)
        assert seen[:place].max(initial=0.0) == 0.0
        assert seen[place + 1:].min() > 50 * TOL, "the marked token does not stand out"
        assert nu.rel_err(run_cut(runner, "p", toks, [n])[-60:], want[-60:]) < TOL, place
        cuts = [place + 1] + ([n - 30 - place - 1] if n - 30 - place - 1 > 0 else [])
        tail = min(60, n - place - 1)
        assert nu.rel_err(run_cut(runner, "d", toks, cuts)[-tail:], want[-tail:]) < TOL, place
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size", [1, 2, 11, 16, 40])
def test_one_token_stands_out_at_a_windows_edges(tmp_path, device, size):
    """Rows up to ``size`` - 1 behind the marked token see it, later and earlier ones do not: in prompts, in portions cut
    where it leaves the window, and in decoding."""
    cfg, sd, path, mark, vocab = _marked_model(tmp_path, "window", size)
    runner = load_runner(path, torch.float32, device, max_tokens=128, max_seqs=2)
    n = 72
    base = [int(t) for t in np.random.default_rng(0).integers(8, vocab, n)]
    plain = nu.oracle_logits(cfg, sd, base)
    for place in (0, 15, 16, 31):
        toks = list(base)
        toks[place] = mark
        want = nu.oracle_logits(cfg, sd, toks)
        diff = np.array([nu.rel_err(plain[i:i + 1], want[i:i + 1]) for i in range(n)])
        for i in range(n):
            assert (diff[i] > 100 * TOL) if place <= i < place + size else (diff[i] == 0.0), (place, i, diff[i])
        assert nu.rel_err(run_cut(runner, "p", toks, [n]), want) < TOL, place
        cuts, at = [], 0
        for edge in sorted({place + 1, place + size, place + size + 1}):
            if at < edge < n:
                cuts.append(edge - at)
                at = edge
        assert nu.rel_err(run_cut(runner, "e", toks, cuts + [n - at]), want) < TOL, place
        assert nu.rel_err(run_cut(runner, "d", toks, [max(1, place - 1)]), want) < TOL, place
    runner.close()


# ----------------------------------------------------- shards, bf16, generation
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("lnps", [1, 3])
def test_few_layers_per_shard_stream_weights(tmp_path, device, lnps):
    """Weights streamed shard by shard: the passes of a looped layer land in different shards or in one; the embedding rows
    travel with the residual rows."""
    cfg = nu.config(STACK, loop=LOOP)
    sd = nu.random_weights(cfg, 13)
    path = nu.write_model(str(tmp_path / "s"), cfg, sd)
    runner = load_runner(path, torch.float32, device, max_tokens=64, layer_num_per_shard=lnps, resident=False)
    toks = nu.tokens(40, cfg["vocab"], 3)
    assert nu.rel_err(run_cut(runner, "r", toks, [20, 2]), nu.oracle_logits(cfg, sd, toks)) < TOL
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_bf16_products_stay_close(tmp_path, device):
    """(Every expert is chosen, so that rounding cannot flip a choice.)"""
    f = nu.moe(experts=3, identity=1, top=4, groups=(2, 2))
    cfg, sd, runner, _ = build(tmp_path, [(m, f if p and p["kind"] == "moe" else p) for m, p in STACK], seed=14, device=device,
                               dtype=torch.bfloat16, loop=LOOP)
    toks = nu.tokens(60, cfg["vocab"], 4)
    want = nu.oracle_logits(cfg, sd, toks)
    whole, cut = run_cut(runner, "a", toks, [60]), run_cut(runner, "b", toks, [9, 2, 20])
    for got, ref in ((whole, want), (cut, want), (cut, whole)):
        e = nu.row_errs(got, ref)
        assert e.max() < 0.2 and e.mean() < 0.05, (e.max(), e.mean())
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind,sizes", [
    ("latent", dict(heads=3, dim=64, rot_dim=64, vdim=128, kv_rank=512, q_rank=40)),
    ("latent", dict(heads=2, dim=48, rot_dim=16, vdim=64, kv_rank=128, q_rank=24)),
    ("latent", dict(heads=5, dim=96, rot_dim=64, vdim=40, kv_rank=256, q_rank=24)),
    ("window", dict(heads=3, dim=128, vdim=128, kv_rank=512, size=60)),
    ("window", dict(heads=4, dim=64, vdim=64, kv_rank=256, size=33)),
    ("window", dict(heads=34, dim=24, vdim=16, kv_rank=128, size=128)),
    ("delta", dict(heads=3, kv_heads=1, dim=128, vdim=128)),
    ("delta", dict(heads=2, kv_heads=2, dim=64, vdim=192)),
])
def test_sizes_of_the_tiled_kernels(tmp_path, device, kind, sizes):
    """bf16 with head and latent sizes that the matrix-core kernels and the register tiles serve on the GPU, and some they do
    not: a prompt of several row tiles, a portion that continues it, then decoding; a marked token far back must not drown in
    the rounding."""
    cfg, sd, path, mark, vocab = _marked_model(tmp_path, kind, **sizes)
    runner = load_runner(path, torch.bfloat16, device, max_tokens=512)
    toks = [int(t) for t in np.random.default_rng(5).integers(8, vocab, 200)]
    toks[21] = toks[140] = mark
    want = nu.oracle_logits(cfg, sd, toks)
    whole = run_cut(runner, "a", toks, [200])
    cut = run_cut(runner, "b", toks, [110, 60])
    for got, ref in ((whole, want), (cut, want), (cut, whole)):
        e = nu.row_errs(got, ref)
        assert e.max() < 0.08 and e.mean() < 0.03, (e.max(), e.mean())
    runner.close()


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(tmp_path, device):
    """serve.generate: prompts of unequal length, 12 new tokens each; the tokens are the oracle's greedy continuation."""
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
    """The registry picks the family by config.json's architecture; ranks that config.json leaves open come from the
    checkpoint; every pass of a looped layer has a state of its own and shares its layer's weight image; every tensor of
    the checkpoint lands, none is invented; a config outside the kernels' bounds or one that contradicts the checkpoint is
    refused."""
    from flexible_llm_sharding_amd.config import NumolornConfig, load_config
    from flexible_llm_sharding_amd.models import hybrid_family, numolorn
    from flexible_llm_sharding_amd.runtime.weights import CheckpointSource, HostStore
    cfg = nu.config(STACK, loop=LOOP)
    sd = nu.random_weights(cfg, 18, ranks=(6, 4))
    path = nu.write_model(str(tmp_path / "c"), cfg, sd)
    c = load_config(path)
    assert isinstance(c, NumolornConfig) and hybrid_family(c) is numolorn
    assert c.layer_names() == ["embed", "l0", "l1", "l2", "l3", "l1@1", "l2@1", "l3@1", "l4", "l5", "final.norm", "head"]
    assert c.state_width == 2 * 36 and [n for n in c.layer_names()[1:-2] if c.reenters(n)] == ["l1@1"]
    assert (c.layer("l2@1").mixer["decay_rank"], c.layer("l4").mixer["gate_rank"]) == (6, 4)
    spec = numolorn.state_spec(c)
    assert spec["prev_token"] and set(spec["paged"]) == {"l0", "l1", "l3", "l1@1", "l3@1", "l5"}
    assert spec["paged"]["l1@1"] == {"ckr": 11 + 8} and spec["paged"]["l0"] == {"ckr": 10}
    assert spec["slots"]["l2@1"] == {"conv": (3, 2 * 14 + 36), "state": (4, 9, 7)}
    names = {pl.hf_name for n in c.layer_names() for pl in numolorn.placements(c, n)}
    assert names == set(sd)
    assert json.loads(json.dumps(NumolornConfig.from_dict(c.to_dict()).to_dict())) == c.to_dict()
    store = HostStore.from_source(CheckpointSource(c, path, torch.float32), pinned=False)
    assert store.host_buffer("l2@1") is store.host_buffer("l2") and store.host_buffer("l4") is not store.host_buffer("l2")
    flat = json.loads(json.dumps(c.to_dict()))
    del flat["loop"]
    assert NumolornConfig.from_dict(flat).state_width == 36
    for edit in (lambda d: d["layers"][0].update(type="attention"),
                 lambda d: d["layers"][2]["mixer"].update(kv_heads=3),
                 lambda d: d["layers"][2]["mixer"].update(conv=0),
                 lambda d: d["layers"][2]["mixer"].update(dim=257),
                 lambda d: d["layers"][2]["mixer"].update(vdim=513),
                 lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7),
                 lambda d: d["layers"][1]["mixer"]["rot"].update(dims=10),
                 lambda d: d["layers"][1]["mixer"].update(kv_rank=513),
                 lambda d: d["layers"][0]["mixer"]["mask"].update(size=0),
                 lambda d: d["layers"][0]["mlp"].update(kind="other"),
                 lambda d: d["layers"][1]["mlp"]["router"].update(top=17),
                 lambda d: d["layers"][1]["mlp"]["router"].update(top=7),
                 lambda d: d["layers"][1]["mlp"]["router"].update(groups={"count": 4, "keep": 2}),
                 lambda d: d["layers"][1]["mlp"]["router"].update(groups={"count": 3, "keep": 4}),
                 lambda d: d["embedding"]["bigram"].update(buckets=0),
                 lambda d: d.update(loop={"start": 2, "stop": 9, "times": 2}),
                 lambda d: d.update(loop={"start": 0, "stop": 2, "times": 0})):
        bad = json.loads(json.dumps(c.to_dict()))
        edit(bad)
        with pytest.raises((NotImplementedError, ValueError)):
            NumolornConfig.from_dict(bad)
    wrong = json.loads(json.dumps(cfg))
    wrong["layers"][0]["mixer"]["vdim"] = 15
    nu.write_model(str(tmp_path / "w"), wrong, sd)
    with pytest.raises(ValueError):
        load_runner(str(tmp_path / "w"), torch.float32, "cpu")


@pytest.mark.gpu
def test_captured_decode_steps_equal_eager(tmp_path, monkeypatch):
    """Decode steps replay as captured HIP graphs; every replay is checked against the same steps run eagerly, with eager
    prompt steps of other requests and batch-size changes between the replays."""
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
    """bin/trace_run as a process on a two-request schedule: prompts of unequal length in one step, then one token each; a
    flushed 'done <step>' after each step, logits files for the steps that want some, exit code 0 at end of input."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = nu.config(STACK[:4], vocab=37, loop=(1, 3, 2))
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
    """The benchmark's synthetic stack (bench.py --hybrid --hybrid-family numolorn) at a toy size: random layer images
    straight into a host store, a prompt step and a decode step through the runner; and the stack beside it."""
    from flexible_llm_sharding_amd.engine import ShardedRunner
    from flexible_llm_sharding_amd.utils.hybrid_bench import FAMILIES, numolorn_config, synthetic_hybrid_store
    z = dict(width=64, heads=4, kv=2, dim=16, ff=96, experts=4, top=2, eff=16, blocks=2, mh=2, mp=8, state=8, chunk=12, vocab=50)
    cfg = numolorn_config(z)
    assert cfg.num_hidden_layers == FAMILIES["numolorn"][1](z).num_hidden_layers == 6
    src = synthetic_hybrid_store(cfg, "cpu", torch.float32)
    r = ShardedRunner(cfg, src, device="cpu", layer_num_per_shard=2, storage_location="cpu", compute_dtype=torch.float32,
                      state_tokens=64, state_seqs=2)
    out = r.step([StepEntry("a", list(range(20)), [19]), StepEntry("b", [1, 2, 3], [2])])
    assert out[0][0].shape == (1, 50) and np.isfinite(out[0][0]).all() and np.isfinite(out[1][0]).all()
    out = r.step([StepEntry("a", [5], [0]), StepEntry("b", [6], [])], ["a", "b"])
    assert out[1] is None and np.isfinite(out[0][0]).all() and not r.seq_cache.requests
    r.close()
