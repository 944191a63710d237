"""Numolorn layer execution on packed weight images and packed step batches.

A layer runs its mixer and its feed-forward side by side, each on a norm of its own of the same row:

    x <- x + mixer(N1(x)) * ls1 + ff(N2(x)) * ls2        (ls: one number per channel; the last term only with an ff)

x is the fp32 residual row.  It starts as embed[token] + bigram[hash(previous token, token)], and ``loop`` runs some layers
several times on the same weights; every pass but the first adds that first row again, so where there is such a loop
the activation that passes from layer to layer is [x | x0] ([T, 2 D] fp32).  Every pass has pages and states of its
own (execution names ``l0``, ``l0@1``, ...).  Mixers:

* ``latent_attention`` -- softmax attention whose keys and values are linear maps of one cached latent row c_j
  (RMS-normed) plus a rotated key part shared by all heads (pairs (i, i + dims / 2)); the queries come through a latent
  too.  A learned number per head joins the softmax's denominator, and head h's output is multiplied by
  sigmoid(W_g h)_h;
* ``latent_attention_2`` -- the same kind of cache without positions: plain queries, a sliding window, an ordinary softmax;
* ``channel_delta`` -- a gated delta rule.  q, k and v pass a short causal convolution and SiLU; per head a state S
  [key, value] decays per key channel, S <- diag(g) S, moves what it holds for the unit key k towards v,
  u = beta (v - S^T k), S <- S + k u^T, and is read after the write, o = S^T q; o is RMS-normed per head and gated.

Steps that continue a sequence fold a latent attention's maps around it (the query side becomes W_uk,h^T q_h, the
attention runs with one key/value head over the latent rows, W_uv,h maps each head's weighted latent); whole prompts
make per-head keys and values from the step's rows where the matrix-core attention serves their sizes.

Feed-forwards: W_down(silu(W_gate h) * W_up h), or a mixture of clamped experts, chosen among the best groups of router
outputs by softmax score plus a correction and weighted by the bare scores; the last router outputs are identity
experts, whose output is the input itself.  Each mechanism is an op of the backend (``ops/hip_seq.py``: the kernels of
``csrc/kernels/seq``; ``ops/torch_seq.py`` on the CPU) with its constants as arguments; this file only strings them
together.  Latent rows, recurrent states and each request's last token live in
:class:`~..runtime.seq_state.SequenceStateCache`.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from .kagolix import HybridContext  # noqa: F401  (the context the engine builds for every hybrid family)
from .layout import LayerLayout, Placement, layer_image, layer_kind, spec_layout, spec_placements
from .lopilix import NO_WINDOW

F32 = "f32"
UNIT_EPS = 1e-6                    # q, k / sqrt(sum(x^2) + UNIT_EPS)
EXPERT_ALPHA = 1.702               # an expert's gate: g sigmoid(EXPERT_ALPHA g)


def _latent_sizes(L):
    """(heads, dim, rot_dim, vdim, kv_rank, q_rank) of a latent attention (rot_dim, q_rank 0: it has no such part)."""
    m = L.mixer
    full = L.type == "latent_attention"
    return (int(m["heads"]), int(m["dim"]), int(m["rot_dim"]) if full else 0, int(m["vdim"]), int(m["kv_rank"]),
            int(m["q_rank"]) if full else 0)


def _cols(L) -> Dict[str, tuple]:
    """Column ranges (start, width) of a mixer's stacked input projection."""
    m = L.mixer
    if L.type == "latent_attention":
        H, _, dr, _, r, qr = _latent_sizes(L)
        widths = [("dq", qr), ("dkv", r + dr), ("g", H)]
    elif L.type == "latent_attention_2":
        H, d, _, _, r, _ = _latent_sizes(L)
        widths = [("dkv", r), ("q", H * d)]
    else:
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        widths = [("qkv", 2 * G * d + H * dv), ("a1", m["decay_rank"]), ("g1", m["gate_rank"]), ("b", H)]
    out, at = {}, 0
    for n, w in widths:
        out[n] = (at, int(w))
        at += int(w)
    out["all"] = (0, at)
    return out


def _specs(cfg, name: str):
    """[(slot, shape, dtype tag, [(checkpoint tensor, element offset in the slot, shape[, options])])]."""
    D, V = cfg.width, cfg.vocab
    kind = layer_kind(name)
    if kind == "embed":
        out = [("embed", (V, D), None, [("embed", 0, (V, D))])]
        if cfg.bigram is not None:
            n = int(cfg.bigram["buckets"]) + 1                 # (the last row: nothing comes before)
            out.append(("bigram", (n, D), None, [("bigram", 0, (n, D))]))
        return out
    if kind == "head":
        return [("head", (V, D), None, [("embed", 0, (V, D))])]        # the logits come from the embedding table
    if kind == "norm":
        return [("norm", (D,), F32, [("final.norm", 0, (D,))])]
    name = layer_image(name)
    L, p, x = cfg.layer(name), name + ".", name + ".mix."
    m, c = L.mixer, _cols(L)
    n_in = c["all"][1]
    row = lambda n: c[n][0] * D
    out = [("norm1", (D,), F32, [(p + "norm1", 0, (D,))]), ("ls1", (D,), F32, [(p + "ls1", 0, (D,))])]
    if L.type == "channel_delta":
        H, G, d, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
        ra, rg, qk = c["a1"][1], c["g1"][1], G * d
        out += [("win", (n_in, D), None,
                 [(x + "q", 0, (qk, D)), (x + "k", qk * D, (qk, D)), (x + "v", 2 * qk * D, (H * dv, D)),
                  (x + "a1", row("a1"), (ra, D)), (x + "g1", row("g1"), (rg, D)), (x + "b", row("b"), (H, D))]),
                ("conv", (c["qkv"][1], taps), F32,
                 [(x + "q.conv", 0, (qk, taps)), (x + "k.conv", qk * taps, (qk, taps)), (x + "v.conv", 2 * qk * taps, (H * dv, taps))]),
                ("wa2", (H * d, ra), None, [(x + "a2", 0, (H * d, ra))]), ("wg2", (H * dv, rg), None, [(x + "g2", 0, (H * dv, rg))]),
                ("dt_bias", (H * d,), F32, [(x + "dt_bias", 0, (H * d,))]), ("A_log", (H,), F32, [(x + "A_log", 0, (H,))]),
                ("mnorm", (dv,), F32, [(x + "norm", 0, (dv,))]), ("wo", (D, H * dv), None, [(x + "o", 0, (D, H * dv))])]
    else:
        H, d, dr, dv, r, qr = _latent_sizes(L)
        if L.type == "latent_attention":
            out += [("win", (n_in, D), None, [(x + "dq", 0, (qr, D)), (x + "dkv", row("dkv"), (r + dr, D)), (x + "g", row("g"), (H, D))]),
                    ("dqn", (qr,), F32, [(x + "dq.norm", 0, (qr,))]),
                    ("wuq", (H * (d + dr), qr), None, [(x + "uq", 0, (H * (d + dr), qr))]),
                    ("sink", (H,), F32, [(x + "sink", 0, (H,))])]
        else:
            out.append(("win", (n_in, D), None, [(x + "dkv", 0, (r, D)), (x + "q", row("q"), (H * d, D))]))
        out += [("dkvn", (r,), F32, [(x + "dkv.norm", 0, (r,))]),
                # W_uk per head, transposed: the product that folds it into the queries reads it as [N = r, K = d]
                ("wukt", (H, r, d), None, [(x + "uk", 0, (H * d, r), {"view": (H, d, r), "perm": (0, 2, 1)})]),
                ("wuk", (H, d, r), None, [(x + "uk", 0, (H * d, r))]),
                ("wuv", (H, dv, r), None, [(x + "uv", 0, (H * dv, r))]),
                ("wo", (D, H * dv), None, [(x + "o", 0, (D, H * dv))])]
    if L.mlp is not None:
        y = p + "mlp."
        out += [("norm2", (D,), F32, [(p + "norm2", 0, (D,))]), ("ls2", (D,), F32, [(p + "ls2", 0, (D,))])]
        if L.mlp["kind"] == "dense":
            ff = int(L.mlp["ff"])
            out += [("wgu", (2 * ff, D), None, [(y + "gate", 0, (ff, D)), (y + "up", ff * D, (ff, D))]),
                    ("wdown", (D, ff), None, [(y + "down", 0, (D, ff))])]
        else:
            E, ff = int(L.mlp["router"]["experts"]), int(L.mlp["expert"]["ff"])
            Z = E + int(L.mlp["router"].get("identity", 0))
            gu, dn = [], []
            for e in range(E):
                gu += [(f"{y}e{e}.gate", e * 2 * ff * D, (ff, D)), (f"{y}e{e}.up", (e * 2 + 1) * ff * D, (ff, D))]
                dn.append((f"{y}e{e}.down", e * D * ff, (D, ff)))
            out += [("wrouter", (Z, D), None, [(y + "router", 0, (Z, D))]), ("corr", (Z,), F32, [(y + "correction", 0, (Z,))]),
                    ("wgu", (E, 2 * ff, D), None, gu), ("wdown", (E, D, ff), None, dn)]
    return out


def layout(cfg, name: str, elem_size: int = 2) -> LayerLayout:
    return spec_layout(layer_kind(name), _specs(cfg, name), elem_size)


def placements(cfg, name: str, elem_size: int = 2) -> List[Placement]:
    return spec_placements(layout(cfg, name, elem_size), _specs(cfg, name), elem_size)


def _window(m: dict) -> int:
    return int(m["mask"]["size"]) if m.get("mask") is not None else 0


def state_spec(cfg) -> dict:
    """What a request keeps between steps, per pass of every layer: latent rows [c | rotated key part] of a latent
    attention and how far back it looks, the convolution's last inputs and the fp32 state ([vdim, dim] per head) of a
    delta rule; and its last token, which the next one's bigram row depends on."""
    paged, slots, horizons = {}, {}, []
    for name in cfg.layer_names():
        if layer_kind(name) != "decoder":
            continue
        L = cfg.layer(name)
        m = L.mixer
        if L.type == "channel_delta":
            slots[name] = {"conv": (m["conv"] - 1, _cols(L)["qkv"][1]), "state": (m["heads"], m["vdim"], m["dim"])}
        else:
            paged[name] = {"ckr": _latent_sizes(L)[4] + _latent_sizes(L)[2]}
            horizons.append(("window", _window(m) or NO_WINDOW, 0))
    return {"paged": paged, "alias": {}, "slots": slots, "horizons": horizons, "prev_token": cfg.bigram is not None}


# ------------------------------------------------------------------------------------ execution
def _latent_attention(ctx, L, W, h, meta, name: str):
    ops, eps, cdt, m = ctx.ops, ctx.cfg.norm_eps, ctx.compute_dtype, L.mixer
    H, d, dr, dv, r, qr = _latent_sizes(L)
    c = _cols(L)
    rot = (int(m["rot"]["dims"]), float(m["rot"]["base"])) if dr and int(m["rot"]["dims"]) > 1 else None
    pool = ctx.cache.pools(name)["ckr"]                                   # [pages, page, c | kr]
    rows = pool.view(-1, r + dr)
    z = ops.matmul_nt(h, W["win"])                                         # fp32 [T, c_q | c | kr | g] or [T, c | q]
    cq = ops.latent_rows(z, qr, r, dr, W.get("dqn"), W["dkvn"], eps, rot, rows, meta, cdt)
    q = ops.matmul_nt(cq, W["wuq"]) if qr else z[:, c["q"][0]:c["q"][0] + H * d]
    T = z.shape[0]
    how = dict(scale=float(m["scale"]), softcap=0.0, r1=None, r2=None, chunk=0, window=_window(m), sink=W.get("sink"), out_dtype=cdt,
               head_gate=z[:, c["g"][0]:c["g"][0] + H] if "g" in c else None)
    local = meta.get("local_table")
    if local is not None and ops.unfolded_attention_ok(d + dr, dv, cdt):
        # whole prompts (every request of the step starts at position 0, so all keys are this step's rows):
        # keys and values are made per head from the rows as cached, [W_uk,h c | kr] and W_uv,h c
        ckr = ops.gather_rows(rows, meta["kv_slot"])                      # [T, c | kr]
        kf = torch.empty(T, H * (d + dr), dtype=cdt, device=z.device)
        ops.head_matmul_nt(ckr, W["wuk"], H, 0, kf, d + dr)
        if dr:
            ops.head_norm_rope(ckr, H, dr, r, 0, kf, d, d + dr, meta)     # the one rotated part beside every head's keys
            ops.head_norm_rope(q, H, dr, d, d + dr, q, d, d + dr, meta, rot=rot, half=True)        # (in place)
        vf = ops.matmul_nt(ckr[:, :r], W["wuv"].view(H * dv, r), out_dtype=cdt)
        o = ops.attn_paged(q, kf.view(T, 1, -1), vf.view(T, 1, -1), dict(meta, page_table=local), H, H, d + dr, dv, page_size=1, **how)
        return ops.matmul_nt(o, W["wo"])
    # decoding, portions: the query each head asks the latent rows with is [W_uk,h^T q_unrotated | q_rotated]
    qa = torch.empty(T, H * (r + dr), dtype=torch.float32, device=z.device)
    ops.head_matmul_nt(q, W["wukt"], H, d + dr, qa, r + dr)
    if dr:
        ops.head_norm_rope(q, H, dr, d, d + dr, qa, r, r + dr, meta, rot=rot, half=True)
    a = ops.attn_paged(qa, pool, pool, meta, H, 1, r + dr, r, page_size=ctx.cache.page_size, **how)
    o = torch.empty(T, H * dv, dtype=cdt, device=z.device)
    ops.head_matmul_nt(a, W["wuv"], H, r, o, dv)                          # each head's weighted latent -> its values
    return ops.matmul_nt(o, W["wo"])


def _channel_delta(ctx, L, W, h, meta, name: str):
    ops, cdt, m = ctx.ops, ctx.compute_dtype, L.mixer
    c = _cols(L)
    st = ctx.cache.recurrent(name)
    z = ops.matmul_nt(h, W["win"])                                         # fp32 [T, q | k | v | a1 | g1 | b]
    col = lambda n: z[:, c[n][0]:c[n][0] + c[n][1]]
    qkv = ops.causal_conv(col("qkv"), W["conv"], None, st["conv"], meta, act="silu")
    decay = ops.matmul_nt(col("a1"), W["wa2"], bias=W["dt_bias"], decay=W["A_log"])      # the decays leave the product's epilogue
    gate = ops.matmul_nt(col("g1"), W["wg2"])
    # unit norms, step sizes, recurrence, output norm and gate
    o = ops.gated_delta_scan(qkv, col("b"), decay, gate, W["mnorm"], st["state"], meta, m["heads"], m["kv_heads"], m["dim"], m["vdim"],
                             unit_eps=UNIT_EPS, norm_eps=ctx.cfg.norm_eps, out_dtype=cdt)
    return ops.matmul_nt(o, W["wo"])


def _dense(ctx, mlp: dict, W, h):
    ops, cdt = ctx.ops, ctx.compute_dtype
    return ops.matmul_nt(ops.gate_mul(ops.matmul_nt(h, W["wgu"]), cdt, act="silu"), W["wdown"])


def _moe(ctx, mlp: dict, W, h):
    """-> (expert output rows, route, h, experts) for ``parallel_update_``, which sums them into the residual row."""
    ops, cdt = ctx.ops, ctx.compute_dtype
    r = mlp["router"]
    E, g = int(r["experts"]), r.get("groups") or {}
    logits = ops.matmul_nt(h, W["wrouter"])                                # fp32 accumulation of the rows
    route = ops.moe_route_softmax_grouped(logits, W["corr"], int(r["top"]), int(g.get("count", 0)), int(g.get("keep", 0)),
                                          float(r.get("scale", 1.0)))
    offs = route.offs[:E + 1]                                              # (rows of identity experts sort behind the experts')
    hp = ops.gather_rows(h, route.rows)
    gu = ops.grouped_matmul_nt(hp, W["wgu"], offs)                         # fp32 [T top, gate | up]
    act = ops.gate_mul(gu, cdt, act="clamped", limit=float(mlp["expert"]["limit"]), alpha=EXPERT_ALPHA)
    return ops.grouped_matmul_nt(act, W["wdown"], offs), route, h, E


_MIXERS = {"latent_attention": _latent_attention, "latent_attention_2": _latent_attention, "channel_delta": _channel_delta}


def run_block(ctx, W, xs: torch.Tensor, meta: dict, name: str) -> torch.Tensor:
    cfg, ops = ctx.cfg, ctx.ops
    L, D = cfg.layer(name), cfg.width
    x = xs[:, :D]
    # both norms of the row in one pass; a pass other than the first adds the embedding row on the way
    h1, h2 = ops.rmsnorm_pair(x, W["norm1"], W.get("norm2"), cfg.norm_eps, ctx.compute_dtype, add=xs[:, D:] if cfg.reenters(name) else None)
    y = _MIXERS[L.type](ctx, L, W, h1, meta, name)
    if L.mlp is None:
        ops.parallel_update_(x, y, W["ls1"])
    elif L.mlp["kind"] == "dense":
        ops.parallel_update_(x, y, W["ls1"], _dense(ctx, L.mlp, W, h2), W["ls2"])
    else:
        ops.parallel_update_(x, y, W["ls1"], wb=W["ls2"], moe=_moe(ctx, L.mlp, W, h2))
    return xs


def run_layer(ctx, name: str, W: Dict[str, torch.Tensor], state, batch, meta: dict) -> torch.Tensor:
    """One layer run of the stack on a step batch: residual rows (beside them the embedding rows, where passes add
    them) in and out, fp32; ``final.norm`` keeps the rows whose logits are wanted, ``head`` returns their logits."""
    cfg, ops = ctx.cfg, ctx.ops
    kind = layer_kind(name)
    if kind == "embed":
        out, ctx.embed_out = ctx.embed_out, None
        b = cfg.bigram
        return ops.embed_rows(meta["ids"], W["embed"], out=out, copies=cfg.state_width // cfg.width,
                              bigram=None if b is None else (W["bigram"], meta["prev_ids"], int(b["mul_prev"]), int(b["mul_cur"])))
    if kind == "decoder":
        return run_block(ctx, W, state, meta, name)
    if kind == "norm":
        return ops.group_rmsnorm(state[:, :cfg.width], W["norm"], 1, cfg.norm_eps, out_dtype=ctx.compute_dtype, row_idx=meta["want_idx"])
    z = ops.matmul_nt(state, W["head"])
    return ops.scale_(z, cfg.logit_scale) if cfg.logit_scale != 1.0 else z


def layer_flops(cfg, name: str, rows: int, ctx_keys: float = 0.0) -> float:
    """Approximate forward FLOPs of layer run ``name`` on ``rows`` tokens (matrix products; the attention's score and
    value products over ``ctx_keys`` visible keys per row on average)."""
    L, D = cfg.layer(name), cfg.width
    m, n_in = L.mixer, _cols(L)["all"][1]
    f = 2.0 * rows * D * (n_in + m["heads"] * m["vdim"])
    if L.type == "channel_delta":
        f += 2.0 * rows * m["heads"] * (m["dim"] * m["decay_rank"] + m["vdim"] * m["gate_rank"]) + 8.0 * rows * m["heads"] * m["dim"] * m["vdim"]
    else:
        H, d, dr, dv, r, qr = _latent_sizes(L)
        keys = min(ctx_keys, float(_window(m))) if _window(m) else ctx_keys
        f += 2.0 * rows * H * (qr * (d + dr) + d * r + r * dv) + 2.0 * rows * keys * H * (2 * r + dr)
    if L.mlp is not None:
        if L.mlp["kind"] == "dense":
            f += 6.0 * rows * D * int(L.mlp["ff"])
        else:
            r = L.mlp["router"]
            f += 2.0 * rows * D * (int(r["experts"]) + int(r.get("identity", 0)) + 3 * int(r["top"]) * int(L.mlp["expert"]["ff"]))
    return f
