"""Nudadra layer execution on packed weight images and packed step batches.

A layer runs two mixers and a feed-forward side by side on one normed row (the norm's weight is one
number g):

    h = g x / sqrt(mean(x^2) + eps)
    x <- x + (rms(left(h)) w_l + rms(right(h)) w_r) / 2 + W_down max(W_up h, 0)^2

* left -- grouped-query attention.  q and k are rotated in pairs (i, i + dims / 2) over the first
  ``rot.dims`` entries (frequencies rescaled by how often an entry turns over the original context, cosines
  and sines amplified).  Row i sees its last ``mask.size`` tokens and, in the same softmax, one key and value
  for each block of ``mask.pool`` tokens that ends before that window: the mean of the block's cached keys
  (values).  The means are rows of block pools beside the pages, written when a block's last token is.  Head
  h's output is multiplied by sigmoid(g_h) before the output projection;
* right -- a Mamba-2 mixer: S_t = exp(-exp(A) dt_t) S_(t-1) + dt_t B_t x_t^T, y_t = S_t^T C_t + D x_t over
  convolved x, B and C, y gated by silu(z) and RMS-normed in ``norm_groups`` parts.

``loop``: before every pass over the looped layers x <- W_in [x; x0] + step_t with x0 the embedding row, so
the activation that passes from layer to layer is [x | x0] ([T, 2 D] fp32): the product reads it as it lies,
step_t is its bias.  W_in and the step vectors are part of the first looped layer's image.  Every pass has
pages, blocks and states of its own (execution names ``l0``, ``l0@1``, ...).

Each mechanism is an op of the backend (``ops/hip_seq.py``: the kernels of ``csrc/kernels/seq``;
``ops/torch_seq.py`` on the CPU) with its constants as arguments; this file only strings them together.
Keys, values, blocks and recurrent states live in :class:`~..runtime.seq_state.SequenceStateCache`.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from .kagolix import HybridContext, _mamba_cols  # noqa: F401  (the context the engine builds for every hybrid family)
from .layout import LayerLayout, Placement, layer_image, layer_kind, spec_layout, spec_placements
from .lopilix import _rot

F32 = "f32"
BRANCH_WEIGHT = 0.5                # each mixer's share of the sum


def _cols(mixer: dict) -> Dict[str, tuple]:
    """Column ranges (start, width) of the stacked input projection of both mixers: q | k | v | z | xBC | dt | g."""
    a, r = mixer["left"], mixer["right"]
    inner, gn, _ = _mamba_cols(r)
    out, at = {}, 0
    for n, w in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"]),
                 ("z", inner), ("xbc", inner + 2 * gn), ("dt", r["heads"]), ("g", a["heads"])):
        out[n] = (at, int(w))
        at += int(w)
    out["all"] = (0, at)
    return out


def _specs(cfg, name: str):
    """[(slot, shape, dtype tag, [(checkpoint tensor, element offset in the slot, shape)])]."""
    D, V = cfg.width, cfg.vocab
    kind = layer_kind(name)
    if kind == "embed":
        return [("embed", (V, D), None, [("embed", 0, (V, D))])]
    if kind == "head":
        return [("head", (V, D), None, [("head", 0, (V, D))])]
    if kind == "norm":
        return [("norm", (1,), F32, [("final.norm", 0, ())])]
    image = layer_image(name)
    L, p = cfg.layer(name), image + "."
    a, r = L.mixer["left"], L.mixer["right"]
    c = _cols(L.mixer)
    inner, gn, n_in = _mamba_cols(r)
    C, nh, taps, o = inner + 2 * gn, r["heads"], r["conv"], a["heads"] * a["vdim"]
    x, y = p + "mix.left.", p + "mix.right."
    row = lambda n: c[n][0] * D
    out = []
    if cfg.loop_pass(image) is not None:
        times = int(cfg.loop["times"])
        out += [("loop_in", (D, 2 * D), None, [("loop.in", 0, (D, 2 * D))]),
                ("loop_step", (times, D), F32, [("loop.step", 0, (times, D))])]
    out += [("norm1", (1,), F32, [(p + "norm1", 0, ())]),
            ("win", (c["all"][1], D), None,
             [(x + "q", row("q"), (c["q"][1], D)), (x + "k", row("k"), (c["k"][1], D)), (x + "v", row("v"), (c["v"][1], D)),
              (y + "in", row("z"), (n_in, D)), (x + "g", row("g"), (c["g"][1], D))]),
            ("wol", (D, o), None, [(x + "o", 0, (D, o))]),
            ("conv", (C, taps), F32, [(y + "conv", 0, (C, taps))]), ("convb", (C,), F32, [(y + "conv.b", 0, (C,))]),
            ("dt_bias", (nh,), F32, [(y + "dt_bias", 0, (nh,))]),
            ("A_log", (nh,), F32, [(y + "A_log", 0, (nh,))]), ("Dskip", (nh,), F32, [(y + "D", 0, (nh,))]),
            ("mnorm", (inner,), F32, [(y + "norm", 0, (inner,))]),
            ("wor", (D, inner), None, [(y + "o", 0, (D, inner))]),
            ("outl", (D,), F32, [(p + "mix.left.out", 0, (D,))]), ("outr", (D,), F32, [(p + "mix.right.out", 0, (D,))])]
    if L.mlp is not None:
        ff = int(L.mlp["ff"])
        out += [("wup", (ff, D), None, [(p + "mlp.up", 0, (ff, D))]), ("wdown", (D, ff), None, [(p + "mlp.down", 0, (D, ff))])]
    return out


def layout(cfg, name: str, elem_size: int = 2) -> LayerLayout:
    return spec_layout(layer_kind(name), _specs(cfg, name), elem_size)


def placements(cfg, name: str, elem_size: int = 2) -> List[Placement]:
    return spec_placements(layout(cfg, name, elem_size), _specs(cfg, name), elem_size)


def state_spec(cfg) -> dict:
    """What a request keeps between steps, per pass of every layer: key and value pages of the window (given back
    behind it, but not before the block they belong to is complete), block pools with a mean key and value per
    block, the convolution's last inputs and the recurrent state."""
    paged, blocks, slots, horizons = {}, {}, {}, []
    for name in cfg.layer_names():
        if layer_kind(name) != "decoder":
            continue
        a, r = cfg.layer(name).mixer["left"], cfg.layer(name).mixer["right"]
        kw = {"k": a["kv_heads"] * a["dim"], "v": a["kv_heads"] * a["vdim"]}
        size, pool = int(a["mask"]["size"]), int(a["mask"]["pool"])
        paged[name] = kw
        blocks[name] = (pool, dict(kw))
        horizons += [("window", size, 0), ("chunk", pool, 0)]        # (the unfinished block's tokens are read again)
        inner, gn, _ = _mamba_cols(r)
        slots[name] = {"conv": (r["conv"] - 1, inner + 2 * gn), "state": (r["heads"], r["state"], r["vdim"])}
    return {"paged": paged, "alias": {}, "blocks": blocks, "slots": slots, "horizons": horizons}


# ------------------------------------------------------------------------------------ execution
def _attention(ctx, m: dict, W, z, c, meta, name: str):
    ops, cdt, cache = ctx.ops, ctx.compute_dtype, ctx.cache
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    kc, vc = cache.kv(name)
    blocks = cache.block_pools(name, meta)
    q = torch.empty(z.shape[0], H * d, dtype=torch.float32, device=z.device)
    # rotation, the write into the pages and the means of the blocks that these rows complete
    ops.qkv_conv_rope_store(z, None, None, meta, H, G, d, dv, q, kc, vc, rot=_rot(m), norm=False, half=True, blocks=blocks)
    a = ops.attn_paged(q, kc, vc, meta, H, G, d, dv, scale=float(m["scale"]), softcap=0.0, r1=None, r2=None, chunk=0,
                       page_size=cache.page_size, out_dtype=cdt, window=int(m["mask"]["size"]), blocks=blocks,
                       head_gate=z[:, c["g"][0]:c["g"][0] + H])
    return ops.matmul_nt(a, W["wol"])


def _state_space(ctx, m: dict, W, z, c, meta, name: str):
    ops = ctx.ops
    col = lambda n: z[:, c[n][0]:c[n][0] + c[n][1]]
    st = ctx.cache.recurrent(name)
    xbc = ops.causal_conv(col("xbc"), W["conv"], W["convb"], st["conv"], meta, act="silu")
    y = ops.ssd_scan(xbc, col("z"), col("dt"), W["dt_bias"], W["A_log"], W["Dskip"], st["state"], meta, m["heads"], m["vdim"],
                     m["state"], m["groups"])                              # fp32, gated by silu(z)
    return ops.matmul_nt(ops.group_rmsnorm(y, W["mnorm"], m["norm_groups"], ctx.cfg.norm_eps, out_dtype=ctx.compute_dtype), W["wor"])


def run_block(ctx, W, xs: torch.Tensor, meta: dict, name: str) -> torch.Tensor:
    cfg, ops, cdt = ctx.cfg, ctx.ops, ctx.compute_dtype
    L, eps = cfg.layer(name), cfg.norm_eps
    x = xs[:, :cfg.width]
    t = cfg.loop_pass(name)
    if t is None:
        h = ops.group_rmsnorm(x, W["norm1"], 1, eps, out_dtype=cdt)
    else:                                                                   # the row is replaced: W_in [x; x0] + step_t
        entry = ops.matmul_nt(ops.cast_rows(xs, cdt), W["loop_in"], bias=W["loop_step"][t])
        h = ops.residual_branches_(x, add=entry, keep=False, eps=eps, norm_w=W["norm1"], out_dtype=cdt)
    c = _cols(L.mixer)
    z = ops.matmul_nt(h, W["win"])                                          # fp32 [T, q | k | v | z | xBC | dt | g]
    left = _attention(ctx, L.mixer["left"], W, z, c, meta, name)
    right = _state_space(ctx, L.mixer["right"], W, z, c, meta, name)
    ff = None
    if L.mlp is not None:
        ff = ops.matmul_nt(ops.matmul_nt(h, W["wup"], relu2=True, out_dtype=cdt), W["wdown"])
    ops.residual_branches_(x, ((left, W["outl"]), (right, W["outr"])), coef=BRANCH_WEIGHT, add=ff, eps=eps)
    return xs


def run_layer(ctx, name: str, W: Dict[str, torch.Tensor], state, batch, meta: dict) -> torch.Tensor:
    """One layer run of the stack on a step batch: residual rows (beside them the embedding rows, in a looped
    stack) in and out, fp32; ``final.norm`` keeps the rows whose logits are wanted, ``head`` returns their logits."""
    cfg, ops = ctx.cfg, ctx.ops
    kind = layer_kind(name)
    if kind == "embed":
        out, ctx.embed_out = ctx.embed_out, None
        return ops.embed_rows(meta["ids"], W["embed"], out=out, scale=cfg.embedding_scale, copies=cfg.state_width // cfg.width)
    if kind == "decoder":
        return run_block(ctx, W, state, meta, name)
    if kind == "norm":
        return ops.group_rmsnorm(state[:, :cfg.width], W["norm"], 1, cfg.norm_eps, out_dtype=ctx.compute_dtype, row_idx=meta["want_idx"])
    return ops.matmul_nt(state, W["head"])


def layer_flops(cfg, name: str, rows: int, ctx_keys: float = 0.0) -> float:
    """Approximate forward FLOPs of layer run ``name`` on ``rows`` tokens (matrix products; the attention's score
    and value products over ``ctx_keys`` earlier tokens per row on average, seen as window and blocks)."""
    L, D = cfg.layer(name), cfg.width
    a, r = L.mixer["left"], L.mixer["right"]
    inner, _, _ = _mamba_cols(r)
    f = 2.0 * rows * D * (_cols(L.mixer)["all"][1] + a["heads"] * a["vdim"] + inner) + 6.0 * rows * inner * r["state"]
    size = float(a["mask"]["size"])
    keys = min(ctx_keys, size) + max(0.0, ctx_keys - size) / int(a["mask"]["pool"])
    f += 2.0 * rows * keys * a["heads"] * (a["dim"] + a["vdim"])
    if L.mlp is not None:
        f += 4.0 * rows * D * int(L.mlp["ff"])
    if cfg.loop_pass(name) is not None:
        f += 4.0 * rows * D * D
    return f
