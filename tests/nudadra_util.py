"""Small random Nudadra models for the tests: configurations, weights on disk, and the oracle's answers.
Sizes are deliberately odd and unlike each other (3 query heads per key head, key and value sizes that differ
and are no powers of two, a rotation over part of a head, windows and blocks that divide neither each other nor
a page, state sizes and norm groups of their own) and differ from layer to layer."""
import json
import os

import torch

import nudadra_oracle as oracle
from flexible_llm_sharding_amd.utils.safetensors_io import save_file
from lopilix_util import f64, rel_err, row_errs, tokens  # noqa: F401  (error measures shared by the hybrid families' tests)

SCALING = {"factor": 3.0, "original": 24, "fast": 4.0, "slow": 0.5}


def left(heads=6, kv_heads=2, dim=10, vdim=14, rot_dims=6, base=50.0, scale=0.4, size=11, pool=6, scaling=SCALING):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size, "pool": pool}}
    if rot_dims:
        m["rot"] = {"dims": rot_dims, "base": base}
        if scaling is not None:
            m["rot"]["scaling"] = dict(scaling)
    return m


def right(heads=4, vdim=9, state=7, groups=2, norm_groups=3, conv=4):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}


def layer(lm=None, rm=None, ff=20):
    return {"type": "parallel", "mixer": {"left": lm or left(), "right": rm or right()},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, width=36, vocab=53, eps=1e-5, emb=1.7, loop=None):
    """layers: entries of ``layer`` -> config.json's content."""
    d = {"architecture": "Nudadra", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": emb},
         "layers": json.loads(json.dumps(layers))}
    if loop:
        d["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return d


def random_weights(cfg, seed=0, std=0.3):
    g = torch.Generator().manual_seed(seed)
    D = cfg["width"]

    def mat(*shape, s=std):
        return torch.randn(*shape, generator=g) * s

    one = lambda: (0.6 + torch.rand((), generator=g))
    sd = {"embed": mat(cfg["vocab"], D, s=1.0), "final.norm": one(), "head": mat(cfg["vocab"], D)}
    if cfg.get("loop"):
        sd["loop.in"] = torch.cat([0.7 * torch.eye(D), 0.5 * torch.eye(D)], 1) + mat(D, 2 * D, s=0.1)
        sd["loop.step"] = mat(cfg["loop"]["times"], D, s=0.5)
    for i, l in enumerate(cfg["layers"]):
        p, a, r = f"l{i}.", l["mixer"]["left"], l["mixer"]["right"]
        x, y = p + "mix.left.", p + "mix.right."
        H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        inner, gn, nh = r["heads"] * r["vdim"], r["groups"] * r["state"], r["heads"]
        C = inner + 2 * gn
        sd.update({p + "norm1": one(), x + "q": mat(H * d, D), x + "k": mat(G * d, D), x + "v": mat(G * dv, D), x + "g": mat(H, D),
                   x + "o": mat(D, H * dv), x + "out": 1.0 + mat(D, s=0.3),
                   y + "in": mat(inner + C + nh, D), y + "conv": mat(C, r["conv"], s=0.5), y + "conv.b": mat(C, s=0.3),
                   y + "dt_bias": mat(nh, s=1.0) - 1.0, y + "A_log": mat(nh, s=0.7), y + "D": 1.0 + mat(nh, s=0.5),
                   y + "norm": 1.0 + mat(inner, s=0.3), y + "o": mat(D, inner), y + "out": 1.0 + mat(D, s=0.3)})
        if l["mlp"] is not None:
            sd.update({p + "mlp.up": mat(l["mlp"]["ff"], D), p + "mlp.down": mat(D, l["mlp"]["ff"])})
    return {k: v.to(torch.bfloat16) for k, v in sd.items()}


def write_model(path, cfg, sd):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(sd, os.path.join(path, "model.safetensors"))
    return path


def oracle_logits(cfg, sd, toks, trace=None):
    return oracle.forward(f64(sd), cfg, list(toks), trace).numpy()
