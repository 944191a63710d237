"""Small random Numolorn models for the tests: configurations, weights on disk, and the oracle's answers.  Sizes are
deliberately odd and unlike each other (heads, key, value and rotated sizes that differ and are no powers of two, a latent
narrower than the heads it feeds, two value heads per key head, three ranks of their own, expert groups that mix experts
and identity experts) and differ from layer to layer."""
import json
import os

import torch

import numolorn_oracle as oracle
from flexible_llm_sharding_amd.utils.safetensors_io import save_file
from lopilix_util import f64, rel_err, row_errs, tokens  # noqa: F401  (error measures shared by the hybrid families' tests)

BIGRAM = {"buckets": 29, "mul_prev": 11, "mul_cur": 3}


def latent(heads=3, dim=6, rot_dim=8, vdim=5, kv_rank=11, q_rank=9, base=100.0, scale=0.3):
    return ("latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                                 "rot": {"dims": rot_dim, "base": base}, "scale": scale})


def window(heads=4, dim=7, vdim=9, kv_rank=10, size=12, scale=0.35):
    return ("latent_attention_2", {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": size}, "scale": scale})


def delta(heads=4, kv_heads=2, dim=7, vdim=9, conv=4):
    return ("channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv})


def dense(ff=20):
    return {"kind": "dense", "ff": ff}


def moe(experts=7, identity=2, top=3, ff=11, groups=(3, 2), scale=1.7, limit=0.8):
    r = {"experts": experts, "identity": identity, "top": top, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "router": r, "expert": {"ff": ff, "limit": limit}}


def config(layers, width=36, vocab=53, eps=1e-5, logit_scale=0.6, loop=None, bigram=BIGRAM):
    """layers: [((type, mixer dict), mlp dict or None)] -> config.json's content."""
    d = {"architecture": "Numolorn", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_scale": logit_scale,
         "embedding": {"bigram": dict(bigram)},
         "layers": [{"type": t, "mixer": json.loads(json.dumps(m)), "mlp": json.loads(json.dumps(f))} for (t, m), f in layers]}
    if loop:
        d["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return d


def random_weights(cfg, seed=0, std=0.3, ranks=(5, 3)):
    """``ranks``: inner sizes of the delta rule's two two-layer maps (decay, gate)."""
    g = torch.Generator().manual_seed(seed)
    D = cfg["width"]

    def mat(*shape, s=std):
        return torch.randn(*shape, generator=g) * s

    near1 = lambda n, s=0.3: 1.0 + mat(n, s=s)
    sd = {"embed": mat(cfg["vocab"], D, s=1.0), "bigram": mat(cfg["embedding"]["bigram"]["buckets"] + 1, D, s=0.7), "final.norm": near1(D)}
    for i, l in enumerate(cfg["layers"]):
        p, m, x = f"l{i}.", l["mixer"], f"l{i}.mix."
        sd.update({p + "norm1": near1(D), p + "ls1": near1(D, 0.4)})
        if l["type"] == "channel_delta":
            H, G, d, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            ra, rg = ranks
            sd.update({x + "q": mat(G * d, D), x + "k": mat(G * d, D), x + "v": mat(H * dv, D), x + "q.conv": mat(G * d, taps, s=0.5),
                       x + "k.conv": mat(G * d, taps, s=0.5), x + "v.conv": mat(H * dv, taps, s=0.5), x + "b": mat(H, D),
                       x + "A_log": mat(H, s=0.7) - 1.0, x + "norm": near1(dv), x + "a1": mat(ra, D), x + "a2": mat(H * d, ra),
                       x + "dt_bias": mat(H * d, s=1.0) - 1.0, x + "g1": mat(rg, D), x + "g2": mat(H * dv, rg), x + "o": mat(D, H * dv)})
        else:
            H, d, dv, r = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
            dr = m.get("rot_dim", 0)
            sd.update({x + "dkv": mat(r + dr, D), x + "dkv.norm": near1(r), x + "uk": mat(H * d, r), x + "uv": mat(H * dv, r),
                       x + "o": mat(D, H * dv)})
            if l["type"] == "latent_attention":
                qr = m["q_rank"]
                sd.update({x + "dq": mat(qr, D), x + "dq.norm": near1(qr), x + "uq": mat(H * (d + dr), qr), x + "sink": mat(H, s=1.0),
                           x + "g": mat(H, D)})
            else:
                sd[x + "q"] = mat(H * d, D)
        f = l["mlp"]
        if f is None:
            continue
        y = p + "mlp."
        sd.update({p + "norm2": near1(D), p + "ls2": near1(D, 0.4)})
        if f["kind"] == "dense":
            sd.update({y + "gate": mat(f["ff"], D), y + "up": mat(f["ff"], D), y + "down": mat(D, f["ff"])})
        else:
            Z = f["router"]["experts"] + f["router"]["identity"]
            sd.update({y + "router": mat(Z, D), y + "correction": mat(Z, s=0.2)})
            for e in range(f["router"]["experts"]):
                sd.update({f"{y}e{e}.gate": mat(f["expert"]["ff"], D), f"{y}e{e}.up": mat(f["expert"]["ff"], D),
                           f"{y}e{e}.down": mat(D, f["expert"]["ff"])})
    return {k: v.to(torch.bfloat16) for k, v in sd.items()}


def write_model(path, cfg, sd):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(sd, os.path.join(path, "model.safetensors"))
    return path


def oracle_logits(cfg, sd, toks, trace=None):
    return oracle.forward(f64(sd), cfg, list(toks), trace).numpy()
