"""A plain, slow Numolorn forward pass in float64, one function per mechanism, written from the
design's equations.  It shares no code with the framework: the tests compare the framework's
kernels, caches and scheduler against it.

Notation: a sequence is a [T, D] matrix of rows x_t, t = 0 .. T-1 its positions; every function
takes the whole sequence and returns the whole output, recomputing everything from t = 0.  ``sd``
maps tensor names to float64 tensors, ``cfg`` is config.json's content.
"""
import torch

F = torch.float64


def rms(x, eps):
    """The last axis divided by sqrt(mean(x^2) + eps)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


# ------------------------------------------------------------------------------ embedding
def bigram_row(prev, cur, b):
    """The bigram table's row for token ``cur`` after ``prev`` (None: nothing precedes it)."""
    n = int(b["buckets"])
    return n if prev is None else (int(prev) * int(b["mul_prev"]) + int(cur) * int(b["mul_cur"])) % n


def embed(sd, cfg, tokens):
    b = cfg["embedding"]["bigram"]
    rows = []
    for t, tok in enumerate(tokens):
        rows.append(sd["embed"][tok] + sd["bigram"][bigram_row(tokens[t - 1] if t else None, tok, b)])
    return torch.stack(rows)


# ------------------------------------------------------------------------------ attention
def rotate(x, dims, base):
    """x: [T, n].  Entries i and i + dims / 2, i < dims / 2, turn by the angle t base^(-2i / dims); entries from dims
    on stay."""
    pos = torch.arange(x.shape[0], dtype=F)
    out = x.clone()
    half = dims // 2
    for i in range(half):
        a = pos * float(base) ** (-2.0 * i / dims)
        out[:, i] = x[:, i] * torch.cos(a) - x[:, i + half] * torch.sin(a)
        out[:, i + half] = x[:, i + half] * torch.cos(a) + x[:, i] * torch.sin(a)
    return out


def sees(i, j, size=None):
    """Whether position i sees position j: never a later one, with a window only its last ``size`` ones."""
    return j <= i and (size is None or i - j < size)


def softmax_attention(q, k, v, scale, size=None, sink=None):
    """q: [T, d], k: [T, d], v: [T, dv] of one head.  ``sink``: a score whose exponential only joins the
    denominator."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F)
    for i in range(q.shape[0]):
        js = [j for j in range(i + 1) if sees(i, j, size)]
        s = (k[js] @ q[i]) * scale
        top = s.max() if sink is None else torch.maximum(s.max(), sink)
        e = torch.exp(s - top)
        den = e.sum() + (0.0 if sink is None else torch.exp(sink - top))
        out[i] = (e / den) @ v[js]
    return out


def latent_attention(sd, x, m, h, eps):
    """Queries through a latent; keys and values from a latent, a rotated key part shared by the heads, a sink and a
    sigmoid gate per head."""
    T = h.shape[0]
    H, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = rms(h @ sd[x + "dq"].T, eps) * sd[x + "dq.norm"]
    q = (cq @ sd[x + "uq"].T).reshape(T, H, d + dr)
    z = h @ sd[x + "dkv"].T
    c = rms(z[:, :r], eps) * sd[x + "dkv.norm"]
    rot = m["rot"]
    kr = rotate(z[:, r:], int(rot["dims"]), rot["base"])
    k, v = (c @ sd[x + "uk"].T).reshape(T, H, d), (c @ sd[x + "uv"].T).reshape(T, H, dv)
    gate = torch.sigmoid(h @ sd[x + "g"].T)
    outs = []
    for hh in range(H):
        qr = rotate(q[:, hh, d:], int(rot["dims"]), rot["base"])
        o = softmax_attention(torch.cat([q[:, hh, :d], qr], 1), torch.cat([k[:, hh], kr], 1), v[:, hh], float(m["scale"]),
                              sink=sd[x + "sink"][hh])
        outs.append(o * gate[:, hh:hh + 1])
    return torch.cat(outs, 1) @ sd[x + "o"].T


def window_latent_attention(sd, x, m, h, eps):
    """Keys and values from a latent, no positions, a sliding window, an ordinary softmax."""
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ sd[x + "q"].T).reshape(T, H, d)
    c = rms(h @ sd[x + "dkv"].T, eps) * sd[x + "dkv.norm"]
    k, v = (c @ sd[x + "uk"].T).reshape(T, H, d), (c @ sd[x + "uv"].T).reshape(T, H, dv)
    outs = [softmax_attention(q[:, hh], k[:, hh], v[:, hh], float(m["scale"]), size=int(m["mask"]["size"])) for hh in range(H)]
    return torch.cat(outs, 1) @ sd[x + "o"].T


# ------------------------------------------------------------------------------ delta rule
def short_conv(u, w):
    """u: [T, C], w: [C, taps] (last column: the current row), zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u)
    for back in range(min(taps, T)):
        out[back:] += u[:T - back] * w[:, taps - 1 - back]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_step(S, q, k, v, g, beta):
    """One token of one head.  S [key, value] decays per key row, the value it holds for k moves towards v by beta, the
    read-out follows the write.  -> (new S, o)."""
    S = g[:, None] * S
    u = beta * (v - S.T @ k)
    S = S + torch.outer(k, u)
    return S, S.T @ q


def channel_delta(sd, x, m, h, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ sd[x + n].T, sd[x + n + ".conv"])) for n in ("q", "k", "v"))
    q, k = unit(q.reshape(T, G, d)) * d ** -0.5, unit(k.reshape(T, G, d))
    v = v.reshape(T, H, dv)
    beta = torch.sigmoid(h @ sd[x + "b"].T)
    a = softplus(h @ sd[x + "a1"].T @ sd[x + "a2"].T + sd[x + "dt_bias"]).reshape(T, H, d)
    g = torch.exp(-torch.exp(sd[x + "A_log"])[None, :, None] * a)
    gate = torch.sigmoid(h @ sd[x + "g1"].T @ sd[x + "g2"].T)
    out = torch.zeros(T, H, dv, dtype=F)
    for hh in range(H):
        S = torch.zeros(d, dv, dtype=F)
        kv = hh // (H // G)
        for t in range(T):
            S, out[t, hh] = delta_step(S, q[t, kv], k[t, kv], v[t, hh], g[t, hh], beta[t, hh])
    y = (rms(out, eps) * sd[x + "norm"]).reshape(T, H * dv) * gate
    return y @ sd[x + "o"].T


# ------------------------------------------------------------------------------ feed-forward
def dense(sd, y, h):
    return (silu(h @ sd[y + "gate"].T) * (h @ sd[y + "up"].T)) @ sd[y + "down"].T


def route(z, corr, r):
    """Router logits of one token -> [(expert, weight)] of the chosen ones."""
    s = torch.softmax(z, -1)
    choice = (s + corr).tolist()
    groups = r.get("groups")
    allowed = list(range(len(choice)))
    if groups:
        per = len(choice) // int(groups["count"])
        worth = [max(choice[g * per:(g + 1) * per]) for g in range(int(groups["count"]))]
        best = sorted(range(len(worth)), key=lambda g: -worth[g])[:int(groups["keep"])]
        allowed = [e for e in allowed if e // per in best]
    chosen = sorted(allowed, key=lambda e: -choice[e])[:int(r["top"])]
    total = sum(float(s[e]) for e in chosen) + 1e-20
    return [(e, float(s[e]) / total * float(r["scale"])) for e in chosen]


def expert(sd, p, h, limit):
    g = torch.clamp(h @ sd[p + "gate"].T, max=limit)
    u = torch.clamp(h @ sd[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ sd[p + "down"].T


def mixture(sd, y, mlp, h):
    """``experts`` experts with weights of their own; the router outputs behind them hand the input on."""
    r, lim = mlp["router"], float(mlp["expert"]["limit"])
    z = h @ sd[y + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], sd[y + "correction"], r):
            out[t] += w * (h[t] if e >= int(r["experts"]) else expert(sd, f"{y}e{e}.", h[t:t + 1], lim)[0])
    return out


# ------------------------------------------------------------------------------ the stack
MIXERS = {"latent_attention": latent_attention, "latent_attention_2": window_latent_attention, "channel_delta": channel_delta}


def layer(sd, cfg, i, x):
    """Mixer and feed-forward side by side, each on its own norm of the same row, each scaled per channel."""
    eps, L, p = float(cfg["norm"]["eps"]), cfg["layers"][i], f"l{i}."
    new = x + MIXERS[L["type"]](sd, p + "mix.", L["mixer"], rms(x, eps) * sd[p + "norm1"], eps) * sd[p + "ls1"]
    if L.get("mlp") is not None:
        h = rms(x, eps) * sd[p + "norm2"]
        f = dense(sd, p + "mlp.", h) if L["mlp"]["kind"] == "dense" else mixture(sd, p + "mlp.", L["mlp"], h)
        new = new + f * sd[p + "ls2"]
    return new


def schedule(cfg):
    """[(layer number, whether the embedding rows join before it)] in the order of execution."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b = int(lp["start"]), int(lp["stop"])
    out = [(i, False) for i in range(a)]
    for t in range(int(lp["times"])):
        out += [(i, t > 0 and i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, n)]


def forward(sd, cfg, tokens, trace=None):
    """tokens: list of ids -> logits [T, vocab].  ``trace``: a list that receives the residual rows
    after every layer run."""
    x0 = embed(sd, cfg, list(tokens))
    x = x0
    for i, again in schedule(cfg):
        if again:
            x = x + x0
        x = layer(sd, cfg, i, x)
        if trace is not None:
            trace.append(x)
    return (rms(x, float(cfg["norm"]["eps"])) * sd["final.norm"]) @ sd["embed"].T * float(cfg["logit_scale"])
