"""A plain, slow Nudadra forward pass in float64, one function per mechanism, written from the
design's equations.  It shares no code with the framework: the tests compare the framework's
kernels, caches and scheduler against it.

Notation: a sequence is a [T, D] matrix of rows x_t, t = 0 .. T-1 its positions; every function
takes the whole sequence and returns the whole output, recomputing everything from t = 0.  ``sd``
maps tensor names to float64 tensors, ``cfg`` is config.json's content.
"""
import math

import torch

F = torch.float64


def rms(x, eps):
    """The last axis divided by sqrt(mean(x^2) + eps)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def rot_freqs(rot):
    """-> (frequencies f_i, i < dims / 2; the factor on every cosine and sine).  Without ``scaling``
    f_i = base^(-2i / dims) and 1.  With it, entry numbers e(t) at which a pair makes t turns over
    ``original`` positions bound a ramp: below e(fast) a frequency stays, above e(slow) it is divided
    by ``factor``, linear between."""
    n, base = int(rot["dims"]), float(rot["base"])
    sc = rot.get("scaling")
    freqs = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if not sc:
        return freqs, 1.0
    factor = float(sc["factor"])
    entry = lambda turns: n * math.log(float(sc["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    first = max(math.floor(entry(float(sc["fast"]))), 0)
    last = min(math.ceil(entry(float(sc["slow"]))), n - 1)
    width = max(last - first, 0.001)
    out = []
    for i, f in enumerate(freqs):
        slow_share = min(1.0, max(0.0, (i - first) / width))
        out.append((1.0 - slow_share) * f + slow_share * f / factor)
    return out, 1.0 + 0.1 * math.log(factor)


def rotate(x, rot):
    """x: [T, heads, n].  Entries i and i + dims / 2 of every head, i < dims / 2, turn by the angle t f_i;
    entries from dims on stay."""
    n = int(rot["dims"])
    freqs, amp = rot_freqs(rot)
    pos = torch.arange(x.shape[0], dtype=F)
    out = x.clone()
    for i, f in enumerate(freqs):
        c, s = amp * torch.cos(pos * f)[:, None], amp * torch.sin(pos * f)[:, None]
        a, b = x[:, :, i], x[:, :, i + n // 2]
        out[:, :, i] = a * c - b * s
        out[:, :, i + n // 2] = b * c + a * s
    return out


def visible(i, size, pool):
    """What position i sees: (token positions, block numbers).  Tokens: its last ``size`` positions, itself
    included.  Blocks: all whose ``pool`` positions are all at least ``size`` back."""
    toks = [j for j in range(i + 1) if i - j < size]
    blocks = [b for b in range(i // pool + 1) if (b + 1) * pool - 1 <= i - size]
    return toks, blocks


def pooled_window_attention(q, k, v, scale, size, pool):
    """q: [T, d], k: [T, d], v: [T, dv] of one head.  One softmax over the visible tokens and the visible
    blocks' mean keys; a block's weight multiplies its mean value."""
    T = q.shape[0]
    out = torch.zeros(T, v.shape[1], dtype=F)
    nb = T // pool
    km = torch.stack([k[b * pool:(b + 1) * pool].mean(0) for b in range(nb)]) if nb else k[:0]
    vm = torch.stack([v[b * pool:(b + 1) * pool].mean(0) for b in range(nb)]) if nb else v[:0]
    for i in range(T):
        toks, blocks = visible(i, size, pool)
        keys, vals = torch.cat([km[blocks], k[toks]]), torch.cat([vm[blocks], v[toks]])
        out[i] = torch.softmax((keys @ q[i]) * scale, 0) @ vals
    return out


def attention(sd, x, m, h):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ sd[x + "q"].T).reshape(T, H, d)
    k = (h @ sd[x + "k"].T).reshape(T, G, d)
    v = (h @ sd[x + "v"].T).reshape(T, G, dv)
    if m.get("rot"):
        q, k = rotate(q, m["rot"]), rotate(k, m["rot"])
    gate = torch.sigmoid(h @ sd[x + "g"].T)
    out = torch.zeros(T, H, dv, dtype=F)
    for hh in range(H):
        g = hh // (H // G)
        o = pooled_window_attention(q[:, hh], k[:, g], v[:, g], float(m["scale"]), int(m["mask"]["size"]), int(m["mask"]["pool"]))
        out[:, hh] = o * gate[:, hh:hh + 1]
    return out.reshape(T, H * dv) @ sd[x + "o"].T


def short_conv(u, w, b):
    """u: [T, C], w: [C, taps] (last column: the current row), zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    out = b[None].repeat(T, 1)
    for back in range(min(taps, T)):
        out[back:] += u[:T - back] * w[:, taps - 1 - back]
    return out


def state_space(sd, x, m, h, eps):
    """Per head a state S [N, P]: S_t = exp(-exp(A) dt_t) S_(t-1) + dt_t B_t x_t^T, y_t = S_t^T C_t + D x_t."""
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, u, dt = torch.split(h @ sd[x + "in"].T, [inner, inner + 2 * G * N, H], 1)
    u = silu(short_conv(u, sd[x + "conv"], sd[x + "conv.b"]))
    xs = u[:, :inner].reshape(T, H, P)
    B = u[:, inner:inner + G * N].reshape(T, G, N)
    C = u[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + sd[x + "dt_bias"])
    out = torch.zeros(T, H, P, dtype=F)
    for hh in range(H):
        g = hh // (H // G)
        S = torch.zeros(N, P, dtype=F)
        for t in range(T):
            S = torch.exp(-torch.exp(sd[x + "A_log"][hh]) * dt[t, hh]) * S + dt[t, hh] * torch.outer(B[t, g], xs[t, hh])
            out[t, hh] = S.T @ C[t, g] + sd[x + "D"][hh] * xs[t, hh]
    y = out.reshape(T, inner) * silu(z)
    ng = int(m["norm_groups"])
    y = rms(y.reshape(T, ng, inner // ng), eps).reshape(T, inner) * sd[x + "norm"]
    return y @ sd[x + "o"].T


def mixer(sd, x, m, h, eps):
    """Half the sum of the two sides' outputs, each RMS-normed over the model width with its own weight."""
    left = rms(attention(sd, x + "left.", m["left"], h), eps) * sd[x + "left.out"]
    right = rms(state_space(sd, x + "right.", m["right"], h, eps), eps) * sd[x + "right.out"]
    return 0.5 * (left + right)


def feed_forward(sd, y, h):
    return torch.relu(h @ sd[y + "up"].T) ** 2 @ sd[y + "down"].T


def layer(sd, cfg, i, x):
    """Mixer and feed-forward side by side on one normed row; the norm's weight is one number."""
    eps = float(cfg["norm"]["eps"])
    h = rms(x, eps) * sd[f"l{i}.norm1"]
    y = mixer(sd, f"l{i}.mix.", cfg["layers"][i]["mixer"], h, eps)
    if cfg["layers"][i].get("mlp") is not None:
        y = y + feed_forward(sd, f"l{i}.mlp.", h)
    return x + y


def schedule(cfg):
    """[(layer number, number of the pass that this layer opens, or None)] in the order of execution."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = int(lp["start"]), int(lp["stop"])
    out = [(i, None) for i in range(a)]
    for t in range(int(lp["times"])):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def forward(sd, cfg, tokens, trace=None):
    """tokens: list of ids -> logits [T, vocab].  ``trace``: a list that receives the residual rows
    after every layer run."""
    x0 = sd["embed"][torch.tensor(tokens)] * float(cfg["embedding"]["scale"])
    x = x0
    for i, opens in schedule(cfg):
        if opens is not None:
            x = torch.cat([x, x0], 1) @ sd["loop.in"].T + sd["loop.step"][opens]
        x = layer(sd, cfg, i, x)
        if trace is not None:
            trace.append(x)
    return (rms(x, float(cfg["norm"]["eps"])) * sd["final.norm"]) @ sd["head"].T
