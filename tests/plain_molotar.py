"""A plain, slow Molotar in float64: whole sequences, one function per mechanism, no cache.

The oracle of the Molotar tests.  It shares nothing with the engine: it takes the raw ``config.json``
dictionary and the tensors by their file names, and computes every position of a sequence from the
sequence's start.

    x_0       = embed[t] * scale + bigram[row(t_prev, t)]
    per layer:  x <- g1 * unit(alpha * x + mixer(x));   x <- g2 * unit(alpha * x + experts(x))
    logits    = head . (g_final * unit(x))

with ``unit(v) = v / sqrt(mean(v^2) + eps)``.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def weighted_norm(x, g, eps):
    return unit(x, eps) * g.to(F64)


def post_norm(x, y, g, alpha, eps):
    """The stream after a sublayer's result ``y``: the norm of the sum."""
    return weighted_norm(alpha * x + y, g, eps)


# ---------------------------------------------------------------- embedding
def pair_rows(tokens, buckets, mul_prev, mul_cur):
    rows = [buckets]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((int(prev) * mul_prev + int(cur) * mul_cur) % buckets)
    return rows


def embed(tokens, cfg, w):
    e = cfg["embedding"]
    x = w["embed"].to(F64)[list(tokens)] * float(e["scale"])
    b = e.get("bigram")
    if b:
        x = x + w["bigram"].to(F64)[pair_rows(list(tokens), b["buckets"], b["mul_prev"], b["mul_cur"])]
    return x


# ---------------------------------------------------------------- attention
def frequencies(rot):
    """Angle per position of every turning pair, slow waves stretched by ``scaling``."""
    dims, sc = rot["dims"], rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = float(rot["base"]) ** (-2.0 * i / dims)
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate(x, rot):
    """``x [n, heads, d]``, row ``p`` at position ``p``: channel ``i`` turns with channel ``i + dims / 2``."""
    if not rot or not rot["dims"]:
        return x
    half = rot["dims"] // 2
    f = torch.tensor(frequencies(rot), dtype=F64)
    angle = torch.arange(x.shape[0], dtype=F64)[:, None] * f
    c, s = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], dim=-1)


def whole_norm(x, g, eps):
    """``x [n, heads * d]`` over its whole width, all heads at once."""
    return weighted_norm(x, g, eps)


def attend(q, k, v, scale, window):
    """``q [n, H, d]``, ``k [n, G, d]``, ``v [n, G, e]``; a denominator with one added; window None: all."""
    n, heads, _ = q.shape
    per = heads // k.shape[1]
    out = torch.zeros(n, heads, v.shape[-1], dtype=F64)
    for i in range(n):
        first = 0 if window is None else max(0, i - window + 1)
        for h in range(heads):
            g = h // per
            s = (k[first:i + 1, g] @ q[i, h]) * scale
            top = max(0.0, float(s.max()))
            e = torch.exp(s - top)
            out[i, h] = (e / (math.exp(-top) + e.sum())) @ v[first:i + 1, g]
    return out


def gate_heads(out, z):
    """``out [n, H, e]`` times the sigmoid of one number per head."""
    return out * torch.sigmoid(z)[..., None]


def keys_values(h, m, w, p, eps):
    """A layer's keys, normed and turned, and its values."""
    n, groups = h.shape[0], m.get("kv_heads", m["heads"])
    k = whole_norm(h @ w[p + "k"].to(F64).T, w[p + "k.norm"], eps)
    v = h @ w[p + "v"].to(F64).T
    return rotate(k.view(n, groups, m["dim"]), m.get("rot")), v.view(n, groups, m["vdim"])


def attention(h, m, w, p, eps, kv):
    n = h.shape[0]
    q = whole_norm(h @ w[p + "q"].to(F64).T, w[p + "q.norm"], eps).view(n, m["heads"], m["dim"])
    out = attend(rotate(q, m.get("rot")), kv[0], kv[1], float(m["scale"]), (m.get("mask") or {}).get("size"))
    out = gate_heads(out, h @ w[p + "g"].to(F64).T)
    return out.reshape(n, -1) @ w[p + "o"].to(F64).T


# ---------------------------------------------------------------- recurrence
def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(x, taps, bias):
    """``y_t = bias + sum_j taps[:, j] x_(t - T + 1 + j)`` with ``T`` taps, zeros before the start."""
    t, wt = taps.shape[1], taps.to(F64)
    past = torch.cat([torch.zeros(t - 1, x.shape[1], dtype=F64), x])
    return bias.to(F64) + sum(past[j:j + x.shape[0]] * wt[:, j] for j in range(t))


def block_gate(u, weight, bias):
    """Part ``b`` of ``u`` through the square matrix ``b``, the bias, a sigmoid."""
    blocks, size, _ = weight.shape
    parts = u.view(u.shape[0], blocks, size)
    z = torch.stack([parts[:, b] @ weight[b].to(F64).T for b in range(blocks)], dim=1) + bias.to(F64)
    return torch.sigmoid(z).reshape(u.shape)


def decay_logs(r, lam):
    return -8.0 * r * torch.nn.functional.softplus(lam.to(F64))


def gated_unit(log_a, gated):
    """``S_t = a_t S_(t-1) + sqrt(1 - a_t^2) gated_t`` from zero."""
    s, out = torch.zeros(gated.shape[1], dtype=F64), []
    for t in range(gated.shape[0]):
        a = torch.exp(log_a[t])
        s = a * s + torch.sqrt(1.0 - a * a) * gated[t]
        out.append(s)
    return torch.stack(out)


def rglru(h, w, p):
    y = gelu_tanh(h @ w[p + "y"].to(F64).T + w[p + "y.b"].to(F64))
    u = causal_conv(h @ w[p + "x"].to(F64).T + w[p + "x.b"].to(F64), w[p + "conv"], w[p + "conv.b"])
    r = block_gate(u, w[p + "ra"], w[p + "ra.b"])
    i = block_gate(u, w[p + "ri"], w[p + "ri.b"])
    s = gated_unit(decay_logs(r, w[p + "lam"]), i * u)
    return (s * y) @ w[p + "o"].to(F64).T


# ---------------------------------------------------------------- experts
def clamped_expert(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].to(F64).T, max=limit)
    u = torch.clamp(h @ w[p + "up"].to(F64).T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].to(F64).T


def route(h, weight, router):
    """Per row a list of ``(expert, weight)``: a group of neighbours counts as the sum of its two largest
    scores, the largest scores of the kept groups win (ties: the smaller index), their scores
    normalised to a sum of ``scale``."""
    s = torch.sigmoid(h @ weight.to(F64).T)
    groups = router.get("groups") or dict(count=1, keep=1)
    per = s.shape[1] // groups["count"]
    picks = []
    for row in s.tolist():
        value = [sum(sorted(row[g * per:(g + 1) * per], reverse=True)[:2]) for g in range(groups["count"])]
        kept = sorted(range(groups["count"]), key=lambda g: (-value[g], g))[:groups["keep"]]
        allowed = [e for g in kept for e in range(g * per, (g + 1) * per)]
        chosen = sorted(allowed, key=lambda e: (-row[e], e))[:router["top"]]
        total = sum(row[e] for e in chosen) + 1e-20
        picks.append([(e, row[e] / total * router["scale"]) for e in chosen])
    return picks


def mixture(h, mlp, w, p):
    picks = route(h, w[p + "router"], mlp["router"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows = [t for t, row in enumerate(picks) if any(c == e for c, _ in row)]
        if rows:
            share = torch.tensor([next(s for c, s in picks[t] if c == e) for t in rows], dtype=F64)
            out[rows] += share[:, None] * clamped_expert(h[rows], w, f"{p}e{e}.", float(mlp["expert"]["limit"]))
    return out


# ---------------------------------------------------------------- the model
def forward(tokens, cfg, w, layers_out=None):
    """Logits ``[n, vocab]`` of a whole sequence; ``layers_out``: a list that receives the stream after
    every layer."""
    eps, alpha = cfg["norm"]["eps"], float(cfg["postln_alpha"])
    x, kept = embed(tokens, cfg, w), {}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        if spec["type"] == "rglru":
            y = rglru(x, w, p + "mix.")
        elif spec["type"] == "attention":
            source = m.get("kv_from")
            kept[i] = kept[source] if source is not None else keys_values(x, m, w, p + "mix.", eps)
            y = attention(x, m, w, p + "mix.", eps, kept[i])
        else:
            raise ValueError(spec["type"])
        x = post_norm(x, y, w[p + "norm1"], alpha, eps)
        if spec.get("mlp"):
            x = post_norm(x, mixture(x, spec["mlp"], w, p + "mlp."), w[p + "norm2"], alpha, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return weighted_norm(x, w["final.norm"], eps) @ w["head"].to(F64).T


def greedy(tokens, cfg, w, count):
    out = list(tokens)
    for _ in range(count):
        out.append(int(forward(out, cfg, w)[-1].argmax()))
    return out[len(tokens):]
