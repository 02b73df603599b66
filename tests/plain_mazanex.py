"""A plain, slow implementation of the Mazanex decoder, one function per mechanism, in float64
on the CPU.  It shares no code with the engine: tensors come as a dictionary by file name, the
configuration as the dictionary of ``config.json``.

Notation: ``h [T, W]`` the rows of one sequence at positions ``0 .. T-1``; ``H`` heads, ``G``
key/value heads, ``D`` the width of a query or key head, ``E`` of a value head.
"""
from __future__ import annotations

import torch

F = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def before(h, first=None):
    """Row ``t`` holds ``h``'s row ``t - 1``; row 0 holds ``first`` (zeros where a sequence starts)."""
    first = torch.zeros_like(h[:1]) if first is None else first.view(1, -1)
    return torch.cat([first, h[:-1]], dim=0)


def token_shift(h, mix, first=None):
    return h + (before(h, first) - h) * mix


# -------------------------------------------------------------- feed-forward
def poly_norm(z, a, b, c, e, eps):
    return a * unit_rms(z, eps) + b * unit_rms(z ** 2, eps) + c * unit_rms(z ** 3, eps) + e


def poly_mlp(h, up, down, act, eps):
    a, b, c, e = (act[i] for i in range(4))
    return poly_norm(h @ up.T, a, b, c, e, eps) @ down.T


# ----------------------------------------------------------------- attention
def short_conv(u, w):
    """``u [T, C]``, ``w [C, taps]``: ``y_t = sum_j w[:, j] u_(t - taps + 1 + j)``, nothing before row 0."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u], dim=0)
    return sum(w[:, j] * padded[j:j + u.shape[0]] for j in range(taps))


def rotate_halves(x, positions, rot):
    """``x [T, heads, D]``: channel ``i < dims/2`` turns together with channel ``i + dims/2`` by
    ``position * base^(-2i/dims)``; the channels from ``dims`` on pass unchanged."""
    dims, base = int(rot["dims"]), float(rot["base"])
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=F)
    angle = (torch.tensor(list(positions), dtype=F).unsqueeze(-1) * f).unsqueeze(1)      # [T, 1, half]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(angle) - v * torch.sin(angle), v * torch.cos(angle) + u * torch.sin(angle),
                      x[..., dims:]], dim=-1)


def visible(i, j, size):
    """Whether the query at position ``i`` sees the key at position ``j`` (``size`` None: no chunks)."""
    return j <= i and (size is None or i // size == j // size)


def chunked_sink_attention(q, k, v, scale, size, sink, q_positions=None):
    """``q [T, H, D]``, ``k [S, G, D]``, ``v [S, G, E]``; softmax over the visible keys with
    ``exp(sink_h)`` in the denominator."""
    T, H, _ = q.shape
    S, G, E = v.shape
    if q_positions is None:
        q_positions = list(range(S - T, S))
    out = torch.zeros(T, H, E, dtype=q.dtype)
    for t, i in enumerate(q_positions):
        lo = next(j for j in range(i + 1) if visible(i, j, size)) if size is None else (i // size) * size
        for hd in range(H):
            g = hd // (H // G)
            s = (k[lo:i + 1, g] @ q[t, hd]) * scale
            m = torch.maximum(s.max(), sink[hd])
            p = torch.exp(s - m)
            out[t, hd] = (p / (p.sum() + torch.exp(sink[hd] - m))) @ v[lo:i + 1, g]
    return out


def attention_mixer(h, p, m, eps):
    """The left half of the 'parallel' mixer."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ p[n].T + p[n + ".b"], p[n + ".conv"]) for n in ("q", "k", "v"))
    q, k, v = q.view(T, H, D), k.view(T, G, D), v.view(T, G, E)
    if m.get("rot"):
        q, k = rotate_halves(q, range(T), m["rot"]), rotate_halves(k, range(T), m["rot"])
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    o = chunked_sink_attention(q, k, v, m["scale"], (m.get("mask") or {}).get("size"), p["sink"])
    o = o.reshape(T, H * E) * torch.sigmoid(h @ p["g"].T)
    return o @ p["o"].T + p["o.b"]


# ------------------------------------------------------------ recurrent mixers
def bonus_rule(r, k, v, w, u, state=None):
    """``r, k, w [T, H, D]``, ``v [T, H, E]``, ``u [H, D]``.  Per head::

        o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t ;  S_t = diag(w_t) S_(t-1) + k_t v_t^T

    Returns ``o [T, H, E]`` and the last state ``[H, D, E]``."""
    T, H, D = r.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=r.dtype) if state is None else state.clone()
    out = torch.zeros(T, H, v.shape[-1], dtype=r.dtype)
    for t in range(T):
        kv = k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        out[t] = ((S + u.unsqueeze(-1) * kv) * r[t].unsqueeze(-1)).sum(1)
        S = w[t].unsqueeze(-1) * S + kv
    return out, S


def time_mixer(h, p, m, eps):
    """The right half of the 'parallel' mixer."""
    T = h.shape[0]
    H, D = m["heads"], m["dim"]
    mixed = {s: token_shift(h, p["mu." + s]) for s in "rkvgw"}
    r, k, v = ((mixed[s] @ p[s].T).view(T, H, D) for s in "rkv")
    w = torch.exp(-torch.exp(torch.tanh(mixed["w"] @ p["w1"].T) @ p["w2"].T + p["w0"])).view(T, H, D)
    o, _ = bonus_rule(r, k, v, w, p["u"])
    o = unit_rms(o, eps).reshape(T, H * D) * p["norm"] * silu(mixed["g"] @ p["g"].T)
    return o @ p["o"].T


def parallel_mixer(h, p, m, eps):
    left = attention_mixer(h, sub(p, "left."), m["left"], eps)
    right = time_mixer(h, sub(p, "right."), m["right"], eps)
    return 0.5 * (rms_norm(left, p["left.out"], eps) + rms_norm(right, p["right.out"], eps))


def decay_rule(q, k, v, a, state=None):
    """``S_t = diag(a_t) S_(t-1) + k_t v_t^T ; o_t = S_t^T q_t`` per head."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = a[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out, S


def gla_mixer(h, p, m, eps):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = (h @ p["q"].T).view(T, H, D) * D ** -0.5
    k = (h @ p["k"].T).view(T, H, D)
    v = (h @ p["v"].T).view(T, H, E)
    z = (h @ p["a1"].T) @ p["a2"].T + p["a2.b"]
    a = (torch.sigmoid(z) ** (1.0 / m["tau"])).view(T, H, D)
    o, _ = decay_rule(q, k, v, a)
    o = rms_norm(o, p["norm"], eps).reshape(T, H * E) * silu(h @ p["g"].T)
    return o @ p["o"].T


def matrix_memory(q, k, v, i, f, state=None):
    """``q, k [T, H, D]``, ``v [T, H, E]``, log gates ``i, f [T, H]``.  With a running maximum ``m``
    (0 at the start)::

        m_t = max(f_t + m_(t-1), i_t)
        S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T,   n_t likewise with k_t alone
        o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)

    Returns ``o`` and the last ``(S, n, m)``."""
    T, H, D = q.shape
    E = v.shape[-1]
    S, n, m = state if state is not None else (torch.zeros(H, D, E, dtype=q.dtype), torch.zeros(H, D, dtype=q.dtype),
                                               torch.zeros(H, dtype=q.dtype))
    out = torch.zeros(T, H, E, dtype=q.dtype)
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        keep, take = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        m = new
        S = keep.view(H, 1, 1) * S + take.view(H, 1, 1) * k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        n = keep.view(H, 1) * n + take.view(H, 1) * k[t]
        size = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t].unsqueeze(-1)).sum(1) / size.unsqueeze(-1)
    return out, (S, n, m)


def mlstm_mixer(h, p, m, eps):
    T = h.shape[0]
    H, D, E, cap = m["heads"], m["dim"], m["vdim"], float(m["gate_cap"])
    q = (h @ p["q"].T).view(T, H, D) * D ** -0.5
    k = (h @ p["k"].T).view(T, H, D)
    v = (h @ p["v"].T).view(T, H, E)
    i = cap * torch.tanh((h @ p["i"].T + p["i.b"]) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((h @ p["f"].T + p["f.b"]) / cap))
    o, _ = matrix_memory(q, k, v, i, f)
    o = unit_rms(o, eps).reshape(T, H * E) * p["norm"] * torch.sigmoid(h @ p["g"].T)
    return o @ p["o"].T


# --------------------------------------------------------------------- model
MIXERS = {"parallel": parallel_mixer, "gla": gla_mixer, "mlstm": mlstm_mixer}


def sub(tensors, prefix):
    return {n[len(prefix):]: t for n, t in tensors.items() if n.startswith(prefix)}


def forward(config, tensors, tokens, return_layers=False):
    """Logits ``[T, vocab]`` of one sequence (and the stream after every layer)."""
    t = {n: x.to(F) for n, x in tensors.items()}
    eps = float(config["norm"]["eps"])
    x = t["embed"][torch.tensor(list(tokens))]
    after = []
    for i, layer in enumerate(config["layers"]):
        p = sub(t, f"l{i}.")
        h = token_shift(x, p["shift"])
        x = x + rms_norm(MIXERS[layer["type"]](h, sub(p, "mix."), layer["mixer"], eps), p["norm1"], eps)
        if layer.get("mlp") is not None:
            x = x + rms_norm(poly_mlp(x, p["mlp.up"], p["mlp.down"], p["mlp.act"], eps), p["norm2"], eps)
        after.append(x)
    logits = rms_norm(x, t["final.norm"], eps) @ t["head"].T
    return (logits, torch.stack(after)) if return_layers else logits


def greedy(config, tensors, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(forward(config, tensors, tokens)[-1].argmax()))
    return tokens[len(prompt):]
