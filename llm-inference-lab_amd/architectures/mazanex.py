"""Mazanex as data: configuration -> ``ModelSpec``.

A stack of layers that norm each sublayer's OUTPUT, ``x += norm1(mixer(h))`` with ``h`` the stream's row
mixed with the row before it (a token shift), then (where the layer has one) ``x +=
norm2(feed_forward(x))``, all RMS norms.  The mixer is a matrix memory with exponential gates, gated
linear attention, or a pair of mixers on one input: grouped-query attention over chunks of
positions (a sink, short convolutions behind the projections, halves of a head turned by position,
heads of unit root mean square, a gate per channel), and time mixing (a recurrent state with a
bonus for the current token); half the sum of both results, each normed.  The feed-forward's
activation is a cubic in the first product's numbers, every power over its own root mean square.
The head is a matrix of its own behind a last norm.

Tensor names: ``embed``, ``head``, ``final.norm``, and per layer ``l<i>.norm1``, ``.norm2``, ``.shift``,
``l<i>.mix.<role>`` (``l<i>.mix.left.<role>`` / ``.right.<role>`` in a parallel layer), ``l<i>.mlp.up`` /
``.down`` / ``.act``.
"""
from __future__ import annotations

import dataclasses

from ..config.mazanex import MazanexConfig
from ..config.registry import register_architecture
from ..config.spec import BlockSpec, ModelSpec, PartSpec, ScheduleEntry


def _attention(a, width, eps, p):
    position = None
    if a.rot is not None and a.rot.dims:
        position = PartSpec("rope", params=dict(dim=a.dim, rotary_dim=a.rot.dims, theta=a.rot.base, padded_dim=a.dim + a.dim % 2))
    names = dict(q_weight="q", k_weight="k", v_weight="v", o_weight="o", q_bias="q.b", k_bias="k.b", v_bias="v.b", o_bias="o.b",
                 sink="sink", gate_weight="g")
    if a.conv:
        names.update(q_conv="q.conv", k_conv="k.conv", v_conv="v.conv")
    return PartSpec(
        "windowed_sink_attention",
        params=dict(hidden_size=width, num_heads=a.heads, num_kv_heads=a.kv_heads, key_dim=a.dim, value_dim=a.vdim,
                    scale=a.scale, chunk=a.chunk, sink=True, qk_norm="head", norm_eps=eps, position=position, qkv_bias=True,
                    out_bias=True, output_gate="channels", conv_taps=a.conv),
        tensors={role: p + name for role, name in names.items()})


def _time_mix(r, width, eps, p):
    names = dict(mix_r="mu.r", mix_k="mu.k", mix_v="mu.v", mix_g="mu.g", mix_w="mu.w", r_weight="r", k_weight="k", v_weight="v",
                 gate_weight="g", decay_down="w1", decay_up="w2", decay_bias="w0", bonus="u", out_norm="norm", o_weight="o")
    return PartSpec("time_mix_attention",
                    params=dict(hidden_size=width, num_heads=r.heads, key_dim=r.dim, norm_eps=eps, gate="silu"),
                    tensors={role: p + name for role, name in names.items()})


def _gla(r, width, eps, p):
    names = dict(q_weight="q", k_weight="k", v_weight="v", gate_weight="g", o_weight="o", out_norm="norm", decay_down="a1",
                 decay_up="a2", decay_bias="a2.b")
    return PartSpec("gated_linear_attention",
                    params=dict(hidden_size=width, num_heads=r.heads, key_dim=r.dim, value_dim=r.vdim, decay_rank=None,
                                tau=r.tau, norm_eps=eps),
                    tensors={role: p + name for role, name in names.items()})


def _memory(r, width, eps, p):
    names = dict(q_weight="q", k_weight="k", v_weight="v", gate_weight="g", o_weight="o", out_norm="norm", i_weight="i",
                 i_bias="i.b", f_weight="f", f_bias="f.b")
    return PartSpec("matrix_memory_attention",
                    params=dict(hidden_size=width, num_heads=r.heads, key_dim=r.dim, value_dim=r.vdim, gate_cap=r.gate_cap,
                                norm_eps=eps, gate="sigmoid"),
                    tensors={role: p + name for role, name in names.items()})


def build_mazanex_spec(cfg: MazanexConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps
    norm = lambda name: PartSpec("rmsnorm", params=dict(size=w, eps=eps), tensors=dict(weight=name))
    blocks = []
    for i, l in enumerate(cfg.layers):
        p = f"l{i}."
        if l.type == "mlstm":
            mixer = _memory(l.recurrent, w, eps, p + "mix.")
        elif l.type == "gla":
            mixer = _gla(l.recurrent, w, eps, p + "mix.")
        else:
            mixer = PartSpec("parallel",
                             params=dict(left=_attention(l.left, w, eps, p + "mix.left."),
                                         right=_time_mix(l.right, w, eps, p + "mix.right."), left_scale=0.5,
                                         right_scale=0.5, norm_eps=eps, hidden_size=w),
                             tensors=dict(left_norm=p + "mix.left.out", right_norm=p + "mix.right.out"))
        parts = dict(mixer=mixer, norm1=norm(p + "norm1"))
        if l.mlp is not None:
            parts.update(
                feed_forward=PartSpec("dense", params=dict(hidden_size=w, intermediate_size=l.mlp.ff,
                                                           activation="poly_norm", norm_eps=eps),
                                      tensors=dict(up_weight=p + "mlp.up", down_weight=p + "mlp.down",
                                                   act_coef=p + "mlp.act")),
                norm2=norm(p + "norm2"))
        blocks.append(BlockSpec("sublayer_norm", parts=parts,
                                params=dict(hidden_size=w, token_shift=True, tensors=dict(shift=p + "shift"))))
    sizes = dict(vocab_size=cfg.vocab, hidden_size=w)
    spec = ModelSpec(
        architecture=MazanexConfig.ARCHITECTURE, vocab_size=cfg.vocab, hidden_size=w,
        max_positions=MazanexConfig.MAX_POSITIONS,
        embedding=PartSpec("token_embedding", params=sizes, tensors=dict(weight="embed")),
        blocks=tuple(blocks), schedule=tuple(ScheduleEntry(i) for i in range(len(blocks))),
        final_norm=norm("final.norm"), head=PartSpec("linear_head", params=sizes, tensors=dict(weight="head")),
        eos_token_ids=tuple(cfg.eos_token_ids))
    spec.validate()
    return spec


def mazanex_random_init(cfg: MazanexConfig, expected, seed: int, dtype):
    """Random-weights mode: a size that the configuration leaves to the tensors' shapes takes
    the configuration class's default."""
    from ..weights.random_init import random_tensors
    rank = MazanexConfig.DEFAULT_DECAY_RANK
    filled = {name: dataclasses.replace(s, shape=tuple(rank if d is None else d for d in s.shape))
              for name, s in expected.items()}
    return random_tensors(filled, seed, dtype)


register_architecture(MazanexConfig.ARCHITECTURE, MazanexConfig, build_mazanex_spec, random_init=mazanex_random_init,
                      replace=True)
