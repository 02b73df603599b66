"""Molotar as data: configuration -> ``ModelSpec``.

A stack of layers that norm the SUM behind each sublayer, ``x = norm1(alpha * x + mixer(x))``, then (where the
layer has one) ``x = norm2(alpha * x + feed_forward(x))``, all RMS norms.  The mixer is grouped-query attention
through a sliding window (a norm over the whole query and key projections, halves of a head turned by
position with slow waves stretched, a one in the softmax's denominator, a gate per head; perhaps on an
earlier layer's keys and values), or a recurrence of single numbers with block-diagonal gates behind a short
convolution, times a gelu branch.  The feed-forward is a mixture of clamped experts behind a sigmoid router
that chooses among the best groups.  The embedding adds a row of a hashed table of token pairs to the
scaled token vector; the head is a matrix of its own behind a last norm.

Tensor names: ``embed``, ``bigram``, ``final.norm``, ``head``, and per layer ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.mix.{q,k,v,q.norm,k.norm,g,o}`` or ``l<i>.mix.{y,y.b,x,x.b,conv,conv.b,ra,ra.b,ri,ri.b,lam,o}``,
``l<i>.mlp.{router,e<j>.gate,e<j>.up,e<j>.down}``.
"""
from __future__ import annotations

import dataclasses

from ..config.molotar import MolotarConfig
from ..config.registry import register_architecture
from ..config.spec import BlockSpec, ModelSpec, PartSpec, ScheduleEntry

DECAY_SCALE = 8.0                       # the recurrence's decay: log a = -8 r softplus(lambda)
EXPERT_SLOPE, EXPERT_SHIFT = 1.702, 1.0      # of the experts' clamped pair
SHARE_EPS = 1e-20                       # added to the sum of the chosen scores


def _attention(a, width, eps, p):
    position = None
    if a.rot is not None and a.rot.dims:
        position = PartSpec("rope", params=dict(dim=a.dim, rotary_dim=a.rot.dims, theta=a.rot.base,
                                                padded_dim=a.dim + a.dim % 2,
                                                scaling=None if a.rot.scaling is None else dataclasses.asdict(a.rot.scaling)))
    names = dict(q_weight="q", q_norm="q.norm", gate_weight="g", o_weight="o")
    if a.kv_from is None:
        names.update(k_weight="k", v_weight="v", k_norm="k.norm")
    return PartSpec("windowed_sink_attention",
                    params=dict(hidden_size=width, num_heads=a.heads, num_kv_heads=a.kv_heads, key_dim=a.dim, value_dim=a.vdim,
                                scale=a.scale, window=a.window, sink=False, plus_one=True, qk_norm="whole", norm_eps=eps,
                                own_kv=a.kv_from is None, position=position, output_gate="sigmoid"),
                    tensors={role: p + name for role, name in names.items()})


def _recurrence(r, width, p):
    names = dict(y_weight="y", y_bias="y.b", x_weight="x", x_bias="x.b", conv="conv", conv_bias="conv.b", r_weight="ra",
                 r_bias="ra.b", i_weight="ri", i_bias="ri.b", decay="lam", o_weight="o")
    return PartSpec("gated_linear_recurrence",
                    params=dict(hidden_size=width, width=r.width, blocks=r.blocks, conv_taps=r.conv, decay_scale=DECAY_SCALE),
                    tensors={role: p + name for role, name in names.items()})


def _experts(f, width, p):
    return PartSpec("routed_experts",
                    params=dict(hidden_size=width, expert_size=f.ff, num_experts=f.experts, top=f.top, scale=f.scale,
                                groups=f.groups, groups_keep=f.groups_keep, correction=False, scoring="sigmoid",
                                expert_form="clamped", expert_constants=(f.limit, EXPERT_SLOPE, EXPERT_SHIFT),
                                group_score="top2", share_eps=SHARE_EPS),
                    tensors=dict(router=p + "router", expert_gate=p + "e{}.gate", expert_up=p + "e{}.up",
                                 expert_down=p + "e{}.down"))


def build_molotar_spec(cfg: MolotarConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps
    norm = lambda name: PartSpec("rmsnorm", params=dict(size=w, eps=eps), tensors=dict(weight=name))
    blocks, schedule = [], []
    for i, l in enumerate(cfg.layers):
        p = f"l{i}."
        mixer = _attention(l.mixer, w, eps, p + "mix.") if l.type == "attention" else _recurrence(l.mixer, w, p + "mix.")
        parts = dict(mixer=mixer, norm1=norm(p + "norm1"))
        if l.mlp is not None:
            parts.update(feed_forward=_experts(l.mlp, w, p + "mlp."), norm2=norm(p + "norm2"))
        blocks.append(BlockSpec("post_norm", parts=parts, params=dict(hidden_size=w, alpha=cfg.alpha)))
        schedule.append(ScheduleEntry(i, cache_of=getattr(l.mixer, "kv_from", None)))
    b = cfg.bigram
    spec = ModelSpec(
        architecture=MolotarConfig.ARCHITECTURE, vocab_size=cfg.vocab, hidden_size=w,
        max_positions=MolotarConfig.MAX_POSITIONS,
        embedding=PartSpec("pair_hash_embedding",
                           params=dict(vocab_size=cfg.vocab, hidden_size=w, scale=cfg.embedding_scale,
                                       buckets=b.buckets if b else 0, mul_prev=b.mul_prev if b else 0,
                                       mul_cur=b.mul_cur if b else 0),
                           tensors=dict(weight="embed", pairs="bigram")),
        blocks=tuple(blocks), schedule=tuple(schedule), final_norm=norm("final.norm"),
        head=PartSpec("linear_head", params=dict(vocab_size=cfg.vocab, hidden_size=w), tensors=dict(weight="head")),
        eos_token_ids=tuple(cfg.eos_token_ids))
    spec.validate()
    return spec


register_architecture(MolotarConfig.ARCHITECTURE, MolotarConfig, build_molotar_spec, replace=True)
