"""Mixers with a recurrent state instead of a cache of keys and values."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..weights.loader import TensorSpec, MATRIX, VECTOR, INIT_NORM
from .base import Mixer, NormedInput, PendingSums, project_normed
from .registry import register_part


def pad_heads(x, heads: int, channels: int, laid: int):
    """Rows (or entries) of ``heads`` heads of ``channels`` channels -> of ``laid``, zeros behind."""
    if channels == laid:
        return x
    per_head = x.unflatten(0, (heads, channels))
    zeros = torch.zeros((heads, laid - channels) + tuple(x.shape[1:]), dtype=x.dtype, device=x.device)
    return torch.cat([per_head, zeros], dim=1).flatten(0, 1)


class ScanMixer(Mixer):
    """What the mixers share whose state ``S [key_dim, value_dim]`` per head follows ``S_t = decay_t * S_(t-1) + k_t
    v_t^T``: the state's slots, the scan over a step's rows (whole, or long portions in chunks side by
    side) and room for it.  ``value_dim`` is a value head as the kernels see it: a multiple of 8 (the
    products' inner sizes), zeros behind the file's ``file_value_dim`` channels."""

    writes_output = True
    keeps_launches = True

    def _set_sizes(self, hidden_size, num_heads, key_dim, value_dim):
        self.hidden_size, self.num_heads, self.key_dim = int(hidden_size), int(num_heads), int(key_dim)
        self.file_value_dim = int(value_dim)
        self.value_dim = (self.file_value_dim + 7) // 8 * 8

    @property
    def qk_size(self):
        return self.num_heads * self.key_dim

    @property
    def v_size(self):
        return self.num_heads * self.value_dim

    def _values(self, x):
        return pad_heads(x, self.num_heads, self.file_value_dim, self.value_dim)

    def _check_sizes(self, ops, dtype, name):
        ops.check_linear_attention_sizes(self.num_heads, self.key_dim, self.value_dim)
        ops.check_product_sizes(self.hidden_size, dtype, f"{name} projections (hidden size)")
        ops.check_product_sizes(self.v_size, dtype, f"{name} output projection (heads * value size)")

    def state_spec(self):
        return {"s": ((self.num_heads, self.key_dim, self.value_dim), torch.float32)}

    def _min_chunk(self) -> int:
        rules = getattr(self.ops, "rules", None)
        return int(getattr(rules, "scan_min_chunk", 16))

    def _scan(self, proj, off_q, off_k, off_v, decay, q_scale, state, ctx, bonus=None, memory=None):
        """The outputs of this step's rows in pieces ``[rows, heads, slices, value_dim]``.  ``memory``: ``(keep,
        take, normaliser's state)``; the normaliser's pieces ``[rows, heads, slices]`` come back beside them."""
        ops, rows = self.ops, proj.shape[0]
        heads, d, e = self.num_heads, self.key_dim, self.value_dim
        slices = ops.gla_slices(d)
        parts = ctx.scratch("linear_attention.parts", (rows, heads, slices, e), torch.float32)
        # room for the chunks of a long portion: at most rows / (smallest chunk) + requests
        most = rows // max(1, self._min_chunk()) + ctx.max_reqs
        chunk_state = ctx.scratch("linear_attention.chunk_state", (most, heads, d, e), torch.float32)
        chunk_decay = ctx.scratch("linear_attention.chunk_decay", (most, heads, d), torch.float32)
        norm_parts = chunk_norm = None
        if memory is not None:
            norm_parts = ctx.scratch("linear_attention.norm_parts", (rows, heads, slices), torch.float32)
            chunk_norm = ctx.scratch("linear_attention.chunk_norm", (most, heads, d), torch.float32)

        def scan():
            # (how many requests the step has and how long the longest portion is are read when
            # the launch is made, also when it is made again from a kept sequence of calls)
            pick = getattr(ops, "gla_scan_chunk", None)
            chunk = pick(rows, ctx.max_q_len, heads, e) if pick is not None else 0
            kind = {}
            if bonus is not None:
                kind["bonus"] = bonus
            if memory is not None:
                kind["memory"] = tuple(memory) + (norm_parts, chunk_norm if chunk else None)
            ops.gla_scan(proj, off_q, off_k, off_v, decay, q_scale, heads, d, e, state, ctx.all_q_start, ctx.all_req_rows,
                         ctx.n_reqs, parts, chunk, chunk_state if chunk else None, chunk_decay if chunk else None, **kind)
        self._live(scan)
        return parts if memory is None else (parts, norm_parts)

    def _live(self, launch):
        live = getattr(self.ops, "live", None)
        if live is not None:
            live(launch)
        else:
            launch()

    def _recur(self, proj, ctx, entry, off, weight, eps, gate, q_scale, many_rows, in_chunks, rank=0, **kind):
        """From the projections to the gated output ``[rows, heads * value_dim]`` (compute dtype).  Where every
        request of the step brings one row and the sizes allow it: one launch; where some bring many:
        ``in_chunks(out)``; else ``many_rows(out)``.
        ``off``: the columns of query, key, value and gate."""
        ops = self.ops
        mixed = ctx.scratch("linear_attention.out", (proj.shape[0], self.v_size), self.dtype)
        takes = getattr(ops, "recurrent_row_takes", None)
        fits = takes is not None and takes(self.key_dim, self.value_dim, rank)
        count = self.file_value_dim if self.file_value_dim != self.value_dim else 0

        def launch():        # (how many rows the requests bring is not a matter of the number of rows)
            if fits and ctx.n_rows == ctx.n_reqs:
                ops.recurrent_row(proj, *off, q_scale, self.num_heads, self.key_dim, self.value_dim, entry.state["s"],
                                  ctx.all_q_start, ctx.all_req_rows, ctx.n_reqs, weight, eps, gate, count, mixed, **kind)
                return
            chunked = getattr(ops, "chunk_scan_takes", None)
            if chunked is not None and chunked(ctx.max_q_len, self.key_dim, self.value_dim):
                in_chunks(mixed)
            else:
                many_rows(mixed)
        self._live(launch)
        return mixed

    def _in_chunks(self, proj, ctx, entry, off, logs, weight, eps, gate, q_scale, mixed, bonus=None, memory=None):
        """Long portions: chunks of rows side by side on the matrix cores, from the logarithms of the decays
        to the gated output.  ``memory``: ``(take, maxima)``."""
        heads, d, e = self.num_heads, self.key_dim, self.value_dim
        most = proj.shape[0] // self.ops.CHUNK_SCAN_ROWS + ctx.max_reqs
        chunk_state = ctx.scratch("linear_attention.chunk_state", (most, heads, d, e), torch.float32)
        chunk_decay = ctx.scratch("linear_attention.chunk_decay", (most, heads, d), torch.float32)
        kind = {}
        if bonus is not None:
            kind["bonus"] = bonus
        if memory is not None:
            chunk_norm = ctx.scratch("linear_attention.chunk_norm", (most, heads, d), torch.float32)
            kind["memory"] = (memory[0], entry.state["n"], memory[1], chunk_norm)
        self.ops.chunk_scan(proj, *off, q_scale, heads, d, e, logs, entry.state["s"], ctx.all_q_start, ctx.all_req_rows,
                            ctx.n_reqs, chunk_state, chunk_decay, weight, eps, gate,
                            self.file_value_dim if self.file_value_dim != self.value_dim else 0, mixed, **kind)

    def _output(self, parts, weight, eps, proj, off_gate, gate, mixed, **memory):
        if self.file_value_dim != self.value_dim:      # (the heads' norm is over the file's channels)
            memory["norm_count"] = self.file_value_dim
        self.ops.gla_output(parts, self.num_heads, self.key_dim, self.value_dim, weight, eps, proj, off_gate, mixed, gate,
                            **memory)

    def forward(self, h, residual, ctx, entry):
        if isinstance(h, NormedInput) and not self.takes_normed_input:
            h = h.tensor()
        y = ctx.scratch("linear_attention.sum", (1,) + tuple(residual.shape), torch.float32)
        self.forward_into(h, y[0], ctx, entry)
        self.ops.add_pending(residual, PendingSums(y, 1))

    def kernel_libraries(self):
        return [("linear_attention", None)]


class GatedLinearAttention(ScanMixer):
    """Linear attention with a decay per key channel and a matrix-valued state per head.

    With ``D = key_dim`` and ``E = value_dim``: ``q = Wq h * q_scale`` (``q_scale`` defaults to
    ``D ** -0.5``), ``k = Wk h`` (``heads x D``), ``v = Wv h`` (``heads x E``); decays ``a =
    sigmoid(W2 (W1 h) + b2) ** (1 / tau)`` (``heads x D``, through a projection of rank
    ``decay_rank``); per head, token by token::

        S_t = diag(a_t) S_(t-1) + k_t v_t^T          (S is D x E, zero at a sequence's start)
        o_t = S_t^T q_t

    then every head's ``o_t`` is divided by its root mean square over ``E`` (``eps`` inside the
    root) and multiplied by one weight of size ``E`` that all heads share, the heads are put
    side by side, multiplied by ``silu(Wg h)`` and projected by ``Wo``.

    The state lives in float32 in one slot per request (``state_spec``) and is carried from
    step to step; the decays, the recurrence and the norm are float32 throughout, and the
    projections reach them unrounded (32-bit sums of the matrix products)."""

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, decay_rank: int,
                 tau: float, tensors: Dict[str, str], norm_eps: float = 1e-6, q_scale: Optional[float] = None):
        super().__init__(tensors)
        self._set_sizes(hidden_size, num_heads, key_dim, value_dim)
        # (None: the rank is whatever the model file's decay tensors have)
        self.decay_rank = None if decay_rank is None else int(decay_rank)
        self.tau, self.norm_eps = float(tau), float(norm_eps)
        if self.tau <= 0:
            raise ValueError(f"tau must be positive, got {tau}")
        self.q_scale = float(q_scale) if q_scale is not None else self.key_dim ** -0.5
        self.w_in = self.w_o = self.w_decay = self.b_decay = self.norm_weight = None

    def tensor_specs(self):
        t, w = self.tensor_names, self.hidden_size
        return {
            t["q_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["k_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["v_weight"]: TensorSpec((self.num_heads * self.file_value_dim, w), MATRIX),
            t["gate_weight"]: TensorSpec((self.num_heads * self.file_value_dim, w), MATRIX),
            t["o_weight"]: TensorSpec((w, self.num_heads * self.file_value_dim), MATRIX),
            t["out_norm"]: TensorSpec((self.file_value_dim,), VECTOR, INIT_NORM),
            t["decay_down"]: TensorSpec((self.decay_rank, w), MATRIX),
            t["decay_up"]: TensorSpec((self.qk_size, self.decay_rank), MATRIX),
            t["decay_bias"]: TensorSpec((self.qk_size,), VECTOR),
        }

    def bind(self, tensors, ops, dtype):
        super().bind(tensors, ops, dtype)
        self._check_sizes(ops, dtype, "linear attention")
        t = self.tensor_names
        rank = int(tensors[t["decay_down"]].shape[0])
        if int(tensors[t["decay_up"]].shape[1]) != rank:
            raise ValueError(f"{t['decay_down']} has {rank} rows but {t['decay_up']} has "
                             f"{int(tensors[t['decay_up']].shape[1])} columns: the two factors of the decay "
                             f"projection do not fit")
        self.decay_rank = rank
        # one product for q, k, v, the gate and the low-rank input of the decays
        self.offsets = {}
        at = 0
        rows = []
        for role in ("q_weight", "k_weight", "v_weight", "gate_weight", "decay_down"):
            self.offsets[role] = at
            rows.append(self._values(tensors[t[role]]) if role in ("v_weight", "gate_weight") else tensors[t[role]])
            at += rows[-1].shape[0]
        self.in_size = at
        self.w_in = ops.prepare_weight(torch.cat(rows, dim=0).contiguous())
        self.w_o = ops.prepare_weight(self._values(tensors[t["o_weight"]].t()).t().contiguous())
        # the second factor of the decays is applied in float32, inside the decay kernel
        self.w_decay = tensors[t["decay_up"]].float().contiguous()
        self.b_decay = tensors[t["decay_bias"]].float().contiguous()
        self.norm_weight = pad_heads(tensors[t["out_norm"]].float(), 1, self.file_value_dim, self.value_dim).contiguous()

    def forward_into(self, h, out, ctx, entry):
        ops, rows, o = self.ops, h.shape[0], self.offsets
        proj = ctx.scratch("linear_attention.proj", (rows, self.in_size), torch.float32)
        ops.linear_logits(h, self.w_in, proj)
        off = [o[role] for role in ("q_weight", "k_weight", "v_weight", "gate_weight")]
        decay = ctx.scratch("linear_attention.decay", (rows, self.qk_size), torch.float32)

        def many_rows(mixed):
            ops.gla_decay(proj[:, o["decay_down"]:], self.decay_rank, self.w_decay, self.b_decay, self.tau, decay)
            parts = self._scan(proj, *off[:3], decay, self.q_scale, entry.state["s"], ctx)
            self._output(parts, self.norm_weight, self.norm_eps, proj, off[3], "silu", mixed)

        def in_chunks(mixed):
            ops.gla_decay(proj[:, o["decay_down"]:], self.decay_rank, self.w_decay, self.b_decay, self.tau, decay, as_log=True)
            self._in_chunks(proj, ctx, entry, off, decay, self.norm_weight, self.norm_eps, "silu", self.q_scale, mixed)
        mixed = self._recur(proj, ctx, entry, off, self.norm_weight, self.norm_eps, "silu", self.q_scale, many_rows,
                            in_chunks, self.decay_rank,
                            decay=(o["decay_down"], self.decay_rank, self.w_decay, self.b_decay, "sigmoid", self.tau))
        ops.linear_logits(mixed, self.w_o, out)

    def weight_bytes(self):
        return sum(w.numel() * w.element_size()
                   for w in (self.w_in, self.w_o, self.w_decay, self.b_decay, self.norm_weight) if w is not None)


class DeltaRuleAttention(Mixer):
    """A recurrent mixer whose matrix-valued state forgets along the current key before it
    learns the new pair (a generalised delta rule).

    With ``D = key_dim`` and ``E = value_dim`` (default ``D``): ``r = Wr h``, ``k = Wk h`` (``heads x
    D``), ``v = Wv h`` (``heads x E``); decays ``w = exp(-decay_scale * sigmoid(W2 tanh(W1 h) + w0))``
    and removal rates ``a = sigmoid(Wa h + ba)``, both per head and key channel; per head, token by
    token, with the unit key ``u = k / sqrt(|k|^2 + key_eps)``::

        S_t = diag(w_t) S_(t-1) - (a_t * u_t) (u_t^T S_(t-1)) + k_t v_t^T     (S is D x E; decay and removal
        o_t = S_t^T r_t                                                        both act on S_(t-1))

    then every head's ``o_t`` is divided by its root mean square over ``E`` (``norm_eps`` inside the
    root), the heads are put side by side, multiplied by a weight of all heads' size and by
    ``sigmoid(Wg h)`` (``gate="silu"``: by ``silu``), and projected by ``Wo``.

    The state lives in float32 in one slot per request (``state_spec``), zero at a sequence's
    start, and is carried from step to step; decays, rates, the unit key, the recurrence and the
    norm are float32 throughout, and the projections reach them unrounded (the 32-bit sums of the
    matrix products).  ``decay_rank`` None: the rank of the decay projection is whatever the model
    file's tensors have.

    Tensor roles: ``r_weight, k_weight, v_weight, gate_weight, rate_weight, rate_bias, decay_down,
    decay_up, decay_bias, out_norm, o_weight``."""

    writes_output = True
    takes_normed_input = True
    keeps_launches = True
    DEFAULT_DECAY_SCALE = 0.6065306597126334      # exp(-1/2)

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, tensors: Dict[str, str],
                 value_dim: Optional[int] = None, decay_rank: Optional[int] = None,
                 decay_scale: float = DEFAULT_DECAY_SCALE, key_eps: float = 1e-6, norm_eps: float = 1e-6,
                 gate: str = "sigmoid"):
        super().__init__(tensors)
        self.hidden_size, self.num_heads, self.key_dim = int(hidden_size), int(num_heads), int(key_dim)
        self.file_value_dim = self.key_dim if value_dim is None else int(value_dim)      # as the model file has it
        # (the products' inner sizes are multiples of 8: zeros behind a head's value channels)
        self.value_dim = (self.file_value_dim + 7) // 8 * 8
        self.decay_rank = None if decay_rank is None else int(decay_rank)
        self.decay_scale, self.key_eps, self.norm_eps = float(decay_scale), float(key_eps), float(norm_eps)
        if gate not in ("sigmoid", "silu"):
            raise ValueError(f"the output gate is 'sigmoid' or 'silu', got {gate!r}")
        self.gate = gate
        self.w_in = self.w_o = self.w_decay = self.b_decay = self.b_rate = self.norm_weight = None
        self.offsets = {}
        self.in_size = 0

    @property
    def qk_size(self):
        return self.num_heads * self.key_dim

    @property
    def v_size(self):
        return self.num_heads * self.value_dim

    def tensor_specs(self):
        t, w = self.tensor_names, self.hidden_size
        file_v = self.num_heads * self.file_value_dim
        return {
            t["r_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["k_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["v_weight"]: TensorSpec((file_v, w), MATRIX),
            t["gate_weight"]: TensorSpec((file_v, w), MATRIX),
            t["rate_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["rate_bias"]: TensorSpec((self.qk_size,), VECTOR),
            t["decay_down"]: TensorSpec((self.decay_rank, w), MATRIX),
            t["decay_up"]: TensorSpec((self.qk_size, self.decay_rank), MATRIX),
            t["decay_bias"]: TensorSpec((self.qk_size,), VECTOR),
            t["out_norm"]: TensorSpec((file_v,), VECTOR, INIT_NORM),
            t["o_weight"]: TensorSpec((w, file_v), MATRIX),
        }

    def bind(self, tensors, ops, dtype):
        super().bind(tensors, ops, dtype)
        ops.check_delta_rule_sizes(self.num_heads, self.key_dim, self.value_dim)
        ops.check_product_sizes(self.hidden_size, dtype, "delta rule projections (hidden size)")
        ops.check_product_sizes(self.v_size, dtype, "delta rule output projection (heads * value size)")
        t = self.tensor_names
        rank = int(tensors[t["decay_down"]].shape[0])
        if int(tensors[t["decay_up"]].shape[1]) != rank:
            raise ValueError(f"{t['decay_down']} has {rank} rows but {t['decay_up']} has "
                             f"{int(tensors[t['decay_up']].shape[1])} columns: the two factors of the decay "
                             f"projection do not fit")
        self.decay_rank = rank

        def value_heads(x):
            return pad_heads(x, self.num_heads, self.file_value_dim, self.value_dim)
        # one product for r, k, v, the gate, the rates and the low-rank input of the decays
        self.offsets, at, rows = {}, 0, []
        for role in ("r_weight", "k_weight", "v_weight", "gate_weight", "rate_weight", "decay_down"):
            self.offsets[role] = at
            rows.append(value_heads(tensors[t[role]]) if role in ("v_weight", "gate_weight") else tensors[t[role]])
            at += rows[-1].shape[0]
        self.in_size = at
        self.w_in = ops.prepare_weight(torch.cat(rows, dim=0).contiguous())
        self.w_o = ops.prepare_weight(value_heads(tensors[t["o_weight"]].t()).t().contiguous())
        # the second factor of the decays is applied in float32, inside the gates' kernel
        self.w_decay = tensors[t["decay_up"]].float().contiguous()
        self.b_decay = tensors[t["decay_bias"]].float().contiguous()
        self.b_rate = tensors[t["rate_bias"]].float().contiguous()
        self.norm_weight = value_heads(tensors[t["out_norm"]].float()).contiguous()

    def _min_chunk(self) -> int:
        rules = getattr(self.ops, "rules", None)
        return int(getattr(rules, "scan_min_chunk", 16))

    def state_spec(self):
        return {"s": ((self.num_heads, self.key_dim, self.value_dim), torch.float32)}

    def forward_into(self, h, out, ctx, entry):
        ops, rows, o = self.ops, h.shape[0], self.offsets
        proj = ctx.scratch("delta_rule.proj", (rows, self.in_size), torch.float32)
        project_normed(ops, h, self.w_in, proj, self.dtype, self.hidden_size)
        decay = ctx.scratch("delta_rule.decay", (rows, self.qk_size), torch.float32)
        unit = ctx.scratch("delta_rule.unit", (rows, self.qk_size), torch.float32)
        removal = ctx.scratch("delta_rule.removal", (rows, self.qk_size), torch.float32)
        ops.delta_gates(proj, o["decay_down"], self.decay_rank, o["rate_weight"], o["k_weight"], self.w_decay,
                        self.b_decay, self.b_rate, self.decay_scale, self.key_eps, self.num_heads, self.key_dim, decay,
                        unit, removal)
        outs = ctx.scratch("delta_rule.outputs", (rows, self.num_heads, 1, self.value_dim), torch.float32)
        state = entry.state["s"]
        # room for the chunks of a long portion: at most rows / (smallest chunk) + requests
        most = rows // max(1, self._min_chunk()) + ctx.max_reqs
        chunk_state = ctx.scratch("delta_rule.chunk_state", (most, self.num_heads, self.key_dim, self.value_dim),
                                  torch.float32)
        chunk_trans = ctx.scratch("delta_rule.chunk_trans", (most, self.num_heads, self.key_dim, self.key_dim),
                                  torch.float32)

        def scan():
            # (how many requests the step has and how long the longest portion is are read when the
            # launch is made, also when it is made again from a kept sequence of calls)
            pick = getattr(ops, "delta_scan_chunk", None)
            chunk = (pick(rows, ctx.max_q_len, self.num_heads, self.key_dim, self.value_dim) if pick is not None else 0)
            ops.delta_scan(proj, o["r_weight"], o["k_weight"], o["v_weight"], decay, unit, removal, self.num_heads,
                           self.key_dim, self.value_dim, state, ctx.all_q_start, ctx.all_req_rows, ctx.n_reqs, outs,
                           chunk, chunk_state if chunk else None, chunk_trans if chunk else None)
        live = getattr(ops, "live", None)
        if live is not None:
            live(scan)
        else:
            scan()
        mixed = ctx.scratch("delta_rule.out", (rows, self.v_size), self.dtype)
        if self.file_value_dim != self.value_dim:      # (the heads' unit norm is over the file's channels)
            ops.gla_output(outs, self.num_heads, self.key_dim, self.value_dim, self.norm_weight, self.norm_eps, proj,
                           o["gate_weight"], mixed, self.gate, self.file_value_dim)
        else:
            ops.gla_output(outs, self.num_heads, self.key_dim, self.value_dim, self.norm_weight, self.norm_eps, proj,
                           o["gate_weight"], mixed, self.gate)
        ops.linear_logits(mixed, self.w_o, out)

    def forward(self, h, residual, ctx, entry):
        y = ctx.scratch("delta_rule.sum", (1,) + tuple(residual.shape), torch.float32)
        self.forward_into(h, y[0], ctx, entry)
        self.ops.add_pending(residual, PendingSums(y, 1))

    def kernel_libraries(self):
        return [("linear_attention", None)]

    def weight_bytes(self):
        return sum(w.numel() * w.element_size() for w in (self.w_in, self.w_o, self.w_decay, self.b_decay, self.b_rate,
                                                          self.norm_weight) if w is not None)


class TimeMixAttention(ScanMixer):
    """A recurrent mixer whose projections each read their own mix of the current token and the one
    before it, with a decay per key channel and a bonus for the current token.

    With ``h'`` the previous token's input (zeros for a sequence's first): each ``s`` of ``r, k, v, g, w``
    reads ``h + (h' - h) * mix_s``.  ``r, k`` (``heads x D``) and ``v`` (``heads x E``, default ``E = D``) are
    products with their mixes, the decays ``w = exp(-exp(W2 tanh(W1 mix_w) + w0))`` per head and key channel;
    per head, token by token, with the learned bonus ``u``::

        o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t
        S_t = diag(w_t) S_(t-1) + k_t v_t^T                  (S is D x E, zero at a sequence's start)

    then every head's ``o_t`` is divided by its root mean square over ``E`` (``norm_eps`` inside the root), the
    heads are put side by side, multiplied by a weight of all heads' size and by ``silu`` of the product
    of the ``g`` mix (``gate="sigmoid"``: its sigmoid), and projected by ``Wo``.

    State per request: ``S`` in float32 and the last input row (compute dtype).  Decays, bonus, the
    recurrence and the norm are float32, and the projections reach them unrounded; the mixes are
    rounded once.  The rank of the decay projection is whatever the model file's tensors have.

    Tensor roles: ``mix_r, mix_k, mix_v, mix_g, mix_w, r_weight, k_weight, v_weight, gate_weight, decay_down,
    decay_up, decay_bias, bonus, out_norm, o_weight``."""

    MIXES = (("mix_r", "r_weight"), ("mix_k", "k_weight"), ("mix_v", "v_weight"), ("mix_g", "gate_weight"),
             ("mix_w", "decay_down"))

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, tensors: Dict[str, str],
                 value_dim: Optional[int] = None, norm_eps: float = 1e-6, gate: str = "silu"):
        super().__init__(tensors)
        self._set_sizes(hidden_size, num_heads, key_dim, key_dim if value_dim is None else value_dim)
        self.norm_eps = float(norm_eps)
        if gate not in ("sigmoid", "silu"):
            raise ValueError(f"the output gate is 'sigmoid' or 'silu', got {gate!r}")
        self.gate = gate
        self.decay_rank = None
        self.mix = self.w_o = self.w_decay = self.b_decay = self.bonus = self.norm_weight = None
        self.w_mixed, self.offsets, self.in_size = None, {}, 0

    def tensor_specs(self):
        t, w = self.tensor_names, self.hidden_size
        file_v = self.num_heads * self.file_value_dim
        specs = {t[role]: TensorSpec((w,), VECTOR) for role, _ in self.MIXES}
        specs.update({
            t["r_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["k_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["v_weight"]: TensorSpec((file_v, w), MATRIX),
            t["gate_weight"]: TensorSpec((file_v, w), MATRIX),
            t["decay_down"]: TensorSpec((None, w), MATRIX),
            t["decay_up"]: TensorSpec((self.qk_size, None), MATRIX),
            t["decay_bias"]: TensorSpec((self.qk_size,), VECTOR),
            t["bonus"]: TensorSpec((self.num_heads, self.key_dim), VECTOR),
            t["out_norm"]: TensorSpec((file_v,), VECTOR, INIT_NORM),
            t["o_weight"]: TensorSpec((w, file_v), MATRIX),
        })
        return specs

    def bind(self, tensors, ops, dtype):
        super().bind(tensors, ops, dtype)
        self._check_sizes(ops, dtype, "time mixing")
        t = self.tensor_names
        rank = int(tensors[t["decay_down"]].shape[0])
        if int(tensors[t["decay_up"]].shape[1]) != rank:
            raise ValueError(f"{t['decay_down']} has {rank} rows but {t['decay_up']} has "
                             f"{int(tensors[t['decay_up']].shape[1])} columns: the two factors of the decay "
                             f"projection do not fit")
        self.decay_rank = rank
        self.mix = torch.stack([tensors[t[role]].float() for role, _ in self.MIXES]).contiguous()
        at, weights = 0, []
        for _, role in self.MIXES:
            weights.append(self._values(tensors[t[role]]) if role in ("v_weight", "gate_weight") else tensors[t[role]])
            self.offsets[role] = at
            at += (weights[-1].shape[0] + 15) // 16 * 16       # (as the segments of the weight lie)
        self.in_size = at
        self.w_mixed = ops.prepare_segments(weights)
        self.w_o = ops.prepare_weight(self._values(tensors[t["o_weight"]].t()).t().contiguous())
        # the second factor of the decays is applied in float32, inside the decay kernel
        self.w_decay = tensors[t["decay_up"]].float().contiguous()
        self.b_decay = tensors[t["decay_bias"]].float().contiguous()
        self.bonus = tensors[t["bonus"]].float().reshape(-1).contiguous()
        self.norm_weight = self._values(tensors[t["out_norm"]].float()).contiguous()

    def state_spec(self):
        return dict(super().state_spec(), previous_row=((self.hidden_size,), None))

    def forward_into(self, h, out, ctx, entry):
        ops, rows, o = self.ops, h.shape[0], self.offsets
        mixed = ctx.scratch("time_mix.mixed", (len(self.MIXES), rows, self.hidden_size), self.dtype)
        ops.shift_mix(h, self.mix, entry.state["previous_row"], ctx.row_req, ctx.all_q_start, ctx.all_req_rows, mixed)
        proj = ctx.scratch("time_mix.proj", (rows, self.in_size), torch.float32)
        ops.segmented_products(mixed, self.w_mixed, proj, [o[role] for _, role in self.MIXES])
        off = [o[role] for role in ("r_weight", "k_weight", "v_weight", "gate_weight")]
        decay = ctx.scratch("linear_attention.decay", (rows, self.qk_size), torch.float32)

        def many_rows(gated):
            ops.gla_decay(proj[:, o["decay_down"]:], self.decay_rank, self.w_decay, self.b_decay, 1.0, decay, "double_exp")
            parts = self._scan(proj, *off[:3], decay, 1.0, entry.state["s"], ctx, bonus=self.bonus)
            self._output(parts, self.norm_weight, self.norm_eps, proj, off[3], self.gate, gated)

        def in_chunks(gated):
            ops.gla_decay(proj[:, o["decay_down"]:], self.decay_rank, self.w_decay, self.b_decay, 1.0, decay, "double_exp",
                          as_log=True)
            self._in_chunks(proj, ctx, entry, off, decay, self.norm_weight, self.norm_eps, self.gate, 1.0, gated,
                            bonus=self.bonus)
        gated = self._recur(proj, ctx, entry, off, self.norm_weight, self.norm_eps, self.gate, 1.0, many_rows, in_chunks,
                            self.decay_rank, bonus=self.bonus,
                            decay=(o["decay_down"], self.decay_rank, self.w_decay, self.b_decay, "double_exp", 1.0))
        ops.linear_logits(gated, self.w_o, out)

    def kernel_libraries(self):
        return [("stream_ops", None), ("linear_attention", None)]

    def weight_bytes(self):
        return sum(w.numel() * w.element_size() for w in (self.w_mixed, self.mix, self.w_o, self.w_decay,
                                                          self.b_decay, self.bonus, self.norm_weight) if w is not None)


class MatrixMemoryAttention(ScanMixer):
    """A matrix memory with exponential gates: one log input gate and one log forget gate per head, a
    running maximum that keeps the exponentials in range, and a normaliser.

    With ``D = key_dim`` and ``E = value_dim``: ``q = Wq h * q_scale`` (``q_scale`` defaults to ``D ** -0.5``), ``k = Wk
    h`` (``heads x D``), ``v = Wv h`` (``heads x E``); per head ``i = cap * tanh((Wi h + bi) / cap)`` and ``f =
    logsigmoid(cap * tanh((Wf h + bf) / cap))``; token by token, all of ``S``, ``n`` and ``m`` zero at a
    sequence's start::

        m_t = max(f_t + m_(t-1), i_t)
        S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T        (S is D x E)
        n_t = exp(f_t + m_(t-1) - m_t) n_(t-1) + exp(i_t - m_t) k_t
        o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)

    then every head's ``o_t`` is divided by its root mean square over ``E`` (``norm_eps`` inside the root), the
    heads are put side by side, multiplied by a weight of all heads' size and by ``sigmoid(Wg h)``
    (``gate="silu"``: by ``silu``), and projected by ``Wo``.

    State per request, float32: ``S``, ``n`` and ``m``.  Gates, maximum, recurrence, normaliser and norm are
    float32, and the projections reach them unrounded (32-bit sums of the matrix products).

    Tensor roles: ``q_weight, k_weight, v_weight, gate_weight, i_weight, i_bias, f_weight, f_bias, out_norm,
    o_weight``."""

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, gate_cap: float,
                 tensors: Dict[str, str], norm_eps: float = 1e-6, q_scale: Optional[float] = None, gate: str = "sigmoid"):
        super().__init__(tensors)
        self._set_sizes(hidden_size, num_heads, key_dim, value_dim)
        self.gate_cap, self.norm_eps = float(gate_cap), float(norm_eps)
        if self.gate_cap <= 0:
            raise ValueError(f"the gates' cap must be positive, got {gate_cap}")
        if gate not in ("sigmoid", "silu"):
            raise ValueError(f"the output gate is 'sigmoid' or 'silu', got {gate!r}")
        self.gate = gate
        self.q_scale = float(q_scale) if q_scale is not None else self.key_dim ** -0.5
        self.w_in = self.w_o = self.b_i = self.b_f = self.norm_weight = None
        self.offsets, self.in_size = {}, 0

    def tensor_specs(self):
        t, w = self.tensor_names, self.hidden_size
        file_v = self.num_heads * self.file_value_dim
        return {
            t["q_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["k_weight"]: TensorSpec((self.qk_size, w), MATRIX),
            t["v_weight"]: TensorSpec((file_v, w), MATRIX),
            t["gate_weight"]: TensorSpec((file_v, w), MATRIX),
            t["i_weight"]: TensorSpec((self.num_heads, w), MATRIX),
            t["i_bias"]: TensorSpec((self.num_heads,), VECTOR),
            t["f_weight"]: TensorSpec((self.num_heads, w), MATRIX),
            t["f_bias"]: TensorSpec((self.num_heads,), VECTOR),
            t["out_norm"]: TensorSpec((file_v,), VECTOR, INIT_NORM),
            t["o_weight"]: TensorSpec((w, file_v), MATRIX),
        }

    def bind(self, tensors, ops, dtype):
        super().bind(tensors, ops, dtype)
        self._check_sizes(ops, dtype, "matrix memory")
        t = self.tensor_names
        at, rows = 0, []
        for role in ("q_weight", "k_weight", "v_weight", "gate_weight", "i_weight", "f_weight"):      # (one product)
            self.offsets[role] = at
            rows.append(self._values(tensors[t[role]]) if role in ("v_weight", "gate_weight") else tensors[t[role]])
            at += rows[-1].shape[0]
        self.in_size = at
        self.w_in = ops.prepare_weight(torch.cat(rows, dim=0).contiguous())
        self.w_o = ops.prepare_weight(self._values(tensors[t["o_weight"]].t()).t().contiguous())
        self.b_i = tensors[t["i_bias"]].float().contiguous()
        self.b_f = tensors[t["f_bias"]].float().contiguous()
        self.norm_weight = self._values(tensors[t["out_norm"]].float()).contiguous()

    def state_spec(self):
        return dict(super().state_spec(), n=((self.num_heads, self.key_dim), torch.float32),
                    m=((self.num_heads,), torch.float32))

    def forward_into(self, h, out, ctx, entry):
        ops, rows, o = self.ops, h.shape[0], self.offsets
        proj = ctx.scratch("linear_attention.proj", (rows, self.in_size), torch.float32)
        ops.linear_logits(h, self.w_in, proj)
        keep, take, maxima = (ctx.scratch("matrix_memory." + name, (rows, self.num_heads), torch.float32)
                              for name in ("keep", "take", "maxima"))
        off = [o[role] for role in ("q_weight", "k_weight", "v_weight", "gate_weight")]

        def gates(**how):
            ops.memory_gates(proj, o["i_weight"], o["f_weight"], self.b_i, self.b_f, self.gate_cap, self.num_heads,
                             entry.state["m"], ctx.all_q_start, ctx.all_req_rows, ctx.n_reqs, keep, take, maxima, **how)

        def in_chunks(mixed):
            gates(as_log=True)
            self._in_chunks(proj, ctx, entry, off, keep, self.norm_weight, self.norm_eps, self.gate, self.q_scale, mixed,
                            memory=(take, maxima))

        def many_rows(mixed):
            gates()
            parts, norm_parts = self._scan(proj, *off[:3], None, self.q_scale, entry.state["s"], ctx,
                                           memory=(keep, take, entry.state["n"]))
            self._output(parts, self.norm_weight, self.norm_eps, proj, off[3], self.gate, mixed, norm_parts=norm_parts,
                         maxima=maxima)
        mixed = self._recur(proj, ctx, entry, off, self.norm_weight, self.norm_eps, self.gate, self.q_scale, many_rows,
                            in_chunks, memory=(o["i_weight"], o["f_weight"], self.b_i, self.b_f, self.gate_cap, entry.state["n"],
                                    entry.state["m"]))
        ops.linear_logits(mixed, self.w_o, out)

    def weight_bytes(self):
        return sum(w.numel() * w.element_size() for w in (self.w_in, self.w_o, self.b_i, self.b_f, self.norm_weight)
                   if w is not None)


register_part("mixer", "gated_linear_attention", GatedLinearAttention)
register_part("mixer", "time_mix_attention", TimeMixAttention)
register_part("mixer", "matrix_memory_attention", MatrixMemoryAttention)
register_part("mixer", "delta_rule_attention", DeltaRuleAttention)
