"""A mixer whose state is one number per channel."""
from __future__ import annotations

from typing import Dict

import torch

from ..weights.loader import TensorSpec, MATRIX, VECTOR
from .base import Mixer, NormedInput, PendingSums
from .linear_attention import pad_heads
from .registry import register_part


class GatedLinearRecurrence(Mixer):
    """Two branches of ``width`` channels; one runs through a short causal convolution and a linear
    recurrence of single numbers with gates, the other multiplies its result.

    ``y = gelu_tanh(Wy h + by)``; ``x = Wx h + bx``; ``u_t = b + sum_j w[:, j] x_(t - taps + 1 + j)`` channel by channel
    (nothing before the sequence's start).  ``u`` is cut into ``blocks`` equal parts; part ``p`` has square matrices
    ``R_p, I_p`` (``[out, in]``): ``r = sigmoid(R_p u_p + rb_p)``, ``i = sigmoid(I_p u_p + ib_p)``.  Then token by token,
    channel by channel, from zero::

        log a_t = -decay_scale * r_t * softplus(lambda)
        S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t

    and the result is ``Wo (S * y)``.

    State per request: ``S`` in float32, and the convolution's last inputs in float32 in a ring of ``taps`` rows,
    position ``p`` at row ``p mod taps`` (a step of one row overwrites a row that no tap of it reads).  Gates,
    decays and the recurrence are float32; the gates' products take ``u`` and the matrices in the compute dtype
    with 32-bit sums.  A part is laid out in a multiple of 32 channels (zeros behind), the matrix cores' inner
    size.

    Tensor roles: ``y_weight, y_bias, x_weight, x_bias, conv [width, taps], conv_bias, r_weight [blocks, n, n], r_bias
    [blocks, n], i_weight, i_bias, decay [width], o_weight``."""

    writes_output = True
    keeps_launches = True

    def __init__(self, hidden_size: int, width: int, blocks: int, conv_taps: int, tensors: Dict[str, str],
                 decay_scale: float = 8.0):
        super().__init__(tensors)
        self.hidden_size, self.width, self.blocks, self.taps = int(hidden_size), int(width), int(blocks), int(conv_taps)
        self.decay_scale = float(decay_scale)
        if self.width <= 0 or self.blocks <= 0 or self.width % self.blocks:
            raise ValueError(f"a width of {width} does not form {blocks} equal parts")
        if self.taps < 1:
            raise ValueError(f"the convolution has at least one tap, got {conv_taps}")
        self.part = self.width // self.blocks                    # a part as the model file has it
        self.laid = (self.part + 31) // 32 * 32                  # and as the kernels see it
        self.w_in = self.b_in = self.conv = self.conv_bias = self.gates = self.r_bias = self.i_bias = self.decay = None
        self.w_o = None

    @property
    def channels(self):
        return self.blocks * self.laid

    def tensor_specs(self):
        t, w, n, h = self.tensor_names, self.width, self.part, self.hidden_size
        specs = {}
        for role in ("y", "x"):
            specs[t[role + "_weight"]] = TensorSpec((w, h), MATRIX)
            specs[t[role + "_bias"]] = TensorSpec((w,), VECTOR)
        specs[t["conv"]] = TensorSpec((w, self.taps), MATRIX)
        specs[t["conv_bias"]] = TensorSpec((w,), VECTOR)
        for role in ("r", "i"):
            specs[t[role + "_weight"]] = TensorSpec((self.blocks, n, n), MATRIX)
            specs[t[role + "_bias"]] = TensorSpec((self.blocks, n), VECTOR)
        specs[t["decay"]] = TensorSpec((w,), VECTOR)
        specs[t["o_weight"]] = TensorSpec((h, w), MATRIX)
        return specs

    def state_spec(self):
        spec = {"s": ((self.channels,), torch.float32)}
        if self.taps > 1:
            spec["conv"] = ((self.taps, self.channels), torch.float32)
        return spec

    def bind(self, tensors, ops, dtype):
        super().bind(tensors, ops, dtype)
        ops.check_product_sizes(self.hidden_size, dtype, "recurrence projections (hidden size)")
        t = self.tensor_names

        def parts(x):
            return pad_heads(x, self.blocks, self.part, self.laid)

        def matrices(x):
            more = self.laid - self.part
            return torch.nn.functional.pad(x, (0, more, 0, more)).contiguous()
        # one product for both branches: x, then y
        self.w_in = ops.prepare_weight(torch.cat([parts(tensors[t["x_weight"]]), parts(tensors[t["y_weight"]])]).contiguous())
        self.b_in = torch.cat([parts(tensors[t["x_bias"]].float()), parts(tensors[t["y_bias"]].float())]).contiguous()
        self.conv = parts(tensors[t["conv"]].float()).t().contiguous()
        self.conv_bias = parts(tensors[t["conv_bias"]].float()).contiguous()
        self.gates = ops.prepare_block_gates(matrices(tensors[t["r_weight"]]), matrices(tensors[t["i_weight"]]))
        self.r_bias = parts(tensors[t["r_bias"]].float().reshape(-1)).contiguous()
        self.i_bias = parts(tensors[t["i_bias"]].float().reshape(-1)).contiguous()
        softplus = torch.nn.functional.softplus(tensors[t["decay"]].double())
        self.decay = parts((-self.decay_scale * softplus).float()).contiguous()
        self.w_o = ops.prepare_weight(parts(tensors[t["o_weight"]].t()).t().contiguous())

    def _mixed(self, h, ctx, entry):
        """``S * y`` of this step's rows, in the compute dtype."""
        if isinstance(h, NormedInput):
            h = h.tensor()
        ops, rows, n = self.ops, h.shape[0], self.channels
        proj = ctx.scratch("gated_recurrence.proj", (rows, 2 * n), torch.float32)
        ops.linear_logits(h, self.w_in, proj, self.b_in)
        decays = ctx.scratch("gated_recurrence.decays", (rows, n), torch.float32)
        states = ctx.scratch("gated_recurrence.states", (rows, n), torch.float32)
        mixed = ctx.scratch("gated_recurrence.mixed", (rows, n), self.dtype)

        def launch():        # (how many rows the requests bring is not a matter of the number of rows)
            ops.gated_recurrence(proj, 0, n, self.laid, self.conv, self.conv_bias, entry.state.get("conv"), self.gates,
                                 self.r_bias, self.i_bias, self.decay, entry.state["s"], ctx.positions, ctx.all_q_start,
                                 ctx.all_req_rows, ctx.n_reqs, decays, states, mixed, ctx.n_rows == ctx.n_reqs)
        live = getattr(ops, "live", None)
        if live is not None:
            live(launch)
        else:
            launch()
        return mixed

    def forward_into(self, h, out, ctx, entry):
        self.ops.linear_logits(self._mixed(h, ctx, entry), self.w_o, out)

    def forward_split(self, h, out, ctx, entry):
        return self._product_split(self._mixed(h, ctx, entry), self.w_o, out, ctx)

    def forward(self, h, residual, ctx, entry):
        y = ctx.scratch("gated_recurrence.sum", (1,) + tuple(residual.shape), torch.float32)
        self.forward_into(h, y[0], ctx, entry)
        self.ops.add_pending(residual, PendingSums(y, 1))

    def kernel_libraries(self):
        return [("gated_recurrence", None)]

    def weight_bytes(self):
        return sum(w.numel() * w.element_size() for w in (self.w_in, self.b_in, self.conv, self.conv_bias, self.gates,
                                                          self.r_bias, self.i_bias, self.decay, self.w_o) if w is not None)


register_part("mixer", "gated_linear_recurrence", GatedLinearRecurrence)
