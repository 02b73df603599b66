"""A mixer made of two: both on one input, their results summed."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..config.spec import PartSpec
from ..weights.loader import TensorSpec, VECTOR, INIT_NORM
from .base import Mixer, NormedInput, NormedPair, PendingSums
from .registry import register_part, build_part


class ParallelMixers(Mixer):
    """``left_scale * left(h) + right_scale * right(h)``: two mixers of any registered kind read
    the same input; their float32 results are summed with two fixed weights.  At most one of the
    two keeps a per-token cache (the run's pages are that one's); per-request state of both is kept
    under the names they give it, which must differ.

    ``norm_eps``: each of the two results is first divided by its root mean square over the width
    (``norm_eps`` inside the root) and multiplied by a weight of that width, ``left_scale * norm_l(left(h))
    + right_scale * norm_r(right(h))``; tensor roles ``left_norm`` and ``right_norm``, ``hidden_size`` wide."""

    writes_output = True
    takes_normed_input = True      # (each of the two takes it as it can; the norm itself runs at most once)

    def __init__(self, left: PartSpec, right: PartSpec, left_scale: float = 1.0, right_scale: float = 1.0,
                 tensors: Optional[Dict[str, str]] = None, norm_eps: Optional[float] = None,
                 hidden_size: Optional[int] = None):
        super().__init__(tensors)
        self.norm_eps = None if norm_eps is None else float(norm_eps)
        self.hidden_size = None if hidden_size is None else int(hidden_size)
        if self.norm_eps is not None and self.hidden_size is None:
            raise ValueError("norms of the two results need their width")
        self.out_norms = None
        self.left, self.right = build_part("mixer", left), build_part("mixer", right)
        self.left_scale, self.right_scale = float(left_scale), float(right_scale)
        if self.left.cache_spec() is not None and self.right.cache_spec() is not None:
            raise ValueError("the two mixers share one run of the schedule: only one of them may keep a cache")
        clash = set(self.left.state_spec()) & set(self.right.state_spec())
        if clash:
            raise ValueError(f"both mixers keep per-request state called {sorted(clash)}")

    def members(self):
        return [self.left, self.right]

    def tensor_specs(self):
        specs = dict(self.left.tensor_specs())
        specs.update(self.right.tensor_specs())
        if self.norm_eps is not None:
            for role in ("left_norm", "right_norm"):
                specs[self.tensor_names[role]] = TensorSpec((self.hidden_size,), VECTOR, INIT_NORM)
        return specs

    def bind(self, tensors, ops, dtype):
        super().bind(tensors, ops, dtype)
        for m in self.members():
            m.bind(tensors, ops, dtype)
        if self.norm_eps is not None:
            self.out_norms = [tensors[self.tensor_names[role]].float().contiguous() for role in ("left_norm", "right_norm")]

    def cache_spec(self):
        return self.left.cache_spec() or self.right.cache_spec()

    def state_spec(self):
        spec = dict(self.left.state_spec())
        spec.update(self.right.state_spec())
        return spec

    @property
    def graph_safe(self):
        return all(m.graph_safe for m in self.members())

    @property
    def keeps_launches(self):
        return all(m.keeps_launches for m in self.members())

    def kernel_libraries(self):
        return [("stream_ops", None)] + [lib for m in self.members() for lib in m.kernel_libraries()]

    def _result(self, mixer, name, h, shape, ctx, entry):
        if isinstance(h, NormedInput) and not mixer.takes_normed_input:
            h = h.tensor()
        y = ctx.scratch(name, shape, torch.float32)
        if mixer.writes_output:
            mixer.forward_into(h, y, ctx, entry)
        else:                               # (a mixer made to add into the stream: into zeros)
            self.ops.activation(y, y, "zero")
            mixer.forward(h, y, ctx, entry)
            pending = getattr(ctx, "pending", None)
            if pending is not None:
                self.ops.add_pending(y, pending)
                ctx.pending = None
        return y

    def forward_pending(self, h, out, ctx, entry):
        """The two normed results as a ``NormedPair`` (where the results are normed), for a caller that sums
        them on its own way; else their sum in ``out`` and None."""
        if self.out_norms is None:
            self.forward_into(h, out, ctx, entry)
            return None
        y1, y2 = self._results(h, tuple(out.shape), ctx, entry)
        return NormedPair(y1, self.out_norms[0], self.left_scale, y2, self.out_norms[1], self.right_scale, self.norm_eps)

    def _results(self, h, shape, ctx, entry):
        return (self._result(self.left, "parallel.left", h, shape, ctx, entry),
                self._result(self.right, "parallel.right", h, shape, ctx, entry))

    def forward_into(self, h, out, ctx, entry):
        y1, y2 = self._results(h, tuple(out.shape), ctx, entry)
        if self.out_norms is not None:
            self.ops.normed_sum(out, y1, self.out_norms[0], self.left_scale, y2, self.out_norms[1], self.right_scale,
                                self.norm_eps)
        else:
            self.ops.scaled_sum(out, y1, self.left_scale, y2, self.right_scale)

    def forward(self, h, residual, ctx, entry):
        y = ctx.scratch("parallel.sum", (1,) + tuple(residual.shape), torch.float32)
        self.forward_into(h, y[0], ctx, entry)
        self.ops.add_pending(residual, PendingSums(y, 1))

    def weight_bytes(self):
        own = sum(w.numel() * w.element_size() for w in self.out_norms or ())
        return own + sum(m.weight_bytes() for m in self.members())


register_part("mixer", "parallel", ParallelMixers)
