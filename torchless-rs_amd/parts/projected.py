"""Mixers of the form W_o heads(W_in y), and two of them side by side.

`ProjectedMixer`: one product makes a row of everything the mixer reads, something happens to that
row (`heads`: attention, a recurrence), one product brings the result back to the model's width.

`ParallelMixer`: two such mixers that read the same input, left_scale * left + right_scale * right,
as one: their input rows lie side by side in one product, their results side by side in front of
one output product, and the scales go into the results before they are rounded (`factor`).
"""
from __future__ import annotations

from typing import Dict, Tuple

import torch

from ..weights.binding import WeightSpec
from .base import Mixer, PartSpec, make_part, register_part
from .linear import Linear

ROW_STEP = 16           # input rows are padded with zeros to a multiple of this many channels where they are made up of odd parts


def same_dtype(weights):
    """The weights as they are if they share a dtype, else all in float32."""
    if len({w.dtype for w in weights}) > 1:
        return [w.to(torch.float32) for w in weights]
    return list(weights)


def stacked(weights, step: int = ROW_STEP) -> torch.Tensor:
    """The rows of all `weights` below each other, with zeros up to a multiple of `step` rows."""
    ws = same_dtype(weights)
    short = -sum(w.shape[0] for w in ws) % step
    if short:
        ws.append(torch.zeros((short, ws[0].shape[1]), dtype=ws[0].dtype, device=ws[0].device))
    return torch.cat(ws, dim=0)


class ProjectedMixer(Mixer):
    """A subclass implements `load_terms` and `heads`; `factor` multiplies its result (set before loading)."""
    graph_safe = True
    closes_stream = True          # its last write to the stream is `Linear.add_into`
    factor = 1.0
    tag = "projected"             # names its buffers in the workspace
    in_width = heads_width = 0    # channels of a row of the input product, and of the result; known once loaded
    proj = o = None

    def load_terms(self, tensors: Dict[str, torch.Tensor], compute_dtype: torch.dtype) -> Tuple[torch.Tensor, torch.Tensor]:
        """Take what `heads` needs and set `in_width` and `heads_width`; returns the two products' weights
        [in_width, H] and [H, heads_width]."""
        raise NotImplementedError

    def heads(self, ctx, run, proj: torch.Tensor, out: torch.Tensor) -> None:
        """proj float32 [n, in_width] -> out [n, heads_width] in the compute dtype; rows of either may be strided."""
        raise NotImplementedError

    def load(self, tensors, compute_dtype) -> None:
        w_in, w_out = self.load_terms(tensors, compute_dtype)
        self.proj, self.o = Linear(w_in, tiled=True), Linear(w_out, tiled=True)

    def may_capture(self, n_rows: int) -> bool:
        return self.proj is not None and self.proj.own_kernels(n_rows) and self.o.own_kernels(n_rows)

    def _result(self, ctx, run, y: torch.Tensor) -> torch.Tensor:
        n, ws = y.shape[0], ctx.workspace
        proj = ws.get(self.tag + "_proj", (n, self.in_width), torch.float32)
        self.proj(y, proj)
        h = ws.get(self.tag + "_heads", (n, self.heads_width), ctx.dtype)
        self.heads(ctx, run, proj, h)
        return h

    def forward(self, ctx, run, y: torch.Tensor, x: torch.Tensor) -> None:
        self.o.add_into(self._result(ctx, run, y), x, ctx, self.tag + "_o_parts")

    def produce(self, ctx, run, y: torch.Tensor, out: torch.Tensor):
        """The result stored in `out` (float32 [n, H]) instead of added to the stream."""
        self.o(self._result(ctx, run, y), out)


class ParallelMixer(ProjectedMixer):
    """left_scale * left(y) + right_scale * right(y): `left` and `right` are projected mixers without a bias on
    their output, of which one at most keeps keys and values and one at most a state."""
    tag = "parallel"

    def __init__(self, left: PartSpec, right: PartSpec, left_scale: float = 1.0, right_scale: float = 1.0):
        self.sides = [make_part("mixer", left), make_part("mixer", right)]
        for side, scale in zip(self.sides, (left_scale, right_scale)):
            if not isinstance(side, ProjectedMixer) or getattr(side, "has_o_bias", False):
                raise ValueError(f"parallel mixers: {type(side).__name__} is no projected mixer without a bias on its output")
            side.factor = float(scale) * self.factor
        self.graph_safe = all(s.graph_safe for s in self.sides)
        for ask in ("kv_request", "state_request"):
            if all(getattr(s, ask)() is not None for s in self.sides):
                raise ValueError(f"parallel mixers: both sides have a {ask}")

    def _asked(self, ask: str):
        return next((r for r in (getattr(s, ask)() for s in self.sides) if r is not None), None)

    def kv_request(self):
        return self._asked("kv_request")

    def state_request(self):
        return self._asked("state_request")

    def may_capture(self, n_rows: int) -> bool:
        return super().may_capture(n_rows) and all(s._steps_capture(n_rows) for s in self.sides if hasattr(s, "_steps_capture"))

    def prefers_eager(self, n_new, len_before, device) -> bool:
        return any(s.prefers_eager(n_new, len_before, device) for s in self.sides)

    def weight_specs(self) -> Dict[str, WeightSpec]:
        out: Dict[str, WeightSpec] = {}
        for s in self.sides:
            out.update(s.weight_specs())
        return out

    def load_terms(self, tensors, compute_dtype):
        pairs = [s.load_terms(tensors, compute_dtype) for s in self.sides]
        self.in_width, self.heads_width = (sum(getattr(s, k) for s in self.sides) for k in ("in_width", "heads_width"))
        return torch.cat(same_dtype([p[0] for p in pairs]), dim=0), torch.cat(same_dtype([p[1] for p in pairs]), dim=1)

    def heads(self, ctx, run, proj: torch.Tensor, out: torch.Tensor) -> None:
        a, b = self.sides
        a.heads(ctx, run, proj[:, :a.in_width], out[:, :a.heads_width])
        b.heads(ctx, run, proj[:, a.in_width:], out[:, a.heads_width:])


register_part("mixer", "parallel", ParallelMixer)
