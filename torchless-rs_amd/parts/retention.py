"""Retention: linear attention with a fixed decay per head, no softmax and no denominator.

With H heads of `head_dim` (queries, keys) and `v_head_dim` (values), one product over the mixer's
input gives a row [q | k | v | g].  q and k are rotated by position (`position`), k is then
multiplied by head_dim^(-1/2), and per head

    S <- decay_h S + k v^T ,   o = S^T q      (S: [head_dim, v_head_dim], from zero)
    out = W_o ( concat_h( o / sqrt(mean(o^2) + eps) ) * silu(g) )

the norm per head without a weight.  What a sequence keeps is S in float32 (`StateRequest`),
whatever its length; nothing per position.  Decays, the state, the norm and silu(g) are float32 in
both dtypes.

Single tokens, short portions and the 32-bit path go row by row with everything in float32
(`ops.retention_scan`); longer bfloat16 steps go by chunks of rows on the matrix cores
(`ops.retention_chunks`).
"""
from __future__ import annotations

import math
from typing import Dict, Optional, Sequence

import torch

from ..cache.cache import StateRequest
from ..kernels import ops
from ..weights.binding import WeightSpec
from .base import Mixer, PartSpec, make_part, register_part
from .linear import Linear

CHUNKS_FROM = 32             # a bfloat16 step whose longest sequence brings this many rows goes by chunks
NO_DECAY_LEFT = -10000.0     # log2 of a decay of 0, as the chunks' kernels take it


class RetentionMixer(Mixer):
    graph_safe = True
    closes_stream = True          # its last write to the stream is `Linear.add_into`

    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o"}

    def __init__(self, hidden_size: int, n_heads: int, head_dim: int, decay: Sequence[float], norm_eps: float,
                 v_head_dim: Optional[int] = None, position: Optional[PartSpec] = None, prefix: str = "mix.",
                 names: Optional[Dict[str, str]] = None):
        unknown = set(names or {}) - set(self.NAMES)
        if unknown:
            raise ValueError(f"retention: no tensors called {sorted(unknown)}; there are {sorted(self.NAMES)}")
        if len(decay) != n_heads or any(not float(a) >= 0.0 for a in decay):
            raise ValueError(f"retention: {n_heads} heads need as many decays, none below 0")
        self.names = dict(self.NAMES, **(names or {}))
        self.H, self.heads, self.dk = int(hidden_size), int(n_heads), int(head_dim)
        self.dv = self.dk if v_head_dim is None else int(v_head_dim)
        self.decay_host = [float(a) for a in decay]
        self.eps, self.prefix = float(norm_eps), prefix
        self.kscale = self.dk ** -0.5
        self.position = make_part("position", position if position is not None else PartSpec("none"))
        self.proj = self.o = self.decay = None

    def state_request(self):
        return StateRequest((self.heads * self.dk * self.dv,), torch.float32)

    def may_capture(self, n_rows: int) -> bool:
        return self.proj is not None and self.proj.own_kernels(n_rows) and self.o.own_kernels(n_rows)

    def weight_specs(self) -> Dict[str, WeightSpec]:
        p, nm = self.prefix, self.names
        Q, V = self.heads * self.dk, self.heads * self.dv
        return {p + nm["q"]: WeightSpec((Q, self.H)), p + nm["k"]: WeightSpec((Q, self.H)),
                p + nm["v"]: WeightSpec((V, self.H)), p + nm["g"]: WeightSpec((V, self.H)),
                p + nm["o"]: WeightSpec((self.H, V))}

    def load(self, tensors, compute_dtype) -> None:
        p, nm = self.prefix, self.names
        ws = [tensors[p + nm[k]] for k in ("q", "k", "v", "g")]
        if len({w.dtype for w in ws}) > 1:
            ws = [w.to(torch.float32) for w in ws]
        self.proj = Linear(torch.cat(ws, dim=0), tiled=True)
        self.o = Linear(tensors[p + nm["o"]], tiled=True)
        self.decay = torch.tensor(self.decay_host, dtype=torch.float64).to(torch.float32).to(ws[0].device)
        logs = [math.log2(a) if a > 0.0 else NO_DECAY_LEFT for a in self.decay_host]
        self.log2_decay = torch.tensor(logs, dtype=torch.float64).to(torch.float32).to(ws[0].device)

    def _heads(self, ctx, run, y: torch.Tensor) -> torch.Tensor:
        """The normed and gated heads [n, H * dv] in the compute dtype."""
        n, H, dk, dv = y.shape[0], self.heads, self.dk, self.dv
        ws = ctx.workspace
        proj = ws.get("ret_proj", (n, 2 * H * (dk + dv)), torch.float32)
        self.proj(y, proj)
        rotation = self.position.rotation(y.device) or ops.NO_ROTATION
        h = ws.get("ret_h", (n, H * dv), ctx.dtype)
        if ctx.max_new >= CHUNKS_FROM and ops.retention_chunks_serve(ctx.dtype, dk, dv):
            C = ops.retention_chunk()
            chunks = int(sum(-(-int(r) // C) for r in ctx.host["n_new"]))
            ops.retention_chunks(proj, ctx.row_pos, rotation, H, dk, dv, self.kscale, self.log2_decay, self.eps, run.state,
                                 ctx.cu_seqlens, ctx.slots, chunks, ws, h)
            return h
        o = ws.get("ret_o", (n, H * dv), torch.float32)
        ops.retention_scan(proj, ctx.row_pos, rotation, H, dk, dv, self.kscale, self.decay, run.state, ctx.cu_seqlens,
                           ctx.slots, o)
        ops.retention_norm_gate(o, proj[:, 2 * H * dk + H * dv:], H, self.eps, h)
        return h

    def forward(self, ctx, run, y: torch.Tensor, x: torch.Tensor) -> None:
        self.o.add_into(self._heads(ctx, run, y), x, ctx, "ret_o_parts")

    def produce(self, ctx, run, y: torch.Tensor, out: torch.Tensor) -> None:
        """The result stored in `out` (float32 [n, H]) instead of added to the stream."""
        self.o(self._heads(ctx, run, y), out)


register_part("mixer", "retention", RetentionMixer)
