"""Feed-forwards without a gate, and a routed mixture of them.

`PlainFeedForward`: down(act(up y)), act one of `ops.EXPERT_ACTIVATIONS` (relu2: the square of
max(., 0); xielu: a z^2 + z/2 for z > 0 and b (exp(z) - 1 - z) + z/2 elsewhere, a = softplus(p) and
b = 1/2 + softplus(q) from a tensor `act` of the two numbers p and q).

`RoutedExperts`: `n_experts` such layers of which every token uses `top`.  The router is one
more product, in float32: s = softmax(W_r y) over all experts.  The experts form
`group_count` equal groups of neighbours; a group's score is its largest s, and only experts of
the `group_keep` best groups can be chosen (no groups: any expert).  The `top` experts with the
largest s are chosen; the result is the sum of their outputs weighted by their s, not
renormalised, plus a shared expert's (`shared_size`; None: none) that runs for every token.
`score` "sigmoid" makes every expert's score its own logistic function of the router's product
instead of a softmax over the experts.  `gated` experts have a gate beside the up projection,
down(act(gate t, up t)) with the clamped activation of `ops.GateTerms` (`activation_constants`:
limit, alpha, shift; the shared expert's limit may differ, `shared_limit`), and `weight_on`
"input" multiplies an expert's INPUT t = s y by the router's weight instead of its output.  The
activation "silu" makes gated experts silu(gate t) * (up t), with no clamp and no constants.
`correction` adds a learned number per expert to the scores for the CHOICE alone (the weights stay
the scores without it; choice scores may be negative); `group_score` "two_largest" scores a group by
the sum of its two largest choice scores; `normalise_eps` divides the chosen experts' scores by (their
sum + that number); `shared_gated` multiplies the shared expert's output by the logistic function of
one more row of the router (tensor `shared.sg`).  `router_bias` adds a learned number per expert to the router's product; with
`score` "softmax" and `normalise_eps` 0 the weights are the softmax over the chosen experts' logits alone.

All experts run as ONE wide feed-forward: their up projections stacked by rows (the shared
expert's behind them), the activation times the row's weight of the column's expert, which is
zero for an expert that was not chosen, and their down projections side by side.  That is two
products of the framework's own kinds and no gather or scatter, whatever the tokens choose; it
reads every expert's weights in every step, as a step of many rows does anyway, and multiplies
`n_experts / top` times what the chosen experts alone would.

A step of many rows in bfloat16 (on average `GROUPED_ROWS_PER_EXPERT` rows an expert or more, more rows
than the framework's own product kernels take, so that no graph holds the step) sorts the
(row, chosen expert) pairs by expert and runs every expert's two products over its own rows
(`_grouped`): the chosen experts' multiplications alone, at the price of one count per expert
read back by the host.

A step of few rows (rows * top <= n_experts: the rows cannot use every expert) runs the chosen
experts alone: per row two products of its experts' matrices with a vector
(`ops.expert_rows_up`, `ops.expert_rows_down`), which read `top` experts' weights a row and
nothing else.  Both ways round the hidden activations, times the router's weight, to the
compute dtype and sum in float32.
"""
from __future__ import annotations

import math
from typing import Dict, Optional

import torch

from ..kernels import ops
from ..weights.binding import WeightSpec
from .base import FeedForward, flush_pending, register_part
from .linear import Linear


GROUPED_ROWS_PER_EXPERT = 128      # from this many rows an expert on average, experts run over their own rows


class PlainFeedForward(FeedForward):
    graph_safe = True
    closes_stream = True

    NAMES = {"up": "up", "down": "down", "act": "act"}

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "relu2", prefix: str = "mlp.",
                 names: Optional[Dict[str, str]] = None):
        if activation not in ops.EXPERT_ACTIVATIONS:
            raise ValueError(f"feed-forward: no activation {activation!r}; there are {sorted(ops.EXPERT_ACTIVATIONS)}")
        self.H, self.I, self.activation, self.prefix = int(hidden_size), int(intermediate_size), activation, prefix
        self.names = dict(self.NAMES, **(names or {}))
        self.up = self.down = self.constants = None

    def may_capture(self, n_rows: int) -> bool:
        return self.up is not None and self.up.own_kernels(n_rows) and self.down.own_kernels(n_rows)

    def weight_specs(self) -> Dict[str, WeightSpec]:
        p, nm = self.prefix, self.names
        out = {p + nm["up"]: WeightSpec((self.I, self.H)), p + nm["down"]: WeightSpec((self.H, self.I))}
        if self.activation == "xielu":
            out[p + nm["act"]] = WeightSpec((2,))
        return out

    def load(self, tensors, compute_dtype) -> None:
        p, nm = self.prefix, self.names
        if self.activation == "xielu":
            a, b = torch.nn.functional.softplus(tensors[p + nm["act"]].to("cpu", torch.float64)).tolist()
            self.constants = {"a": a, "b": 0.5 + b}
        self.up = Linear(tensors[p + nm["up"]], tiled=True)
        self.down = Linear(tensors[p + nm["down"]], tiled=True)

    def _hidden(self, ctx, y: torch.Tensor) -> torch.Tensor:
        n = y.shape[0]
        h = ctx.workspace.get("pff_h", (n, self.I), ctx.dtype)
        if not self.up.own_kernels(n) and self.I % 8 == 0 and ops.bf16_gemm_ok(y, self.up.weight):
            u = ctx.workspace.get("pff_u16", (n, self.I), torch.bfloat16)      # many rows: half the traffic, one rounding more
            ops.gemm_library(y, self.up.weight, u)
        else:
            u = ctx.workspace.get("pff_u", (n, self.I), torch.float32)
            self.up(y, u)
        if self.I % 8 == 0:
            ops.unary_act(u, self.activation, h, self.constants)
        else:
            ops.expert_act(u, None, 0, self.I, self.activation, h, self.constants)
        return h

    def forward(self, ctx, y: torch.Tensor, x: torch.Tensor) -> None:
        self.down.add_into(self._hidden(ctx, y), x, ctx, "pff_down_parts")

    def produce(self, ctx, y: torch.Tensor, out: torch.Tensor) -> None:
        self.down(self._hidden(ctx, y), out)


class RoutedExperts(FeedForward):
    graph_safe = True
    closes_stream = True

    # leaf names under `prefix`; "{e}" is the expert's number
    NAMES = {"router": "router", "up": "e{e}.up", "down": "e{e}.down", "shared_up": "shared.up",
             "shared_down": "shared.down", "gate": "e{e}.gate", "shared_gate": "shared.gate", "correction": "correction",
             "shared_weight": "shared.sg", "router_bias": "router.b"}
    SCORES = ("softmax", "sigmoid")
    GROUP_SCORES = ("largest", "two_largest")
    GATED_ACTIVATION = "swish_clamped"

    def __init__(self, hidden_size: int, n_experts: int, top: int, expert_size: int, group_count: Optional[int] = None,
                 group_keep: Optional[int] = None, shared_size: Optional[int] = None, activation: str = "relu2",
                 prefix: str = "mlp.", names: Optional[Dict[str, str]] = None, score: str = "softmax",
                 gated: bool = False, activation_constants: Optional[Dict[str, float]] = None,
                 shared_limit: Optional[float] = None, weight_on: str = "output", correction: bool = False,
                 group_score: str = "largest", normalise_eps: Optional[float] = None, shared_gated: bool = False,
                 router_bias: bool = False):
        self.gated = bool(gated)
        if group_score not in self.GROUP_SCORES:
            raise ValueError(f"experts: a group's score is one of {self.GROUP_SCORES}, got {group_score!r}")
        self.has_correction, self.two_largest = bool(correction), group_score == "two_largest"
        self.normalise_eps = None if normalise_eps is None else float(normalise_eps)
        self.shared_gated = bool(shared_gated) and bool(shared_size)
        self.has_router_bias = bool(router_bias)
        self.correction = self.router_bias = None
        if score not in self.SCORES:
            raise ValueError(f"experts: scores are one of {self.SCORES}, got {score!r}")
        if weight_on not in ("output", "input"):
            raise ValueError(f"experts: the router's weight is on an expert's 'output' or 'input', got {weight_on!r}")
        if self.gated and activation == "silu":
            if activation_constants or shared_limit is not None:
                raise ValueError("experts: 'silu' has no constants")
            self.gate_terms = ops.GateTerms(math.inf, 1.0, 0.0, None, weight_on == "input")
        elif self.gated:
            need = {"limit", "alpha", "shift"}
            if activation != self.GATED_ACTIVATION or set(activation_constants or {}) != need:
                raise ValueError(f"experts: gated experts have the activation {self.GATED_ACTIVATION!r} with the "
                                 f"constants {sorted(need)}, got {activation!r} with {sorted(activation_constants or {})}")
            c = activation_constants
            self.gate_terms = ops.GateTerms(c["limit"], c["alpha"], c["shift"], shared_limit, weight_on == "input")
        elif activation not in ops.EXPERT_ACTIVATIONS:
            raise ValueError(f"experts: no activation {activation!r}; there are {sorted(ops.EXPERT_ACTIVATIONS)}")
        elif activation in ops.UNARY_CONSTANTS:
            raise ValueError(f"experts: {activation!r} takes learned numbers, which experts have none of")
        elif weight_on != "output" or activation_constants or shared_limit is not None:
            raise ValueError("experts: the weight on the input, constants and a shared limit go with gated experts")
        self.logistic = score == "sigmoid"
        if not (1 <= top <= n_experts):
            raise ValueError(f"experts: {top} of {n_experts}")
        if group_count:
            if n_experts % group_count or not (1 <= (group_keep or 0) <= group_count) or group_keep * (n_experts // group_count) < top:
                raise ValueError(f"experts: {n_experts} in {group_count} groups of which {group_keep} are kept cannot give {top}")
        self.H, self.E, self.top, self.ff = int(hidden_size), int(n_experts), int(top), int(expert_size)
        self.groups, self.keep = (int(group_count), int(group_keep)) if group_count else (0, 0)
        self.shared = int(shared_size) if shared_size else 0
        self.total = self.E * self.ff + self.shared
        self.activation, self.prefix = activation, prefix
        self.names = dict(self.NAMES, **(names or {}))
        self.router = self.up = self.down = None

    def may_capture(self, n_rows: int) -> bool:
        return self.up is not None and self.up.own_kernels(n_rows) and self.down.own_kernels(n_rows)

    def weight_specs(self) -> Dict[str, WeightSpec]:
        p, nm = self.prefix, self.names
        out: Dict[str, WeightSpec] = {}
        for e in range(self.E):
            if self.gated:
                out[p + nm["gate"].format(e=e)] = WeightSpec((self.ff, self.H))
            out[p + nm["up"].format(e=e)] = WeightSpec((self.ff, self.H))
            out[p + nm["down"].format(e=e)] = WeightSpec((self.H, self.ff))
        out[p + nm["router"]] = WeightSpec((self.E, self.H))
        if self.has_router_bias:
            out[p + nm["router_bias"]] = WeightSpec((self.E,))
        if self.has_correction:
            out[p + nm["correction"]] = WeightSpec((self.E,))
        if self.shared:
            if self.gated:
                out[p + nm["shared_gate"]] = WeightSpec((self.shared, self.H))
            out[p + nm["shared_up"]] = WeightSpec((self.shared, self.H))
            out[p + nm["shared_down"]] = WeightSpec((self.H, self.shared))
            if self.shared_gated:
                out[p + nm["shared_weight"]] = WeightSpec((1, self.H))
        return out

    def load(self, tensors, compute_dtype) -> None:
        p, nm = self.prefix, self.names
        ups = []
        for e in range(self.E):          # a gated expert's rows: [gate | up]
            ups += ([tensors[p + nm["gate"].format(e=e)]] if self.gated else []) + [tensors[p + nm["up"].format(e=e)]]
        downs = [tensors[p + nm["down"].format(e=e)] for e in range(self.E)]
        if self.shared:
            ups += ([tensors[p + nm["shared_gate"]]] if self.gated else []) + [tensors[p + nm["shared_up"]]]
            downs.append(tensors[p + nm["shared_down"]])
        if len({w.dtype for w in ups + downs}) > 1:
            ups, downs = [w.to(torch.float32) for w in ups], [w.to(torch.float32) for w in downs]
        self.up = Linear(torch.cat(ups, dim=0), tiled=True)          # [E * ff + shared, H]; gated: twice the rows
        self.down = Linear(torch.cat(downs, dim=1), tiled=True)      # [H, E * ff + shared]
        router = [tensors[p + nm["router"]].to(torch.float32)]
        if self.shared_gated:                                        # the shared expert's gate: one row more
            router.append(tensors[p + nm["shared_weight"]].to(torch.float32))
        self.router = torch.cat(router, dim=0).contiguous()
        if self.has_router_bias:
            self.router_bias = tensors[p + nm["router_bias"]].to(torch.float32).contiguous()
        if self.has_correction:
            self.correction = tensors[p + nm["correction"]].to(torch.float32).contiguous()

    def _route(self, ctx, y: torch.Tensor, chosen: bool):
        """The step's weights [n, E], chosen experts [n, top] (or None) and the shared expert's weight [n] (or None)."""
        n, ws = y.shape[0], ctx.workspace
        weights = ws.get("experts_w", (n, self.E), torch.float32)
        picked = ws.get("experts_chosen", (n, self.top), torch.int32) if chosen else None
        shared_weight = ws.get("experts_sw", (n,), torch.float32) if self.shared_gated else None
        ops.route(y, self.router, self.groups, self.keep, self.top, weights, picked, logistic=self.logistic,
                  correction=self.correction, two_largest=self.two_largest, normalise_eps=self.normalise_eps,
                  shared_weight=shared_weight, bias=self.router_bias)
        return weights, picked, shared_weight

    def few_rows(self, y: torch.Tensor) -> bool:
        """Do the rows of `y` run their chosen experts alone?"""
        return y.shape[0] * self.top <= self.E and self.up.weight.dtype == self.down.weight.dtype == y.dtype

    def _rows(self, ctx, y: torch.Tensor, out: torch.Tensor, accumulate: bool) -> None:
        n = y.shape[0]
        ws = ctx.workspace
        weights, chosen, sw = self._route(ctx, y, True)
        hs = ws.get("experts_hs", (n, self.top * self.ff + self.shared), y.dtype)
        if self.gated:
            ops.expert_rows_gated_up(y, self.up.weight, chosen, weights, self.ff, self.shared, self.gate_terms, hs, sw)
        else:
            ops.expert_rows_up(y, self.up.weight, chosen, weights, self.ff, self.shared, self.activation, hs, shared_weight=sw)
        ops.expert_rows_down(hs, self.down.weight, chosen, self.E, self.ff, self.shared, out, accumulate)

    def many_rows(self, ctx, y: torch.Tensor) -> bool:
        """Do the rows of `y` run expert by expert over each expert's own rows?"""
        n = y.shape[0]
        return (y.dtype == torch.bfloat16 and self.up.weight.dtype == self.down.weight.dtype == torch.bfloat16
                and n * self.top >= GROUPED_ROWS_PER_EXPERT * self.E and not self.up.own_kernels(n)
                and not ctx.host.get("fixed_launches"))

    def _grouped(self, ctx, y: torch.Tensor, out: torch.Tensor, accumulate: bool) -> None:
        n, E, top, ff, H = y.shape[0], self.E, self.top, self.ff, self.H
        ws = ctx.workspace
        weights, chosen, sw = self._route(ctx, y, True)
        flat = chosen.view(-1).long()
        order = torch.argsort(flat, stable=True)                       # pairs by expert, a row's place kept within one
        counts = torch.bincount(flat, minlength=E).tolist()            # (the host waits for the router here)
        rows = torch.div(order, top, rounding_mode="floor")
        ys = y.index_select(0, rows)                                   # [n * top, H]
        scale = weights.gather(1, chosen.long()).view(-1).index_select(0, order).view(-1, 1).contiguous()
        up_w, down_w = self.up.weight, self.down.weight
        wide = 2 if self.gated else 1               # a gated expert's rows are [gate | up]
        u = ws.get("experts_gu", (n * top, wide * ff), torch.float32)
        at = 0
        for e, c in enumerate(counts):
            if c:
                ops.gemm(ys[at:at + c], up_w[wide * e * ff:wide * (e + 1) * ff], u[at:at + c])
                at += c
        h = ws.get("experts_gh", (n * top, ff), y.dtype)
        if self.gated:
            ops.expert_gated_act(u, scale, 1, ff, 0, self.gate_terms, h)
        else:
            ops.expert_act(u, scale, 1, ff, self.activation, h)
        z = ws.get("experts_gz", (n * top, H), torch.float32)
        at = 0
        for e, c in enumerate(counts):
            if c:
                torch.mm(h[at:at + c], down_w[:, e * ff:(e + 1) * ff].t(), out_dtype=torch.float32, out=z[at:at + c])
                at += c
        back = torch.empty_like(order)
        back[order] = torch.arange(n * top, device=order.device)
        total = z.index_select(0, back).view(n, top, H).sum(dim=1)     # a row's experts in the order it chose them
        if self.shared:
            us = ws.get("experts_su", (n, wide * self.shared), torch.float32)
            ops.gemm(y, up_w[wide * E * ff:], us)
            hs = ws.get("experts_sh", (n, self.shared), y.dtype)
            if self.gated:
                ops.expert_gated_act(us, None, 0, 0, self.shared, self.gate_terms, hs, sw)
            else:
                ops.expert_act(us, None, 0, self.shared, self.activation, hs, shared_weight=sw)
            total.add_(torch.mm(hs, down_w[:, E * ff:].t(), out_dtype=torch.float32))
        if accumulate:
            out.add_(total)
        else:
            out.copy_(total)

    def _hidden(self, ctx, y: torch.Tensor) -> torch.Tensor:
        n = y.shape[0]
        ws = ctx.workspace
        weights, _, sw = self._route(ctx, y, False)
        u = ws.get("experts_u", (n, (2 if self.gated else 1) * self.total), torch.float32)
        self.up(y, u)
        h = ws.get("experts_h", (n, self.total), ctx.dtype)
        if self.gated:
            ops.expert_gated_act(u, weights, self.E, self.ff, self.shared, self.gate_terms, h, sw)
        else:
            ops.expert_act(u, weights, self.E, self.ff, self.activation, h, shared_weight=sw)
        return h

    def forward(self, ctx, y: torch.Tensor, x: torch.Tensor) -> None:
        if self.few_rows(y):
            flush_pending(ctx, x)
            self._rows(ctx, y, x, True)
            return
        if self.many_rows(ctx, y):
            flush_pending(ctx, x)
            self._grouped(ctx, y, x, True)
            return
        self.down.add_into(self._hidden(ctx, y), x, ctx, "experts_down_parts")

    def produce(self, ctx, y: torch.Tensor, out: torch.Tensor) -> None:
        if self.few_rows(y):
            self._rows(ctx, y, out, False)
            return
        if self.many_rows(ctx, y):
            self._grouped(ctx, y, out, False)
            return
        self.down(self._hidden(ctx, y), out)


register_part("ffn", "plain", PlainFeedForward)
register_part("ffn", "routed_experts", RoutedExperts)
