"""Linear attention with a decay per head and key channel, plain or by the delta rule.

One product over the mixer's input gives a row of queries, keys, values and what the decays, the
write strengths and the gate come from.  Per head, with q, k, g of `head_dim` channels and v of
`v_head_dim` (S: [head_dim, v_head_dim], from zero):

    S <- diag(g) S ;  u = v, or with `delta` beta (v - S^T k) ;  S <- S + k u^T ;  o = S^T q
    out = W_o ( concat_h( o / sqrt(mean(o^2) + eps) * w ) * gate )

w being one head's weight that all heads share.  The terms are constructor parameters:

* `conv_taps`: q, k and v pass a causal convolution per channel over their last `conv_taps` rows (zeros
  before the start of a sequence) and silu (0: none);
* `unit_eps`: q and k of every head are made unit vectors, x / sqrt(sum(x^2) + unit_eps) (None: as they are);
* `scale` on q;
* heads share q and k in groups (`n_kv_heads` heads of them; head h reads number h / (H / n_kv_heads));
* `decay`: "softplus", g = exp(-exp(A_h) softplus(z)), A a tensor of a number per head, or "logistic",
  g = logistic(z)^(1 / tau), with z = W_a2 (W_a1 y) + b;
* `delta`: the delta rule with beta = logistic(W_b y), one per head;
* `gate`: "silu" of W_g y, or "logistic" of W_g2 (W_g1 y).

The inner sizes of the two-step projections are the tensors' own (`inner` is what a random model
gets).  What a sequence keeps (`StateRequest`) is of fixed size whatever its length: the convolution's
last inputs and the states, all float32; nothing per position.

Single tokens, short portions and the 32-bit path go row by row with everything between the two
products of the mixer in float32 (`ops.channel_rows`, `ops.channel_scan`); longer bfloat16 steps go by chunks of
rows on the matrix cores (`ops.channel_chunks`), the second steps of the projections as library products of
their inner rows in two bfloat16 terms.  In bfloat16 the gated result is rounded once.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..cache.cache import StateRequest
from ..kernels import ops
from ..weights.binding import WeightSpec
from .base import register_part
from .linear import Linear
from .projected import ProjectedMixer, same_dtype, stacked


CHUNKS_FROM = 32             # a bfloat16 step whose longest sequence brings this many rows goes by chunks
INNER_STEP = 64              # inner rows are padded to this many channels for the products by their second matrices


class SecondStep:
    """The second matrix [N, rank] of a two-step projection, for rows kept in float: the inner row in two bfloat16 terms
    [hi | lo] times [W | W]."""

    def __init__(self, weight: torch.Tensor):
        rank = weight.shape[1]
        self.pad = -(-rank // INNER_STEP) * INNER_STEP
        w = torch.zeros((weight.shape[0], 2 * self.pad), dtype=weight.dtype, device=weight.device)
        w[:, :rank] = weight
        w[:, self.pad:self.pad + rank] = weight
        self.w = Linear(w, tiled=False)

    def __call__(self, ctx, inner: torch.Tensor, out: torch.Tensor, name: str) -> None:
        terms = ctx.workspace.get(name, (inner.shape[0], 2 * self.pad), torch.bfloat16)
        ops.split_columns(inner, self.pad, terms)
        self.w(terms, out)


class ChannelLinearMixer(ProjectedMixer):
    tag = "clin"

    NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv", "beta": "b",
             "rate": "A_log", "norm": "norm", "decay_in": "a1", "decay_out": "a2", "decay_bias": "dt_bias", "gate": "g",
             "gate_in": "g1", "gate_out": "g2"}
    DECAYS = ("softplus", "logistic")
    GATES = ("silu", "logistic")

    def __init__(self, hidden_size: int, n_heads: int, head_dim: int, norm_eps: float, v_head_dim: Optional[int] = None,
                 n_kv_heads: Optional[int] = None, conv_taps: int = 0, unit_eps: Optional[float] = None,
                 scale: Optional[float] = None, decay: str = "softplus", tau: float = 1.0, delta: bool = False,
                 gate: str = "silu", inner: int = 16, prefix: str = "mix.", names: Optional[Dict[str, str]] = None):
        unknown = set(names or {}) - set(self.NAMES)
        if unknown:
            raise ValueError(f"linear attention: no tensors called {sorted(unknown)}; there are {sorted(self.NAMES)}")
        if decay not in self.DECAYS or gate not in self.GATES:
            raise ValueError(f"linear attention: decays are one of {self.DECAYS} and gates of {self.GATES}, got {decay!r}, {gate!r}")
        self.H, self.heads_n, self.dk = int(hidden_size), int(n_heads), int(head_dim)
        self.dv = self.dk if v_head_dim is None else int(v_head_dim)
        self.G = self.heads_n if n_kv_heads is None else int(n_kv_heads)
        if self.heads_n % self.G:
            raise ValueError(f"linear attention: {self.heads_n} heads are not a multiple of {self.G} heads of q and k")
        if not tau > 0:
            raise ValueError(f"linear attention: tau {tau} must be positive")
        self.names = dict(self.NAMES, **(names or {}))
        self.eps, self.taps, self.prefix, self.inner = float(norm_eps), int(conv_taps), prefix, int(inner)
        self.unit_eps = None if unit_eps is None else float(unit_eps)
        self.scale = self.dk ** -0.5 if scale is None else float(scale)
        self.decay, self.tau, self.delta, self.gate = decay, float(tau), bool(delta), gate
        self.channels = 2 * self.G * self.dk + self.heads_n * self.dv
        # the states start on a whole vector behind the convolution's rows
        self.conv_elems = -(-max(self.taps - 1, 0) * self.channels // 4) * 4
        self.state_elems = -(-self.heads_n * self.dk * self.dv // 4) * 4
        self.terms = self.norm_w = self.decay_step = self.gate_step = None

    def may_capture(self, n_rows: int) -> bool:
        return super().may_capture(n_rows) and self._steps_capture(n_rows)

    def _steps_capture(self, n_rows: int) -> bool:
        return all(s.w.own_kernels(n_rows) for s in (self.decay_step, self.gate_step) if s is not None)

    def state_request(self):
        return StateRequest((self.conv_elems + self.state_elems,), torch.float32)

    # ---- weights -------------------------------------------------------------
    def weight_specs(self) -> Dict[str, WeightSpec]:
        p, nm = self.prefix, self.names
        H, Q, K, V = self.H, self.G * self.dk, self.heads_n * self.dk, self.heads_n * self.dv
        out = {}
        for key, size in (("q", Q), ("k", Q), ("v", V)):
            out[p + nm[key]] = WeightSpec((size, H))
            if self.taps:
                out[p + nm[key + "_conv"]] = WeightSpec((size, self.taps))
        if self.delta:
            out[p + nm["beta"]] = WeightSpec((self.heads_n, H))
        if self.decay == "softplus":
            out[p + nm["rate"]] = WeightSpec((self.heads_n,))
        out[p + nm["norm"]] = WeightSpec((self.dv,), init="ones")
        out[p + nm["decay_in"]] = WeightSpec((self.inner, H), free=(0,))
        out[p + nm["decay_out"]] = WeightSpec((K, self.inner), free=(1,))
        out[p + nm["decay_bias"]] = WeightSpec((K,))
        if self.gate == "silu":
            out[p + nm["gate"]] = WeightSpec((V, H))
        else:
            out[p + nm["gate_in"]] = WeightSpec((self.inner, H), free=(0,))
            out[p + nm["gate_out"]] = WeightSpec((V, self.inner), free=(1,))
        out[p + nm["o"]] = WeightSpec((H, V))
        return out

    def load_terms(self, tensors, compute_dtype):
        p, nm = self.prefix, self.names

        def t(key):
            return tensors[p + nm[key]]

        def f32(key):
            return t(key).to(torch.float32).contiguous()

        two_step = self.gate == "logistic"
        for a, b in [("decay_in", "decay_out")] + ([("gate_in", "gate_out")] if two_step else []):
            if t(a).shape[0] != t(b).shape[1]:
                raise ValueError(f"linear attention: {p + nm[a]} gives {t(a).shape[0]} channels, {p + nm[b]} takes {t(b).shape[1]}")
        keys = ["q", "k", "v"] + ([] if two_step else ["gate"]) + (["beta"] if self.delta else []) + ["decay_in"] + (
            ["gate_in"] if two_step else [])
        off, at = {}, 0
        for key in keys:
            off[key] = at
            at += t(key).shape[0]
        w_in = stacked([t(k) for k in keys])
        second = [m.contiguous() for m in same_dtype([t("decay_out")] + ([t("gate_out")] if two_step else []))]
        self.gate_off = off.get("gate")
        self.norm_w = f32("norm")
        self.decay_step = self.gate_step = None
        if ops.channel_chunks_serve(compute_dtype, self.dk, self.dv) and second[0].dtype == torch.bfloat16:
            self.decay_step = SecondStep(second[0])
            if two_step:
                self.gate_step = SecondStep(second[1])
        self.terms = ops.ChannelTerms(
            self.G, self.heads_n, self.dk, self.dv, off["decay_in"], second[0], f32("decay_bias"), off.get("beta"),
            off.get("gate_in"), second[1] if two_step else None,
            torch.cat([f32(k + "_conv") for k in "qkv"], dim=0).contiguous() if self.taps else None,
            f32("rate") if self.decay == "softplus" else None, self.tau, self.scale, self.unit_eps)
        self.in_width, self.heads_width = w_in.shape[0], self.heads_n * self.dv
        return w_in, t("o")

    # ---- one step --------------------------------------------------------------
    def heads(self, ctx, run, proj: torch.Tensor, out: torch.Tensor) -> None:
        n, t, ws = proj.shape[0], self.terms, ctx.workspace
        f32 = torch.float32
        Q, K, V = self.G * self.dk, self.heads_n * self.dk, self.heads_n * self.dv
        conv_state, state = run.state[:, :self.conv_elems], run.state[:, self.conv_elems:]
        two_step = self.gate == "logistic"
        if ctx.max_new >= CHUNKS_FROM and self.decay_step is not None:
            z = ws.get("clin_decay", (n, K), f32)
            self.decay_step(ctx, proj[:, t.a_off:t.a_off + t.a2.shape[1]], z, "clin_inner")
            gate = proj[:, self.gate_off:self.gate_off + V] if not two_step else ws.get("clin_gate", (n, V), f32)
            if two_step:
                self.gate_step(ctx, proj[:, t.g_off:t.g_off + t.g2.shape[1]], gate, "clin_inner")
            C = ops.channel_chunk()
            chunks = int(sum(-(-int(r) // C) for r in ctx.host["n_new"]))
            ops.channel_chunks(proj, t, z, conv_state, state, ctx.cu_seqlens, ctx.slots, chunks, ws, gate, self.eps, out,
                               weight=self.norm_w, silu=not two_step, factor=self.factor)
            return
        q, k, v = ws.get("clin_q", (n, Q), f32), ws.get("clin_k", (n, Q), f32), ws.get("clin_v", (n, V), f32)
        decay = ws.get("clin_decay", (n, K), f32)
        beta = ws.get("clin_beta", (n, self.heads_n), f32) if self.delta else None
        gate = ws.get("clin_gate", (n, V), f32) if two_step else proj[:, self.gate_off:self.gate_off + V]
        ops.channel_rows(proj, t, conv_state, ctx.row_seq, ctx.cu_seqlens, ctx.slots, ctx.all_single, q, k, v, decay, beta,
                         gate if two_step else None)
        if ctx.all_single:          # one token a sequence: the norm and the gate ride on the recurrence
            ops.channel_scan_gated(q, k, v, decay, beta, t, state, ctx.cu_seqlens, ctx.slots, gate, self.eps, out,
                                   weight=self.norm_w, silu=not two_step, factor=self.factor)
            return
        o = ws.get("clin_o", (n, V), f32)
        ops.channel_scan(q, k, v, decay, beta, t, state, ctx.cu_seqlens, ctx.slots, o)
        ops.heads_norm_gate(o, gate, self.heads_n, self.eps, out, weight=self.norm_w, silu=not two_step, factor=self.factor)


register_part("mixer", "channel_linear", ChannelLinearMixer)
