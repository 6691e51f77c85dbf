"""Attention whose cache keeps a latent per position, not keys and values per head.

With h the mixer's input, rms(t) = t / sqrt(mean(t^2) + eps) and H heads:

    q_h = [q_n (head_dim) | q_r (rot_dim)] of W_q h                (or of W_uq (rms(W_dq h) * w_q), `q_rank`)
    [a (kv_rank) | b (rot_dim)] = W_dkv h ,  c = rms(a) * w_c
    k_h = [W_uk[h] c | b rotated] ,  v_h = W_uv[h] c
    s_h(p, j) = (q_h(p) . k_h(j)) * scale        over the visible keys (causal, optional window)
    out = W_o concat_h(softmax(s_h) v_h)

q_r is rotated by its position and b by its own (`position`, which sees rot_dim channels); the rotated
key part is one for all heads.  A position keeps [c | b rotated], kv_rank + rot_dim numbers
(`KVRequest` of one head without values).

A step in which every sequence brings one token never makes keys or values per head: with q_n taken
through W_uk[h]^T into the latent's channels, the scores are products with the cached rows
themselves, the softmax's weights sum up the latents, and W_uv[h] follows on the sum.  A step with
more rows makes keys and values per head of its own rows, and of the cached positions that it
looks back to, for the time of the layer, and attends as `attend_and_commit` does: with n rows
that is the cheaper order.  The cached rows are then taken before the step's own are committed.
Scores, softmax weights and the norm are float32 in both dtypes.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..cache.cache import PAGE, KVRequest
from ..kernels import ops
from ..weights.binding import WeightSpec
from .base import Mixer, PartSpec, flush_pending, make_part, register_part
from .linear import Linear


class LatentCacheAttentionMixer(Mixer):
    graph_safe = True

    NAMES = {"q": "q", "dq": "dq", "dq_norm": "dq.norm", "uq": "uq", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk",
             "uv": "uv", "o": "o"}

    def __init__(self, hidden_size: int, n_heads: int, head_dim: int, v_head_dim: int, kv_rank: int, scale: float,
                 norm_eps: float, rot_dim: int = 0, position: Optional[PartSpec] = None, window: Optional[int] = None,
                 q_rank: Optional[int] = None, prefix: str = "mix.", names: Optional[Dict[str, str]] = None):
        unknown = set(names or {}) - set(self.NAMES)
        if unknown:
            raise ValueError(f"latent attention: no tensors called {sorted(unknown)}; there are {sorted(self.NAMES)}")
        if rot_dim % 2 or not 0 <= rot_dim <= ops.LATENT_MAX_ROT or not 1 <= kv_rank <= ops.LATENT_MAX_R:
            raise ValueError(f"latent attention: a latent of {kv_rank} with {rot_dim} rotated channels is not served "
                             f"(up to {ops.LATENT_MAX_R} and {ops.LATENT_MAX_ROT}, the latter even)")
        self.names = dict(self.NAMES, **(names or {}))
        self.H, self.nq, self.dn, self.dr = int(hidden_size), int(n_heads), int(head_dim), int(rot_dim)
        self.dk, self.dv, self.R = self.dn + self.dr, int(v_head_dim), int(kv_rank)
        self.qr = int(q_rank) if q_rank else 0
        self.scale, self.eps = float(scale), float(norm_eps)
        self.window = int(window) if window else None
        self.position = make_part("position", position if position is not None else PartSpec("none"))
        self.prefix = prefix
        self.down = self.uq = self.ukv = self.o = None

    # ---- what it keeps -------------------------------------------------------
    def kv_request(self):
        return KVRequest(1, self.R + self.dr, self.window, 0)

    def kv_reach(self):
        return self.window

    def may_capture(self, n_rows: int) -> bool:
        return self.down is not None and all(l.own_kernels(n_rows) for l in (self.down, self.uq, self.ukv, self.o) if l is not None)

    def prefers_eager(self, n_new, len_before, device) -> bool:
        return any(int(c) > 0 for c in len_before)       # cached rows are made into keys: as many as there are

    # ---- weights -------------------------------------------------------------
    def weight_specs(self) -> Dict[str, WeightSpec]:
        p, nm = self.prefix, self.names
        Q = self.nq * self.dk
        if self.qr:
            out = {p + nm["dq"]: WeightSpec((self.qr, self.H)), p + nm["dq_norm"]: WeightSpec((self.qr,), init="ones"),
                   p + nm["uq"]: WeightSpec((Q, self.qr))}
        else:
            out = {p + nm["q"]: WeightSpec((Q, self.H))}
        out.update({p + nm["dkv"]: WeightSpec((self.R + self.dr, self.H)), p + nm["dkv_norm"]: WeightSpec((self.R,), init="ones"),
                    p + nm["uk"]: WeightSpec((self.nq * self.dn, self.R)), p + nm["uv"]: WeightSpec((self.nq * self.dv, self.R)),
                    p + nm["o"]: WeightSpec((self.H, self.nq * self.dv))})
        return out

    def load(self, tensors, compute_dtype) -> None:
        p, nm = self.prefix, self.names

        def t(key):
            return tensors[p + nm[key]]

        def fused(keys):
            ws = [t(k) for k in keys]
            if len({w.dtype for w in ws}) > 1:
                ws = [w.to(torch.float32) for w in ws]
            return torch.cat(ws, dim=0)

        self.down = Linear(fused(["dq" if self.qr else "q", "dkv"]), tiled=True)       # rows [q or its latent | a | b]
        self.uq = Linear(t("uq"), tiled=True) if self.qr else None
        self.wq = t("dq_norm").to(torch.float32).contiguous() if self.qr else None
        self.wc = t("dkv_norm").to(torch.float32).contiguous()
        self.ukv = Linear(fused(["uk", "uv"]))
        self.o = Linear(t("o"), tiled=True)
        # single tokens: W_uk[h]^T [H, R, head_dim] and W_uv[h] [H, v_head_dim, R], in the compute dtype
        uk = t("uk").to(compute_dtype).view(self.nq, self.dn, self.R)
        self.uk_t = uk.transpose(1, 2).contiguous()
        self.uv = t("uv").to(compute_dtype).view(self.nq, self.dv, self.R).contiguous()

    # ---- one step --------------------------------------------------------------
    def produce(self, ctx, run, y: torch.Tensor, out: torch.Tensor):
        n, nq, dn, dr, dv, R = y.shape[0], self.nq, self.dn, self.dr, self.dv, self.R
        ws = ctx.workspace
        first = self.qr or nq * self.dk
        proj = ws.get("latc_proj", (n, first + R + dr), torch.float32)
        self.down(y, proj)
        cf = proj[:, first:]
        if self.qr:
            a = ws.get("latc_a", (n, self.qr), torch.float32)
            a.copy_(proj[:, :first])
            cq = ws.get("latc_cq", (n, self.qr), ctx.dtype)
            ops.rmsnorm(a, self.wq, self.eps, cq)
            qf = ws.get("latc_qf", (n, nq * self.dk), torch.float32)
            self.uq(cq, qf)
        else:
            qf = proj[:, :first]
        rotation = (self.position.rotation(y.device) or ops.NO_ROTATION) if dr else ops.NO_ROTATION
        att = ws.get("latc_att", (n, nq, dv), ctx.dtype)
        group = run.kv_group
        pages, table = group.storage[run.kv_layer], ctx.tables[run.kv_group_index]
        if ctx.all_single:
            qn = ws.get("latc_qn", (n, nq, dn), ctx.dtype)
            ql = ws.get("latc_ql", (n, nq, R + dr), ctx.dtype)         # q in the cached rows' channels
            ops.latent_prepare(qf, cf, ctx.row_pos, rotation, nq, dn, dr, self.wc, self.eps, qn, ql[:, :, R:], None, None,
                               table=table, ring_pages=group.ring_pages, pages=pages)
            ops.head_products(qn, self.uk_t, ql[:, :, :R])
            cs = ws.get("latc_cs", (n, nq, R), ctx.dtype)
            ops.latent_attention(ql, pages, table, group.ring_pages, ctx, dr, self.window, self.scale, cs)
            ops.head_products(cs, self.uv, att)
        else:
            q = ws.get("latc_q", (n, nq, self.dk), ctx.dtype)
            c = ws.get("latc_c", (n, R), ctx.dtype)
            rows = ws.get("latc_rows", (n, R + dr), ctx.dtype)
            ops.latent_prepare(qf, cf, ctx.row_pos, rotation, nq, dn, dr, self.wc, self.eps, q[:, :, :dn], q[:, :, dn:], c, rows)
            kvf = ws.get("latc_kvf", (n, nq * (dn + dv)), torch.float32)
            self.ukv(c, kvf)
            k = ws.get("latc_k", (n, nq, self.dk), ctx.dtype)
            v = ws.get("latc_v", (n, nq, dv), ctx.dtype)
            ops.latent_heads(kvf, rows[:, R:], nq, dn, dr, dv, k, v)
            old, old_table = self._cached_heads(ctx, group, run.kv_group_index, pages, table)
            ops.attend_heads(ctx, q, k, v, old, old_table, group.ring_pages, self.window, self.scale, att)
            ops.latent_commit(rows, ctx.row_seq, ctx.row_pos, ctx.len_after, table, group.ring_pages, pages)
        self.o(att.view(n, nq * dv), out)
        return None

    def _cached_heads(self, ctx, group, index: int, pages: torch.Tensor, table: torch.Tensor):
        """Keys and values per head of the positions that the step's sequences hold already, in pages of the usual kind
        (in the workspace, for this layer alone), and a page table for them."""
        nq, dn, dr, dv, R = self.nq, self.dn, self.dr, self.dv, self.R
        ws = ctx.workspace
        size = nq * PAGE * (self.dk + dv)
        before = [] if ctx.host.get("fixed_launches") else [int(x) for x in ctx.host["len_before"]]
        if not any(before):
            return ws.get("latc_old", (1, size), ctx.dtype), table       # nothing is read of either
        at = ("latent_pages", index)
        if at not in ctx.host:                                           # the same for every layer of the group
            held = [group.pages_needed(x) for x in before]
            width, B = max(held), len(held)
            off = [0]
            for m in held:
                off.append(off[-1] + m)
            flat = off + [off[b] + min(i, held[b] - 1) if held[b] else 0 for b in range(B) for i in range(width)]
            dev = torch.tensor(flat, dtype=torch.int32).to(pages.device)
            ctx.host[at] = (off[-1], dev[:B + 1], dev[B + 1:].view(B, width))
        total, off, old_table = ctx.host[at]
        c = ws.get("latc_old_c", (total * PAGE, R), ctx.dtype)
        kr = ws.get("latc_old_kr", (total * PAGE, dr), ctx.dtype) if dr else None
        ops.latent_gather(pages, table, off, total, c, kr)
        kvf = ws.get("latc_old_kvf", (total * PAGE, nq * (dn + dv)), torch.float32)
        self.ukv(c, kvf)
        old = ws.get("latc_old", (total, size), ctx.dtype)
        ops.latent_heads_pages(kvf, kr, nq, dn, dr, dv, old)
        return old, old_table

    def forward(self, ctx, run, y: torch.Tensor, x: torch.Tensor) -> None:
        flush_pending(ctx, x)
        z = ctx.workspace.get("latc_z", tuple(x.shape), torch.float32)
        self.produce(ctx, run, y, z)
        ops.add_partials(x, z.view(1, *z.shape))


register_part("mixer", "latent_cache_attention", LatentCacheAttentionMixer)
