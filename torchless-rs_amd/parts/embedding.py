"""Token embedding (a row copy, no scaling: src/model/modules/embedding.rs:15-21
of the reference; `scale` multiplies the row for designs that have one) and the
output head (logits = W x, its own tensor unless the configuration ties it to the
embedding: src/model/mod.rs:364-369, 443-446; `scale` multiplies the logits)."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..cache.cache import StateRequest
from ..kernels import ops
from ..weights.binding import WeightSpec
from .base import Embedding, Part, PartSpec, StreamPart, make_part, register_part
from .linear import Linear
from .projected import same_dtype


class TokenEmbedding(Embedding):
    graph_safe = True

    def __init__(self, vocab_size: int, hidden_size: int, name: str = "embed_tokens.weight", scale: float = 1.0):
        self.V, self.H, self.name, self.scale = int(vocab_size), int(hidden_size), name, float(scale)
        self.table = None

    def weight_specs(self) -> Dict[str, WeightSpec]:
        return {self.name: WeightSpec((self.V, self.H))}

    def load(self, tensors, compute_dtype) -> None:
        self.table = tensors[self.name]

    def forward(self, ctx, ids: torch.Tensor, x: torch.Tensor, state=None) -> None:
        ops.embed(self.table, ids, x, self.scale)


class PairEmbedding(Embedding):
    """A token's row times `scale`, plus a row of a second table that the pair of the previous and the present token picks,
    (previous * mul_prev + present * mul_cur) mod `buckets`, the table's last row (number `buckets`) for a sequence's first
    token (`buckets` None: no such table), and then a norm (`norm`, an RMS norm's `PartSpec`; None: none): one kernel.
    What a sequence keeps is its last token."""
    graph_safe = True

    def __init__(self, vocab_size: int, hidden_size: int, buckets: Optional[int] = None, mul_prev: int = 0,
                 mul_cur: int = 0, name: str = "embed",
                 pair_name: str = "bigram", scale: float = 1.0, norm: Optional[PartSpec] = None, norm_prefix: str = "embed.norm"):
        if (buckets is not None and buckets < 1) or mul_prev < 0 or mul_cur < 0:
            raise ValueError(f"embedding: {buckets} buckets with the factors {mul_prev} and {mul_cur}")
        self.V, self.H, self.name, self.scale = int(vocab_size), int(hidden_size), name, float(scale)
        self.buckets = None if buckets is None else int(buckets)
        self.mul_prev, self.mul_cur, self.pair_name = int(mul_prev), int(mul_cur), pair_name
        self.norm = make_part("norm", norm) if norm is not None else None
        self.norm_prefix = norm_prefix
        self.table = self.pairs = None

    def state_request(self):
        return StateRequest((1,), torch.int32) if self.buckets is not None else None

    def weight_specs(self) -> Dict[str, WeightSpec]:
        out = {self.name: WeightSpec((self.V, self.H))}
        if self.buckets is not None:
            out[self.pair_name] = WeightSpec((self.buckets + 1, self.H))
        if self.norm is not None:
            out.update({self.norm_prefix + k: v for k, v in self.norm.weight_specs().items()})
        return out

    def load(self, tensors, compute_dtype) -> None:
        self.table = tensors[self.name]
        if self.buckets is not None:
            self.table, pairs = same_dtype([self.table, tensors[self.pair_name]])
            self.pairs = ops.PairTable(pairs, self.buckets, self.mul_prev, self.mul_cur)
        if self.norm is not None:
            p = self.norm_prefix
            self.norm.load({k[len(p):]: v for k, v in tensors.items() if k.startswith(p)}, compute_dtype)
            if self.norm.rms_form() is None:
                raise ValueError("embedding: the norm behind it must be an RMS norm")

    def forward(self, ctx, ids: torch.Tensor, x: torch.Tensor, state=None) -> None:
        form = self.norm.rms_form() if self.norm is not None else None
        ops.embed_pairs(self.table, ids, self.scale, self.pairs, ctx.row_pos, ctx.row_seq, ctx.cu_seqlens, ctx.slots, state,
                        form.weight if form else None, form.eps if form else 0.0, x)


class LMHead(Part):
    """`tied`: use the embedding table instead of a tensor of its own."""
    graph_safe = True

    def may_capture(self, n_rows: int) -> bool:
        return self.proj is not None and self.proj.own_kernels(n_rows)

    def __init__(self, vocab_size: int, hidden_size: int, tied: bool = False, name: str = "weight", scale: float = 1.0):
        self.V, self.H, self.tied, self.name = int(vocab_size), int(hidden_size), bool(tied), name
        self.scale = float(scale)
        self.proj = None

    def weight_specs(self) -> Dict[str, WeightSpec]:
        return {} if self.tied else {self.name: WeightSpec((self.V, self.H))}

    def load(self, tensors, compute_dtype) -> None:
        self.proj = Linear(tensors["__embedding__"] if self.tied else tensors[self.name])

    def forward(self, ctx, y: torch.Tensor, logits: torch.Tensor) -> None:
        self.proj(y, logits)
        if self.scale != 1.0:
            ops.scale_(logits, self.scale)


register_part("embedding", "tokens", TokenEmbedding)
register_part("embedding", "token_pairs", PairEmbedding)
register_part("head", "linear", LMHead)


class PassEntry(StreamPart):
    """What the stream receives at the start of each pass over a run of layers that is gone
    through several times with the same weights: before every pass but the first the
    embedding's output is added again (`add_embedding`), and before every pass, the first
    too, row t of a learned table [passes, hidden] (tensor `name`), t the number of the pass."""
    graph_safe = True

    def __init__(self, hidden_size: int, passes: int, name: str = "step", add_embedding: bool = True):
        self.H, self.passes, self.name = int(hidden_size), int(passes), name
        self.needs_embedding = bool(add_embedding) and self.passes > 1
        self.table = None

    def weight_specs(self) -> Dict[str, WeightSpec]:
        return {self.name: WeightSpec((self.passes, self.H))}

    def load(self, tensors, compute_dtype) -> None:
        self.table = tensors[self.name].to(torch.float32).contiguous()
        self.rows = [self.table[t] for t in range(self.passes)]

    def forward(self, ctx, x: torch.Tensor, embedded, t: int) -> None:
        if not (0 <= t < self.passes):
            raise ValueError(f"pass {t} of {self.passes}")
        ops.stream_entry(x, embedded if (t > 0 and self.needs_embedding) else None, self.rows[t])


register_part("stream", "pass_entry", PassEntry)
