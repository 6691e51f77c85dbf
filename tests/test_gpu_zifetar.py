"""Zifetar on the GPU against the plain implementation of `plain_zifetar.py`: every new mechanism alone
(norms around one, the embedding of token pairs, the rows of a linear attention and its recurrence row by row
and by chunks, with states carried far, forgotten at once and written over, decays steep and flat, the norm with
weight and gate, the router with a bias, experts behind it, mixers side by side over pages that are rings with keys
made to stand out at every chunk's edge, the delta rule's whole mixer), then whole models of the tests' own sizes
through the engine: whole prompts, the stream after every layer, decoding token by token, portions down to two
tokens, unequal batches, slots, pages and states used again, long decoding, and greedy generation through the entry
point."""
import copy
import json
import math
import os
import random
import subprocess
import sys
import types

import numpy as np
import pytest
import torch

import plain_zifetar as plain
from test_gpu_sozetar import some_prompts, write_model
from test_zifetar_config import MIXED, delta, layer, model, moe, par, ret
from util import rel_err, rms_err

pytestmark = pytest.mark.gpu
REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
TOL = {"float32": 3e-5, "bfloat16": 6e-2}
RMS = {"float32": 1e-5, "bfloat16": 3.5e-2}
# a model whose sublayers have a handful of channels divides them by root mean squares that may be near zero
FEW_CHANNELS = {"ones": 3.0}
# a router's choice made by less than this may fall the other way under rounding (in bfloat16 every choice of these
# models is wider)
MARGIN = {"float32": 1e-4, "bfloat16": 1e-2}
# a row whose heads' terms have cancelled to less than this (terms of any sign: about 1) holds, behind the norm over the head,
# their rounding made large
LEFT = {"float32": 5e-3, "bfloat16": 0.4}
F64 = torch.float64

# sizes that fill the matrix cores' operands: heads of 64, 96 and 128, values wider and narrower, a convolution of 8 taps
CORES = model(256, 128, 1e-6, [
    layer(delta(2, 1, 128, 128, 4), moe(16, 2, 32)),
    layer(par((4, 2, 64, 64, 0.125, 129, (10000.0, 64, (8.0, 1.0, 4.0, 128))), (2, 64, 128, 16.0)), moe(8, 4, 32)),
    layer(delta(3, 3, 96, 200, 8), None),
    layer(par((2, 1, 128, 128, 0.09, 100, (500.0, 64)), (1, 128, 64, 4.0), (1.0, 0.5)), moe(8, 1, 64)),
    layer(ret(2, 128, 64, [0.998, 0.9], (1000.0, 128)), moe(4, 4, 32)),
])
# what a model may happen to make 1 or leave out: one head, one expert, top = experts, a chunk of one (a position sees itself
# alone) and of two, one tap, no rotation, no chunk, one bucket of pairs, a decay of 0 and of 1
ONES = model(96, 32, 1e-4, [
    layer(par((1, 1, 8, 8, 0.35, 1, (50.0, 8)), (1, 8, 8, 1.0), (1.0, 1.0)), moe(1, 1, 16)),
    layer(delta(1, 1, 8, 8, 1), moe(4, 4, 8)),
    layer(par((2, 1, 4, 8, 0.5, 2, None), (2, 4, 8, 2.0)), None),
    layer(ret(2, 8, 8, [0.0, 1.0], (50.0, 2)), moe(5, 2, 8)),
    layer(par((2, 2, 8, 8, 0.35, None, (50.0, 4)), (1, 8, 8, 16.0)), None),
    layer(delta(2, 1, 4, 8, 2), moe(3, 1, 8)),
], scale=1.0, pairs=(1, 1, 1))
# sizes that no kernel's fast way takes: an odd width and vocabulary, heads of 11 and 21, states of 13 x 7, inner sizes of 5 and 9,
# factors on tokens far beyond the buckets
ODD = model(131, 101, 1e-5, [
    layer(delta(3, 1, 13, 7, 5), moe(6, 2, 11)),
    layer(par((3, 3, 11, 21, 0.29, 33, (300.0, 6, (3.0, 0.7, 3.0, 40))), (5, 9, 11, 12.5), (-0.7, 1.1)), moe(9, 3, 10)),
    layer(ret(1, 20, 30, [0.97], (20.0, 20)), None),
    layer(par((4, 2, 10, 10, 0.3, 65, (1e6, 10)), (2, 33, 17, 3.0)), moe(7, 7, 6)),
    layer(delta(4, 4, 9, 33, 2), moe(8, 2, 12)),
], scale=0.5, pairs=(97, 2 ** 40 + 3, 123456789))
CONFIGS = {"mixed": MIXED, "cores": CORES, "ones": ONES, "odd": ODD}
LENGTHS = {"mixed": [1, 7, 33, 150], "cores": [5, 64, 129, 330], "ones": [2, 65, 130, 200], "odd": [4, 33, 67, 140]}
RANKS = {"mixed": (12, 8), "cores": (128, 16), "ones": (1, 2), "odd": (5, 9)}
NAMES = list(CONFIGS)


def dev(t, dtype=None):
    return t.to("cuda", dtype) if dtype is not None else t.to("cuda")


def step_ctx(dtype, **kw):
    from torchless_rs_amd.parts.base import Workspace
    return types.SimpleNamespace(pending=None, prenormed=None, norm_ahead=None, row_factor=None, dtype=TORCH[dtype],
                                 workspace=Workspace(torch.device("cuda")), host={}, **kw)


def cut_up(lengths, cuts):
    """Steps of several sequences: for every step [(sequence, first row, rows)], `cuts[i]` rows of each that still has some."""
    done, out = [0] * len(lengths), []
    for cut in cuts:
        step = []
        for i, n in enumerate(lengths):
            if done[i] < n:
                take = min(cut, n - done[i])
                step.append((i, done[i], take))
                done[i] += take
        if step:
            out.append(step)
    assert all(d == n for d, n in zip(done, lengths))
    return out


def batch(step, slots):
    """row_pos, row_seq, cu_seqlens and slots of a step on the GPU."""
    def ints(x):
        return torch.tensor(x, dtype=torch.int32, device="cuda")
    return (ints([r for _, at, n in step for r in range(at, at + n)]), ints([b for b, (_, _, n) in enumerate(step) for _ in range(n)]),
            ints(np.concatenate([[0], np.cumsum([n for _, _, n in step])])), ints([slots[i] for i, _, _ in step]))


# ---------------------------------------------------------------------------------------------
# norms and the embedding
# ---------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [30, 101, 320, 2052, 8200])
def test_norms_whose_weight_is_stored_as_its_difference_from_one(dtype, H):
    from torchless_rs_amd.parts.norms import RMSNorm
    g = torch.Generator().manual_seed(H)
    n = 5
    z, x = torch.randn(n, H, generator=g) * 3, torch.randn(n, H, generator=g)
    norms = []
    for i in range(2):
        w = (torch.randn(H, generator=g) * 0.4).to(torch.bfloat16)
        rn = RMSNorm(H, 1e-5 * (i + 1), name="", around_zero=True)
        rn.load({"": dev(w)}, TORCH[dtype])
        norms.append((rn, w.double()))
    (a, wa), (b, wb) = norms
    ctx = step_ctx(dtype)
    out = torch.empty(n, H, dtype=TORCH[dtype], device="cuda")
    a.forward(ctx, dev(z), out)
    tol = 1e-5 if dtype == "float32" else 1e-2
    want = plain.norm(z.double(), a.eps, wa)
    assert rel_err(out, want) < tol
    want_x = x.double() + want
    for then in (None, (b, out)):
        xs = dev(x.clone())
        ctx.prenormed = None
        a.add_to(ctx, dev(z.clone()), xs, then=then)
        assert rel_err(xs, want_x) < 1e-5
        if ctx.prenormed is not None:
            assert rel_err(out, plain.norm(want_x, b.eps, wb)) < tol


@pytest.mark.parametrize("table_dtype", DTYPES)
@pytest.mark.parametrize("H, buckets, mul_prev, mul_cur", [(32, 11, 5, 2), (101, 1, 1, 1), (4096, 997, 31, 17), (4100, 8, 2 ** 33 + 1, 0), (8196, 64, 0, 3)])
def test_the_embedding_of_token_pairs_in_steps_of_any_size(table_dtype, H, buckets, mul_prev, mul_cur):
    """A sequence's first token reads the last row, whatever the slot held before; the token before a portion is the one that
    the step before ended with."""
    from torchless_rs_amd.kernels import ops
    g = torch.Generator().manual_seed(H)
    V, eps, scale = 50, 1e-5, 3.5
    cfg = {"embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}, "norm": {"eps": eps}}
    w = {"embed": torch.randn(V, H, generator=g), "bigram": torch.randn(buckets + 1, H, generator=g), "embed.norm": 0.3 * torch.randn(H, generator=g)}
    w = {k: v.to(TORCH[table_dtype]) for k, v in w.items()}
    w64 = {k: v.double() for k, v in w.items()}
    seqs = some_prompts(V, [1, 9, 30], seed=H)
    want = [plain.embedding(w64, cfg, s) for s in seqs]
    pairs = ops.PairTable(dev(w["bigram"]), buckets, mul_prev, mul_cur)
    norm_w = dev((1.0 + w["embed.norm"].float()))
    slots = [4, 0, 2]
    for cuts in ([30], [1] * 30, [2, 7, 1, 20]):
        last = torch.full((6, 1), 10 ** 9, dtype=torch.int32, device="cuda")
        got = [[] for _ in seqs]
        for step in cut_up([len(s) for s in seqs], cuts):
            pos, seq, cu, sl = batch(step, slots)
            ids = torch.tensor([seqs[i][r] for i, at, n in step for r in range(at, at + n)], dtype=torch.int32, device="cuda")
            out = torch.empty(len(ids), H, device="cuda")
            ops.embed_pairs(dev(w["embed"]), ids, scale, pairs, pos, seq, cu, sl, last, norm_w, eps, out)
            at = 0
            for i, _, n in step:
                got[i].append(out[at:at + n].clone())
                at += n
        for i in range(3):
            assert rel_err(torch.cat(got[i]), want[i]) < 2e-6, (cuts, i)
            assert int(last[slots[i]]) == seqs[i][-1]
        assert (last[[1, 3, 5]] == 10 ** 9).all()
    out = torch.empty(30, H, device="cuda")
    ids = torch.tensor(seqs[2], dtype=torch.int32, device="cuda")
    step = [(2, 0, 30)]
    ops.embed_pairs(dev(w["embed"]), ids, scale, None, *batch(step, slots), None, norm_w, eps, out)          # no pairs
    assert rel_err(out, plain.embedding(w64, {"embedding": {"scale": scale}, "norm": {"eps": eps}}, seqs[2])) < 2e-6
    ops.embed_pairs(dev(w["embed"]), ids, scale, pairs, *batch(step, slots), last, None, 0.0, out)            # no norm
    raw = w64["embed"][seqs[2]] * scale + w64["bigram"][plain.pair_rows(seqs[2], cfg["embedding"]["bigram"])]
    assert rel_err(out, raw) < 2e-6


# ---------------------------------------------------------------------------------------------
# linear attention with a decay per channel
# ---------------------------------------------------------------------------------------------

class Linear:
    """Random terms of a linear attention and rows of its projection: [q | k | v | beta | decays' inner row | gate's inner row |
    gate]."""

    def __init__(self, rule, G, H, dk, dv, taps, rank, seed, steep=0.0, g_rank=0):
        from torchless_rs_amd.kernels import ops
        self.delta = rule == "delta"
        self.G, self.H, self.dk, self.dv, self.taps, self.rank, self.g_rank = G, H, dk, dv, taps, rank, g_rank
        self.C = 2 * G * dk + H * dv
        self.b_off, self.a_off = self.C, self.C + H
        self.g_off = self.a_off + rank
        self.gate_off = self.g_off + g_rank
        self.width = self.gate_off + H * dv
        g = torch.Generator().manual_seed(seed)
        self.gen = g
        self.a2 = (torch.randn(H * dk, rank, generator=g) / math.sqrt(rank)).bfloat16()
        self.g2 = (torch.randn(H * dv, g_rank, generator=g) / math.sqrt(g_rank)).bfloat16() if g_rank else None
        self.bias = torch.randn(H * dk, generator=g) * 1.5 - 2.0 + steep
        self.rate = torch.randn(H, generator=g) * 0.7 - 0.5 + steep if self.delta else None
        self.conv = 0.5 * torch.randn(self.C, taps, generator=g) if taps else None
        self.tau, self.qscale, self.unit_eps = 4.0, dk ** -0.5, 1e-6 if self.delta else None
        self.norm_w = torch.randn(dv, generator=g)
        self.conv_elems = -(-max(taps - 1, 0) * self.C // 4) * 4
        self.block = self.conv_elems + H * dk * dv

        def on(t):
            return None if t is None else dev(t)
        self.terms = ops.ChannelTerms(G, H, dk, dv, self.a_off, on(self.a2), on(self.bias), self.b_off if self.delta else None,
                                      self.g_off if g_rank else None, on(self.g2), on(self.conv), on(self.rate), self.tau, self.qscale,
                                      self.unit_eps)

    def rows(self, n):
        return torch.randn(n, self.width, generator=self.gen)

    def inputs(self, x):
        """q, k, v, decays, beta and the gate of one sequence's rows, per head."""
        x = x.double()
        T, G, H, dk, dv = len(x), self.G, self.H, self.dk, self.dv
        u = x[:, :self.C]
        if self.taps:
            u = plain.short_conv(u, self.conv.double())
        q, k, v = u[:, :G * dk].reshape(T, G, dk), u[:, G * dk:2 * G * dk].reshape(T, G, dk), u[:, 2 * G * dk:].reshape(T, H, dv)
        if self.delta:
            q, k = plain.unit(q), plain.unit(k)
        z = x[:, self.a_off:self.a_off + self.rank] @ self.a2.double().T + self.bias.double()
        if self.delta:
            g = torch.exp(-torch.exp(self.rate.double())[:, None] * plain.softplus(z).view(T, H, dk))
        else:
            g = torch.sigmoid(z).pow(1.0 / self.tau).view(T, H, dk)
        beta = torch.sigmoid(x[:, self.b_off:self.b_off + H]) if self.delta else None
        gate = x[:, self.g_off:self.g_off + self.g_rank] @ self.g2.double().T if self.g_rank else x[:, self.gate_off:]
        return ((q * self.qscale).repeat_interleave(H // G, dim=1), k.repeat_interleave(H // G, dim=1), v, g, beta), gate

    def want(self, x, eps, factor=1.0):
        args, gate = self.inputs(x)
        o, S = plain.linear_heads(*args)
        act = torch.sigmoid(gate) if self.g_rank else plain.silu(gate)
        return (plain.rms(o, eps) * self.norm_w.double()).reshape(len(x), -1) * act * factor, S.transpose(1, 2)

    def run(self, way, dtype, seqs, cuts, slots, n_slots, eps, factor=1.0):
        """The gated results per sequence and the blocks, by `way` "rows" (and single tokens in one kernel) or "chunks"."""
        from torchless_rs_amd.kernels import ops
        from torchless_rs_amd.parts.base import Workspace
        from torchless_rs_amd.parts.channel_linear import SecondStep
        ws, t = Workspace(torch.device("cuda")), self.terms
        ctx = types.SimpleNamespace(workspace=ws)
        pitch = -(-self.block // 4) * 4 + 4
        block = torch.full((n_slots, pitch), float("nan"), device="cuda")[:, :self.block]        # strided rows
        for s in slots:
            block[s].zero_()
        conv, state = block[:, :self.conv_elems], block[:, self.conv_elems:]
        outs = [[] for _ in seqs]
        pad = torch.full((1, 24), float("nan"), device="cuda")
        nw, dt = dev(self.norm_w), TORCH[dtype]
        for step in cut_up([len(s) for s in seqs], cuts):
            _, seq, cu, sl = batch(step, slots)
            wide = torch.cat([dev(torch.cat([seqs[i][at:at + n] for i, at, n in step])), pad.expand(sum(n for _, _, n in step), 24)], dim=1)
            proj = wide[:, :self.width]                                                         # columns of a wider product
            n = proj.shape[0]
            hv = self.H * self.dv
            res = torch.full((n, hv + 8), 7.0, dtype=dt, device="cuda")
            out = res[:, 8:] if way == "rows" else res[:, :hv]

            def f32(size):
                return torch.empty(n, size, device="cuda")
            gate = f32(hv) if self.g_rank else proj[:, self.gate_off:]
            if way == "chunks":
                z = f32(self.H * self.dk)
                SecondStep(dev(self.a2))(ctx, proj[:, self.a_off:self.a_off + self.rank], z, "inner")
                if self.g_rank:
                    SecondStep(dev(self.g2))(ctx, proj[:, self.g_off:self.g_off + self.g_rank], gate, "inner")
                C = ops.channel_chunk()
                ops.channel_chunks(proj, t, z, conv, state, cu, sl, sum(-(-m // C) for _, _, m in step), ws, gate, eps, out, weight=nw,
                                   silu=not self.g_rank, factor=factor)
            else:
                q, k, v, d = f32(self.G * self.dk), f32(self.G * self.dk), f32(hv), f32(self.H * self.dk)
                beta = f32(self.H) if self.delta else None
                single = all(m == 1 for _, _, m in step)
                ops.channel_rows(proj, t, conv, seq, cu, sl, single, q, k, v, d, beta, gate if self.g_rank else None)
                if single:
                    ops.channel_scan_gated(q, k, v, d, beta, t, state, cu, sl, gate, eps, out, weight=nw, silu=not self.g_rank, factor=factor)
                else:
                    o = f32(hv)
                    ops.channel_scan(q, k, v, d, beta, t, state, cu, sl, o)
                    ops.heads_norm_gate(o, gate, self.H, eps, out, weight=nw, silu=not self.g_rank, factor=factor)
            at = 0
            for i, _, m in step:
                outs[i].append(out[at:at + m].clone())
                at += m
            assert (res[:, :8] == 7.0).all() if way == "rows" else (res[:, hv:] == 7.0).all()
        return [torch.cat(o) for o in outs], block

    def state(self, block, slot):
        return block[slot, self.conv_elems:].view(self.H, self.dv, self.dk)


ROW_SHAPES = [("delta", 1, 1, 1, 1, 1, 1, 0), ("delta", 1, 3, 13, 7, 5, 5, 9), ("delta", 2, 4, 32, 48, 3, 24, 16), ("delta", 2, 2, 128, 128, 4, 128, 128),
              ("delta", 1, 2, 200, 256, 8, 40, 0), ("plain", 3, 3, 20, 28, 0, 16, 0), ("plain", 2, 2, 64, 64, 0, 7, 0), ("plain", 1, 2, 256, 12, 2, 64, 32)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rule, G, H, dk, dv, taps, rank, g_rank", ROW_SHAPES)
def test_linear_attention_row_by_row_in_steps_of_any_size(dtype, rule, G, H, dk, dv, taps, rank, g_rank):
    lin = Linear(rule, G, H, dk, dv, taps, rank, seed=dk + dv, g_rank=g_rank)
    seqs = [lin.rows(n) for n in (1, 21, 40)]
    slots = [5, 0, 3]
    want = [lin.want(s, 1e-5, 1.5) for s in seqs]
    tol = 2e-5 if dtype == "float32" else 6e-3
    for cuts in ([40], [1] * 5 + [13] + [2] * 11, [1] * 40):
        got, block = lin.run("rows", dtype, seqs, cuts, slots, 7, 1e-5, 1.5)
        for i in range(3):
            assert rms_err(got[i], want[i][0]) < tol, (cuts, i)
            assert rel_err(lin.state(block, slots[i]), want[i][1]) < 2e-5, (cuts, i, "state")
        assert torch.isnan(block[[1, 2, 4, 6]]).all()           # nobody else's block was touched


@pytest.mark.parametrize("rule, G, H, dk, dv, taps, rank, g_rank, steep", [
    ("delta", 1, 1, 8, 4, 1, 4, 0, 0.0), ("delta", 2, 4, 32, 48, 3, 24, 16, 0.0), ("delta", 1, 2, 64, 64, 4, 64, 64, 0.0), ("delta", 2, 2, 128, 128, 4, 128, 128, 0.0),
    ("delta", 1, 2, 100, 200, 8, 40, 0, 0.0), ("delta", 2, 2, 64, 64, 4, 16, 0, 2.5), ("delta", 1, 1, 128, 32, 2, 16, 8, 1.5), ("plain", 3, 3, 20, 28, 0, 16, 0, 0.0),
    ("plain", 2, 2, 64, 256, 0, 16, 0, 0.0), ("plain", 1, 2, 128, 128, 0, 16, 0, 0.0), ("plain", 2, 2, 33, 64, 0, 16, 0, -30.0)])
def test_linear_attention_by_chunks_in_steps_of_any_size(rule, G, H, dk, dv, taps, rank, g_rank, steep):
    """The state carries 16 bits at least, in flat decays and in steep ones (blocks of 16 rows in which a channel decays by
    2^-60 and more take another way); chunks that begin and end anywhere, beside sequences that bring one row."""
    lin = Linear(rule, G, H, dk, dv, taps, rank, seed=dk, steep=steep, g_rank=g_rank)
    lens = (1, 63, 130, 290)
    seqs = [lin.rows(n) for n in lens]
    slots = [5, 0, 3, 6]
    want = [lin.want(s, 1e-5) for s in seqs]
    for cuts in ([290], [64, 128, 1, 100], [2, 31, 257], [65, 65, 65, 65, 65]):
        got, block = lin.run("chunks", "bfloat16", seqs, cuts, slots, 8, 1e-5)
        for i in range(len(lens)):
            assert rms_err(got[i], want[i][0]) < 6e-3, (cuts, i, rms_err(got[i], want[i][0]))
            assert rel_err(lin.state(block, slots[i]), want[i][1]) < 1e-4, (cuts, i, "state")
        assert torch.isnan(block[[1, 2, 4, 7]]).all()


def test_which_blocks_are_summed_pair_by_pair():
    """The sizes above reach both ways: a block of 16 rows is steep if some channel decays by more than 2^-60 in it."""
    found = set()
    for steep in (0.0, 2.5):
        lin = Linear("delta", 2, 2, 64, 64, 4, 16, seed=64, steep=steep)
        (_, _, _, g, _), _ = lin.inputs(lin.rows(64))
        found.add(bool((torch.log2(g).view(4, 16, 2, 64).sum(dim=1) < -60.0).any()))
    assert found == {True, False}


@pytest.mark.parametrize("way", ["rows", "chunks"])
@pytest.mark.parametrize("rule", ["delta", "plain"])
def test_a_row_that_is_carried_far_and_one_that_is_forgotten_at_once(way, rule):
    """Head 0 never forgets, head 1 keeps nothing: the loud first row still shows after 300 rows in head 0 and nowhere in head 1,
    in steps of any size.  Its key's channel is written by no other row."""
    H, d, L = 2, 32, 300
    lin = Linear(rule, H, H, d, d, 0, 4, seed=2)
    lin.bias[:] = torch.tensor([-40.0, 40.0] if rule == "delta" else [60.0, -200.0]).repeat_interleave(d)
    lin.a2[:] = 0
    if rule == "delta":
        lin.rate[:] = 1.0
    lin.terms.bias.copy_(dev(lin.bias))
    lin.terms.a2.copy_(dev(lin.a2))
    if rule == "delta":
        lin.terms.rate.copy_(dev(lin.rate))
    p = lin.rows(L) * 2.0 ** -4
    Q = H * d
    p[:, :Q:d] = 1.0                                     # channel 0 of q: every row looks for what row 0 left there
    p[:, Q:2 * Q:d] = 0.0
    p[0, Q:2 * Q:d] = 8.0                                # ... and row 0 alone writes it
    p[0, 2 * Q:2 * Q + H * d] = 3.0
    p[:, lin.b_off:lin.b_off + H] = 2.0
    want, S = lin.want(p, 1e-6)
    quiet = p.clone()
    quiet[0, 2 * Q:2 * Q + H * d] = 0.0
    other = lin.want(quiet, 1e-6)[0]
    assert rel_err(other[-1, :d], want[-1, :d]) > 0.3 and rel_err(other[-1, d:], want[-1, d:]) < 1e-9
    for cuts in ([300], [1] * 30 + [120, 150], [63, 2, 235]):
        got, block = lin.run(way, "bfloat16", [p], cuts, [2], 3, 1e-6)
        assert rms_err(got[0], want) < 6e-3, cuts
        assert rel_err(lin.state(block, 2), S) < 1e-4


@pytest.mark.parametrize("way", ["rows", "chunks"])
def test_a_second_write_to_a_key_replaces_the_first_and_a_row_reads_its_own_write(way):
    """Keys and queries along one channel each, no decay, beta near 1: every row's read-out is its own value, and at the end the
    state holds each channel's last value; anything that reads before it writes, or adds instead of replacing, shows."""
    d, L = 64, 200
    lin = Linear("delta", 1, 1, d, d, 0, 4, seed=3)
    lin.bias[:] = -60.0
    lin.a2[:] = 0
    lin.terms.bias.copy_(dev(lin.bias))
    lin.terms.a2.copy_(dev(lin.a2))
    p = lin.rows(L)
    g = torch.Generator().manual_seed(1)
    at = torch.randint(0, 9, (L,), generator=g)
    p[:, :2 * d] = 0.0
    p[torch.arange(L), at] = 1.0
    p[torch.arange(L), d + at] = 1.0
    p[:, lin.b_off] = 30.0
    want, S = lin.want(p, 1e-6)
    v = p[:, 2 * d:3 * d].double()
    last = torch.stack([v[torch.nonzero(at == c).max()] for c in range(9)])
    assert rel_err(S[0].T[:9], last) < 1e-5                      # (the plain one does what the name says)
    for cuts in ([L], [1] * 20 + [180], [70, 2, 128]):
        got, block = lin.run(way, "float32" if way == "rows" else "bfloat16", [p], cuts, [0], 1, 1e-6)
        assert rms_err(got[0], want) < (1e-5 if way == "rows" else 6e-3)
        assert rel_err(lin.state(block, 0).double().cpu()[0].T[:9], last) < 1e-4


@pytest.mark.parametrize("taps", [1, 2, 4, 8])
def test_the_last_inputs_of_a_convolution_are_carried_in_steps_of_any_size(taps):
    """Portions shorter than the taps, down to single tokens, leave the block that one whole step leaves."""
    lin = Linear("delta", 1, 2, 16, 24, taps, 8, seed=taps)
    seqs = [lin.rows(n) for n in (3, 37)]
    want = [lin.want(s, 1e-5)[0] for s in seqs]
    for way, cuts in (("rows", [37]), ("rows", [1, 1, 2, 1, 3, 29]), ("rows", [2] * 19), ("chunks", [1, 2, 34]), ("chunks", [37])):
        got, block = lin.run(way, "bfloat16" if way == "chunks" else "float32", seqs, cuts, [1, 0], 2, 1e-5)
        for i, s in enumerate(seqs):
            assert rms_err(got[i], want[i]) < (6e-3 if way == "chunks" else 1e-5), (way, cuts)
            kept = torch.cat([torch.zeros(taps, lin.C), s[:, :lin.C]])[-(taps - 1):] if taps > 1 else torch.zeros(0, lin.C)
            assert torch.equal(block[[1, 0][i], :(taps - 1) * lin.C].cpu().view(-1, lin.C), kept)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n, H, dv", [(1, 1, 1), (5, 3, 7), (40, 2, 64), (9, 4, 200)])
@pytest.mark.parametrize("silu", [True, False])
def test_the_norm_over_a_head_with_a_weight_and_a_gate(dtype, n, H, dv, silu):
    from torchless_rs_amd.kernels import ops
    g = torch.Generator().manual_seed(dv)
    o, gate, w = torch.randn(n, H * dv, generator=g) * 2, torch.randn(n, H * dv + 5, generator=g), torch.randn(dv, generator=g)
    wide = torch.full((n, H * dv + 3), 5.0, dtype=TORCH[dtype], device="cuda")
    ops.heads_norm_gate(dev(o), dev(gate)[:, 5:], H, 1e-3, wide[:, 3:], weight=dev(w), silu=silu, factor=-0.5)
    gt = gate[:, 5:].double()
    want = (plain.rms(o.double().view(n, H, dv), 1e-3) * w.double()).reshape(n, -1) * (plain.silu(gt) if silu else torch.sigmoid(gt)) * -0.5
    assert rel_err(wide[:, 3:], want) < (1e-5 if dtype == "float32" else 8e-3) and (wide[:, :3] == 5.0).all()


@pytest.mark.parametrize("n, cols, pad", [(1, 1, 64), (33, 24, 64), (200, 128, 128)])
def test_a_float_in_two_terms(n, cols, pad):
    from torchless_rs_amd.kernels import ops
    x = torch.randn(n, cols + 3, generator=torch.Generator().manual_seed(n))
    out = torch.empty(n, 2 * pad, dtype=torch.bfloat16, device="cuda")
    ops.split_columns(dev(x)[:, 3:], pad, out)
    hi, lo = out[:, :pad].double().cpu(), out[:, pad:].double().cpu()
    assert rel_err((hi + lo)[:, :cols], x[:, 3:]) < 2 ** -16 and (hi[:, cols:] == 0).all() and (lo[:, cols:] == 0).all()


# ---------------------------------------------------------------------------------------------
# the router
# ---------------------------------------------------------------------------------------------

@pytest.mark.parametrize("in_dtype", DTYPES)
@pytest.mark.parametrize("n", [3, 90])
@pytest.mark.parametrize("E, top", [(8, 3), (5, 5), (1, 1), (40, 7), (130, 2), (12, 1)])
def test_the_router_with_a_bias_and_weights_of_the_chosen_alone(in_dtype, n, E, top):
    from torchless_rs_amd.kernels import ops
    g = torch.Generator().manual_seed(E * 10 + top)
    W = 48
    h = torch.randn(n, W, generator=g).to(TORCH[in_dtype])
    w = {"router": (torch.randn(E, W, generator=g) * 0.4).double(), "router.b": (torch.randn(E, generator=g) * 2.0).double()}
    weights, chosen = torch.empty(n, E, device="cuda"), torch.empty(n, top, dtype=torch.int32, device="cuda")
    ops.route(dev(h), dev(w["router"].float()), 0, 0, top, weights, chosen, normalise_eps=0.0, bias=dev(w["router.b"].float()))
    margins = []
    want = plain.route(h.double(), w, "", top, margins)
    sure = margins[0] > 1e-4
    assert sure.float().mean() > 0.9
    assert rel_err(weights[sure.cuda()], want[sure]) < 1e-5
    assert torch.allclose(weights.sum(dim=1), torch.ones(n, device="cuda"), atol=1e-5)
    z = torch.gather(h.double() @ w["router"].T + w["router.b"], 1, chosen.long().cpu())
    assert (z[:, :-1] >= z[:, 1:] - 1e-4).all()               # the best first
    # without the bias the choice is another
    if 1 < E and top < E:
        ops.route(dev(h), dev(w["router"].float()), 0, 0, top, weights, None, normalise_eps=0.0)
        assert rel_err(weights[sure.cuda()], want[sure]) > 0.05


def test_far_logits_of_the_router():
    """Logits hundreds apart: the chosen one's weight is 1, and nothing is divided by zero."""
    from torchless_rs_amd.kernels import ops
    h, router = torch.ones(1, 4), torch.zeros(6, 4)
    bias = torch.tensor([-500.0, 300.0, 0.0, -200.0, 299.0, 900.0])
    out = torch.empty(1, 6, device="cuda")
    ops.route(dev(h), dev(router), 0, 0, 3, out, None, normalise_eps=0.0, bias=dev(bias))
    assert torch.allclose(out.cpu(), torch.tensor([[0.0, 0, 0, 0, 0, 1.0]]))
    ops.route(dev(h), dev(router), 0, 0, 2, out, None, normalise_eps=0.0, bias=dev(torch.tensor([-500.0, 300.0, 0.0, -200.0, 299.0, -900.0])))
    want = torch.softmax(torch.tensor([300.0, 299.0]), 0)
    assert torch.allclose(out.cpu()[0, [1, 4]], want, atol=1e-6) and abs(float(out.sum()) - 1.0) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, E, top, ff", [(64, 8, 2, 32), (101, 6, 2, 11), (32, 1, 1, 16), (48, 10, 1, 8), (40, 4, 4, 8)])
def test_experts_behind_the_router(dtype, H, E, top, ff):
    """The chosen experts alone (few rows), all side by side (more rows) and, in bfloat16, over each expert's own rows."""
    from torchless_rs_amd.parts.ffn_routed import RoutedExperts
    mlp = moe(E, top, ff)
    w = {k[3:]: v for k, v in plain.random_weights(model(8, H, 1e-5, [layer(ret(1, 1, 1, [0.5]), mlp)]), H + E, gain=2.0).items()
         if k.startswith("l0.mlp.")}
    part = RoutedExperts(H, E, top, ff, score="softmax", normalise_eps=0.0, router_bias=True, gated=True, activation="silu")
    assert set(part.weight_specs()) == set(w)
    part.load({k: dev(v if dtype == "bfloat16" else v.float()) for k, v in w.items()}, TORCH[dtype])
    w = {k: v.double() for k, v in w.items()}
    g = torch.Generator().manual_seed(E)
    tol = 2e-5 if dtype == "float32" else 2.5e-2
    for n in (1, 3, 40, 200):
        y = torch.randn(n, H, generator=g).to(TORCH[dtype])
        margins = []
        want = plain.routed_ff(y.double(), w, "mlp.", mlp, margins)
        sure = margins[0] > 1e-4
        out = torch.empty(n, H, device="cuda")
        ctx = step_ctx(dtype)
        part.produce(ctx, dev(y), out)
        assert rel_err(out[sure.cuda()], want[sure]) < tol, n
        if dtype == "bfloat16" and n == 200 and H % 8 == 0:
            part._grouped(ctx, dev(y), out, False)
            assert rel_err(out[sure.cuda()], want[sure]) < tol, (n, "expert by expert")


# ---------------------------------------------------------------------------------------------
# whole mixers over the cache
# ---------------------------------------------------------------------------------------------

def mixer_steps(part, w, dtype, seqs, cuts):
    """The mixer's results for several sequences' input rows in steps of any size, over a cache of its own whose pages and
    blocks hold NaN before they are taken."""
    from torchless_rs_amd.cache.cache import Cache
    from torchless_rs_amd.engine.engine import SeqInput, build_context
    from torchless_rs_amd.parts.base import RunBinding, Workspace
    kv, st = part.kv_request(), part.state_request()
    dt = TORCH[dtype]
    cache = Cache({0: kv} if kv else {}, {0: st} if st else {}, 64 * 40, dt, "cuda", max_slots=6)
    for grp in cache.groups:
        grp.storage.fill_(float("nan"))
    for t in cache.state.values():
        t.fill_(float("nan"))
    run = RunBinding(index=0, kv_source=0, state=cache.state.get(0))
    if kv:
        run.kv_group_index = cache.group_of_run[0]
        run.kv_group, run.kv_layer = cache.kv_layer(0)
    part.load({k: dev(v if dtype == "bfloat16" else v.float()) for k, v in w.items()}, dt)
    cache.alloc_slot()                                     # (a slot that stays empty: sequence i is not slot i)
    slots = [cache.alloc_slot() for _ in seqs]
    ws, outs = Workspace(torch.device("cuda")), [[] for _ in seqs]
    for step in cut_up([len(s) for s in seqs], cuts):
        ctx, _, _ = build_context(cache, [SeqInput(slots[i], [0] * n) for i, _, n in step], 1, dt, torch.device("cuda"), ws)
        y = dev(torch.cat([seqs[i][at:at + n] for i, at, n in step]), dt)
        out = torch.empty(y.shape[0], part.sides[0].H if hasattr(part, "sides") else part.H, device="cuda")
        assert part.produce(ctx, run, y, out) is None
        cache.commit([(slots[i], n) for i, _, n in step])
        at = 0
        for i, _, n in step:
            outs[i].append(out[at:at + n].clone())
            at += n
    cache.close()
    return [torch.cat(o) for o in outs]


def mixer_of(cfg):
    from torchless_rs_amd.config.base import config_from_dict
    from torchless_rs_amd.models import model_spec_for
    from torchless_rs_amd.parts.base import make_part
    return make_part("mixer", model_spec_for(config_from_dict(copy.deepcopy(cfg))).layers[0].mixer)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [1, 2, 63, 64, 65, 100, 129, None])
@pytest.mark.parametrize("dk, dv", [(32, 16), (48, 48), (64, 64), (128, 128)])
def test_a_key_just_inside_and_just_outside_a_chunk(dtype, chunk, dk, dv):
    """The keys at both sides of every chunk's edge (and key 3) point where every query looks, along a channel that is not
    rotated, and outweigh all others: a mask that is one position off shows at once.  In one step, in portions that start and
    end at and beside the edges, and token by token, beside the linear attention and another sequence."""
    W, L = 64, 300
    cfg = model(8, W, 1e-5, [layer(par((4, 2, dk, dv, 14.0 / dk, chunk, (100.0, dk // 2, (4.0, 1.0, 4.0, 64))), (2, 24, 40, 8.0), (1.2, 0.4)))])
    w = {k[3:]: v for k, v in plain.random_weights(cfg, dk + (chunk or 0)).items() if k.startswith("l0.mix.")}
    for n in ("q", "k"):
        w[f"mix.left.{n}.norm"] = torch.ones(dk).bfloat16()
    q_b = torch.zeros(4, dk)
    q_b[:, dk - 1] = 40.0                                  # every query looks along the last channel
    w["mix.left.q.b"] = q_b.view(-1).bfloat16()
    k_w = w["mix.left.k"].float().view(2, dk, W)
    k_w[:, :, 0] = 0.0
    k_w[:, dk - 1, 0] = 1.0                                # ... where channel 0 of the input makes a key point
    w["mix.left.k"] = k_w.view(-1, W).bfloat16()
    g = torch.Generator().manual_seed(chunk or 7)
    y = torch.randn(L, W, generator=g)
    y[:, 0] = 0.0
    edges = [3] + [e for c in range(chunk or 64, L, chunk or 64) for e in (c - 1, c)]
    y[edges, 0] = 60.0
    y = y.bfloat16()
    other = torch.randn(77, W, generator=g).bfloat16()
    w64 = {k: v.double() for k, v in w.items()}
    m = cfg["layers"][0]["mixer"]
    want = [plain.parallel(s.double(), w64, "mix.", m, torch.arange(len(s)), 1e-5) for s in (y, other)]
    if chunk and chunk > 2:                                # the loud keys decide: with the chunk one longer the result is another
        off = copy.deepcopy(m)
        off["left"]["mask"]["size"] = chunk + 1
        wrong = plain.parallel(y.double(), w64, "mix.", off, torch.arange(L), 1e-5)
        assert rms_err(wrong[edges[1:]], want[0][edges[1:]]) > 0.04
    e = chunk if chunk and chunk > 2 else 64
    tol = {"float32": 3e-5, "bfloat16": 2.5e-2}[dtype]
    for cuts in ([L], [e - 1, 1, 1, 1, e - 2, 2] + [1] * 5 + [L], [50] + [1] * 250, [2] * 150):
        got = mixer_steps(mixer_of(cfg), w, dtype, [y, other], cuts)
        for i in range(2):
            assert rms_err(got[i], want[i]) < tol, (chunk, cuts[:8], i, rms_err(got[i], want[i]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mix", [delta(4, 2, 24, 40, 3), delta(2, 2, 128, 128, 4), delta(3, 1, 11, 21, 6), delta(1, 1, 1, 1, 1), ret(2, 40, 24, [0.97, 0.5], (500.0, 24))])
def test_recurrent_mixers_in_steps_of_any_size(dtype, mix):
    W = 48
    cfg = model(8, W, 1e-5, [layer(mix)])
    w = {k[3:]: v for k, v in plain.random_weights(cfg, mix[1]["dim"], ranks=(20, 16)).items() if k.startswith("l0.mix.")}
    g = torch.Generator().manual_seed(5)
    seqs = [torch.randn(n, W, generator=g).bfloat16() for n in (1, 33, 150)]
    w64 = {k: v.double() for k, v in w.items()}
    want = [plain.MIXERS[mix[0]](s.double(), w64, "mix.", mix[1], torch.arange(len(s)), 1e-5) for s in seqs]
    few = mix[1]["dim"] == 1                               # one channel: its norm is a sign, which rounding turns near zero
    for cuts in ([150], [1, 1, 30, 2, 100, 16], [1] * 40 + [110], [2] * 75):
        got = mixer_steps(mixer_of(cfg), w, dtype, seqs, cuts)
        for i in range(3):
            err = rms_err(got[i], want[i])
            assert err < ({"float32": 1e-2, "bfloat16": 0.2} if few else {"float32": 3e-5, "bfloat16": 2e-2})[dtype], (cuts[:6], i, err)


def test_the_scales_of_two_mixers_side_by_side():
    """Each side's share by itself: a scale of 0 takes a side out, and the two add up."""
    W = 64
    g = torch.Generator().manual_seed(9)
    y = torch.randn(50, W, generator=g).bfloat16()
    got = {}
    for scales in ((1.5, 0.0), (0.0, -0.7), (1.5, -0.7)):
        cfg = model(8, W, 1e-5, [layer(par((4, 2, 32, 32, 0.2, 40, (100.0, 32)), (2, 16, 24, 8.0), scales))])
        w = {k[3:]: v for k, v in plain.random_weights(cfg, 4).items() if k.startswith("l0.mix.")}
        got[scales] = mixer_steps(mixer_of(cfg), w, "float32", [y], [50])[0]
        m = cfg["layers"][0]["mixer"]
        w64 = {k: v.double() for k, v in w.items()}
        assert rel_err(got[scales], plain.parallel(y.double(), w64, "mix.", m, torch.arange(50), 1e-5)) < 2e-5
    assert rel_err(got[1.5, 0.0] + got[0.0, -0.7], got[1.5, -0.7]) < 2e-5


# ---------------------------------------------------------------------------------------------
# whole models through the engine
# ---------------------------------------------------------------------------------------------

def plain_run(w, cfg, ids, dtype):
    """Logits and, per row, the smallest gap by which a router chose at that row or before it (a recurrence carries a choice's
    outcome on), 0 for a row whose own heads have cancelled."""
    margins, left = [], []
    lg = plain.forward(w, cfg, ids, margins=margins, left=left)
    m = torch.stack(margins).min(dim=0).values if margins else torch.ones(len(ids), dtype=F64)
    m = torch.cummin(m, dim=0).values
    if dtype == "bfloat16":
        assert (m > MARGIN[dtype]).all(), "a choice that rounding may turn"
    if left:
        m = torch.where(torch.stack(left).min(dim=0).values > LEFT[dtype], m, torch.zeros_like(m))
    return lg, m


def weights_for(cfg, seed, dtype, ranks=(16, 16)):
    """For the bfloat16 runs the routers' biases lie far apart beside small products (a choice that rounding turns changes every
    row behind it, and one of some hundred rows would always be that close): the choice is then the same for every row, with
    weights that are not.  The float32 runs choose row by row, and so do the routers' own tests."""
    w = plain.random_weights(cfg, seed=seed, ranks=ranks)
    if dtype == "bfloat16":
        g = torch.Generator().manual_seed(seed)
        for k in w:
            if k.endswith(".router"):
                w[k] = (w[k].float() * 0.06).bfloat16()
            elif k.endswith(".router.b"):
                w[k] = (1.5 * torch.randperm(w[k].numel(), generator=g)).to(w[k].dtype)
    return w


@pytest.fixture(scope="module")
def zoo(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("zifetar")
    out = {}
    for i, name in enumerate(NAMES):
        cfg = copy.deepcopy(CONFIGS[name])
        ps = some_prompts(cfg["vocab"], LENGTHS[name], seed=51 + i)
        for dtype in DTYPES:
            w = weights_for(cfg, 70 + i, dtype, RANKS[name])
            runs = [plain_run(w, cfg, p, dtype) for p in ps]
            out[name, dtype] = dict(dir=write_model(str(tmp / f"{name}_{dtype}"), cfg, w), cfg=cfg, w=w, prompts=ps,
                                    want=[r[0] for r in runs], margin=[r[1] for r in runs])
    return out


_engines = {}


def engine_for(zoo, name, dtype):
    from torchless_rs_amd.engine import Engine, load_model
    key = (name, dtype)
    if key not in _engines:
        _engines[key] = Engine(load_model(zoo[name, dtype]["dir"], dtype), max_tokens=64 * 20, max_slots=8)
    eng = _engines[key]
    assert not eng.cache.length, "a test left slots held"
    for g in eng.cache.groups:              # stale rows and states must never be read: make them NaN (a token: none there is)
        g.storage.fill_(float("nan"))
    for t in eng.cache.state.values():
        t.fill_(float("nan") if t.is_floating_point() else 10 ** 9)
    return eng


def close(got, want, dtype, what, margin=None, tol=None, rms=None):
    """Rows that rounding cannot turn (see `plain_run`) must agree; the others must be numbers."""
    loose = FEW_CHANNELS.get(what[0] if isinstance(what, tuple) else what, 1.0) if dtype == "bfloat16" else 1.0
    tol, rms = (tol or TOL[dtype]) * loose, rms if rms is False else (rms or RMS[dtype]) * loose
    got = got.detach().double().cpu()
    assert torch.isfinite(got).all(), what
    if margin is not None:
        sure = margin > MARGIN[dtype]
        assert len(sure) < 40 or sure.any(), (what, "no sure rows")
        got, want = got[sure], want[sure]
    if not len(got):
        return
    assert rel_err(got, want) < tol, (what, rel_err(got, want))
    if rms is not False:
        assert rms_err(got, want) < rms, (what, rms_err(got, want))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_most_rows_are_sure(zoo, name, dtype):
    ms = torch.cat(zoo[name, dtype]["margin"])
    assert (ms > MARGIN[dtype]).float().mean() > 0.5


def test_the_right_parts_and_caches_are_chosen(zoo):
    from torchless_rs_amd.engine.model import EMBEDDING_RUN
    from torchless_rs_amd.kernels import ops
    from torchless_rs_amd.parts.attention_heads import HeadwiseAttentionMixer
    from torchless_rs_amd.parts.block import SandwichNormBlock
    from torchless_rs_amd.parts.channel_linear import ChannelLinearMixer
    from torchless_rs_amd.parts.ffn_routed import RoutedExperts
    from torchless_rs_amd.parts.projected import ParallelMixer
    from torchless_rs_amd.parts.retention import RetentionMixer
    eng = engine_for(zoo, "cores", "bfloat16")
    blocks = eng.model.blocks
    assert all(isinstance(b, SandwichNormBlock) and b.mixer_out_norm.around_zero for b in blocks)
    assert [type(b.mixer) for b in blocks] == [ChannelLinearMixer, ParallelMixer, ChannelLinearMixer, ParallelMixer, RetentionMixer]
    assert [type(s) for s in blocks[1].mixer.sides] == [HeadwiseAttentionMixer, ChannelLinearMixer]
    assert [type(b.ffn) for b in blocks] == [RoutedExperts, RoutedExperts, type(None), RoutedExperts, RoutedExperts]
    assert sorted(eng.cache.state) == [EMBEDDING_RUN, 0, 1, 2, 3, 4] and eng.cache.state[0].dtype == torch.float32
    assert [g.ring_pages for g in eng.cache.groups] == [3, 2] and [g.runs for g in eng.cache.groups] == [[1], [3]]
    assert blocks[0].mixer.decay_step is not None and ops.channel_chunks_serve(torch.bfloat16, 128, 256)
    assert not ops.channel_chunks_serve(torch.float32, 64, 64) and not ops.channel_chunks_serve(torch.bfloat16, 129, 64)
    assert eng.model.may_capture(1) and eng.model.may_capture(64)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_each_request_alone_and_whole(zoo, name, dtype):
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, name, dtype), zoo[name, dtype]
    for p, want, m in zip(z["prompts"], z["want"], z["margin"]):
        s = eng.alloc()
        got = eng.step([SeqInput(s, p, list(range(len(p))))]).clone()
        eng.free(s)
        close(got, want, dtype, (name, len(p)), m)
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "odd", "cores"])
def test_the_stream_after_every_layer(zoo, name, dtype):
    from torchless_rs_amd.engine import Engine, SeqInput, load_model
    z = zoo[name, dtype]
    p = z["prompts"][2]
    streams = []
    plain.forward(z["w"], z["cfg"], p, streams=streams)
    model_ = load_model(z["dir"], dtype)
    eng = Engine(model_, max_tokens=256, use_graphs=False)
    seen = []
    for blk in model_.blocks:
        inner = blk.forward

        def spy(ctx, run, x, *a, _inner=inner, **kw):
            _inner(ctx, run, x, *a, **kw)
            seen.append(x.clone())
        blk.forward = spy
    s = eng.alloc()
    eng.step([SeqInput(s, p, list(range(len(p))))])
    eng.free(s)
    assert len(seen) == len(streams)
    for i, (got, want) in enumerate(zip(seen, streams)):
        assert got.dtype == torch.float32            # the residual sum is kept in 32 bits in both dtypes
        close(got, want, dtype, (name, "after layer", i), z["margin"][2], tol=2e-5 if dtype == "float32" else 4e-2, rms=False)
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prefill_against_decoding_token_by_token(zoo, name, dtype):
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, name, dtype), zoo[name, dtype]
    for i in (1, 2):
        p = z["prompts"][i]
        s = eng.alloc()
        rows = [eng.step([SeqInput(s, [t], [0])]).clone() for t in p]        # from the very first token
        eng.free(s)
        close(torch.cat(rows), z["want"][i], dtype, (name, len(p), "token by token"), z["margin"][i])
    p = z["prompts"][3]
    k = 40
    s = eng.alloc()
    rows = [eng.step([SeqInput(s, p[:-k], list(range(len(p) - k)))]).clone()]
    rows += [eng.step([SeqInput(s, [t], [0])]).clone() for t in p[-k:]]
    eng.free(s)
    close(torch.cat(rows), z["want"][3], dtype, (name, "prompt then 40 tokens"), z["margin"][3])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("portion", [2, 3, 17, 64, 100])
def test_portions_of_a_prompt(zoo, name, dtype, portion):
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, name, dtype), zoo[name, dtype]
    p, want, m = z["prompts"][3], z["want"][3], z["margin"][3]
    if portion < 4:
        p, want, m = p[:41], want[:41], m[:41]
    s = eng.alloc()
    rows = []
    for at in range(0, len(p), portion):
        part = p[at:at + portion]
        rows.append(eng.step([SeqInput(s, part, list(range(len(part))))]).clone())
    eng.free(s)
    close(torch.cat(rows), want, dtype, (name, portion), m)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_unequal_batches_against_each_alone_with_slots_pages_and_states_used_again(zoo, name, dtype):
    """All prompts in one step, then decoded together while the shorter ones end; a second batch takes the freed slots,
    pages and states (which hold the first batch's) and must give the same; the third one's step mixes a portion that goes
    on, a new prompt and a single token."""
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, name, dtype), zoo[name, dtype]
    tails = [0, 3, 9, 20]
    for turn in range(2):
        order = list(range(4)) if turn == 0 else [3, 1, 0, 2]
        slots = {i: eng.alloc() for i in order}
        heads = {i: len(z["prompts"][i]) - tails[i] for i in order}
        got = {i: [] for i in order}
        lg = eng.step([SeqInput(slots[i], z["prompts"][i][:heads[i]], list(range(heads[i]))) for i in order])
        at = 0
        for i in order:
            got[i].append(lg[at:at + heads[i]].clone())
            at += heads[i]
        live = [i for i in order if tails[i]]
        for i in order:
            if not tails[i]:
                eng.free(slots[i])
        step = 0
        while live:
            lg = eng.step([SeqInput(slots[i], [z["prompts"][i][heads[i] + step]], [0]) for i in live]).clone()
            for r, i in enumerate(live):
                got[i].append(lg[r:r + 1])
            step += 1
            for i in [i for i in live if step == tails[i]]:
                eng.free(slots[i])
            live = [i for i in live if step < tails[i]]
        for i in order:
            close(torch.cat(got[i]), z["want"][i], dtype, (name, turn, i), z["margin"][i])
        eng.cache.check()
    a, b, c = eng.alloc(), eng.alloc(), eng.alloc()
    p, q, r = z["prompts"][3], z["prompts"][2], z["prompts"][1]
    eng.step([SeqInput(a, p[:80], []), SeqInput(c, r[:-1], [])])
    lg = eng.step([SeqInput(a, p[80:], list(range(len(p) - 80))), SeqInput(b, q, list(range(len(q)))), SeqInput(c, r[-1:], [0])]).clone()
    for s in (a, b, c):
        eng.free(s)
    k = len(p) - 80
    for what, lo, hi, i, at in (("goes on", 0, k, 3, 80), ("begins", k, k + len(q), 2, 0), ("a single token", k + len(q), None, 1, len(r) - 1)):
        close(lg[lo:hi], z["want"][i][at:], dtype, (name, what, "beside others"), z["margin"][i][at:])
    assert not eng.cache.length


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_long_decoding_past_every_chunk(zoo, name, dtype):
    """A short prompt, then 300 tokens one by one (through captured graphs): chunks begin and end among decoded tokens, the
    rings of pages wrap, the recurrent states and the previous token are carried 300 times."""
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, name, dtype), zoo[name, dtype]
    ids = some_prompts(z["cfg"]["vocab"], [310], seed=78)[0]
    want, m = plain_run(z["w"], z["cfg"], ids, dtype)
    s = eng.alloc()
    rows = [eng.step([SeqInput(s, ids[:10], list(range(10)))]).clone()]
    rows += [eng.step([SeqInput(s, [t], [0])]).clone() for t in ids[10:]]
    eng.free(s)
    close(torch.cat(rows), want, dtype, name, m)


@pytest.mark.parametrize("dtype", DTYPES)
def test_logits_do_not_depend_on_batch_mates(zoo, dtype):
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, "odd", dtype), zoo["odd", dtype]
    p = z["prompts"][2]
    s = eng.alloc()
    alone = eng.step([SeqInput(s, p, list(range(len(p))))]).clone()
    eng.free(s)
    slots = [eng.alloc() for _ in range(3)]
    lg = eng.step([SeqInput(slots[0], z["prompts"][3], []), SeqInput(slots[1], p, list(range(len(p)))),
                   SeqInput(slots[2], z["prompts"][0], [0])]).clone()
    for s in slots:
        eng.free(s)
    sure = (z["margin"][2] > MARGIN[dtype]).cuda()
    assert rel_err(lg[:len(p)][sure], alone[sure]) < (2e-6 if dtype == "float32" else 2e-2)


def test_a_step_that_is_captured_and_replayed(zoo):
    """The same prompt's shape several times, then with cached rows before it: replays beside eager steps, each against the
    plain logits."""
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, "cores", "bfloat16"), zoo["cores", "bfloat16"]
    p, want, m = z["prompts"][1], z["want"][1], z["margin"][1]
    for turn in range(5):
        s = eng.alloc()
        got = eng.step([SeqInput(s, p[:40], list(range(40)))]).clone()
        close(got, want[:40], "bfloat16", ("prompt", turn), m[:40])
        got = eng.step([SeqInput(s, p[40:], list(range(len(p) - 40)))]).clone()
        close(got, want[40:], "bfloat16", ("goes on", turn), m[40:])
        eng.free(s)


def test_tokens_that_lie_on_the_device_carry_the_previous_token(zoo):
    """Single tokens taken from a tensor on the device (as the sampler leaves them): the pair's row needs the token before, which
    the host has not seen."""
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, "mixed", "float32"), zoo["mixed", "float32"]
    p, want, m = z["prompts"][2], z["want"][2], z["margin"][2]
    s = eng.alloc()
    eng.step([SeqInput(s, p[:5], [])])
    rows = []
    for t in p[5:]:
        rows.append(eng.step([SeqInput(s, [0], [0])], device_tokens=torch.tensor([99, t], dtype=torch.int32, device="cuda"), token_rows=[1]).clone())
    eng.free(s)
    close(torch.cat(rows), want[5:], "float32", "tokens on the device", m[5:])


def test_a_long_prompt_goes_by_chunks_and_many_rows_expert_by_expert(zoo, monkeypatch):
    from torchless_rs_amd.engine import SeqInput
    from torchless_rs_amd.kernels import ops
    from torchless_rs_amd.parts import ffn_routed
    monkeypatch.setattr(ffn_routed, "GROUPED_ROWS_PER_EXPERT", 1)
    calls, chunks = [], []
    inner = ffn_routed.RoutedExperts._grouped
    monkeypatch.setattr(ffn_routed.RoutedExperts, "_grouped", lambda self, *a: (calls.append(a[1].shape[0]), inner(self, *a))[1])
    by_chunks = ops.channel_chunks
    monkeypatch.setattr(ops, "channel_chunks", lambda *a, **k: (chunks.append(a[7]), by_chunks(*a, **k))[1])
    eng, z = engine_for(zoo, "cores", "bfloat16"), zoo["cores", "bfloat16"]
    p, q = z["prompts"][3], z["prompts"][2]
    s = eng.alloc()
    got = eng.step([SeqInput(s, p, list(range(len(p))))]).clone()
    eng.free(s)
    assert calls == [len(p)] * 4 and chunks == [-(-len(p) // 64)] * 4, (calls, chunks)
    close(got, z["want"][3], "bfloat16", "expert by expert", z["margin"][3])
    s = eng.alloc()
    got = eng.step([SeqInput(s, p, [len(p) - 1]), SeqInput(eng.alloc(), q, list(range(len(q))))]).clone()
    for h in eng.cache.held_slots():
        eng.free(h)
    close(got[1:], z["want"][2], "bfloat16", "expert by expert, two prompts", z["margin"][2])


def test_greedy_generation_through_the_entry_point(zoo):
    from torchless_rs_amd import SamplingConfig, generate_until_eos
    for name in ("mixed", "ones", "odd"):
        eng, z = engine_for(zoo, name, "float32"), zoo[name, "float32"]
        ps = z["prompts"][:3]
        out = generate_until_eos(eng, ps, SamplingConfig.greedy(), max_tokens=12)
        for p, r in zip(ps, out):
            assert r.tokens == plain.generate_greedy(z["w"], z["cfg"], p, 12), (name, len(p))


def test_the_command_line_and_the_trace_replay(zoo, tmp_path):
    z = zoo["mixed", "float32"]
    p = z["prompts"][2]
    r = subprocess.run([sys.executable, os.path.join(REPO, "bin", "torchless"), "--temperature", "0", "--max-tokens", "6",
                        "--dtype", "float32", z["dir"], " ".join(map(str, p))], capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    want = plain.generate_greedy(z["w"], z["cfg"], p, 6)
    assert " ".join(map(str, want)) in r.stdout, (r.stdout, want)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": p[:20], "want": [0, 19]}, {"id": "b", "tokens": p[:3], "want": [2]}], "end": ["b"]},
             {"step": 1, "entries": [{"id": "a", "tokens": [p[20]], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [p[21]], "want": [0]}], "end": ["a"]}]
    out = tmp_path / "logits"
    r = subprocess.run([sys.executable, os.path.join(REPO, "bin", "trace_run"), "--model", z["dir"], "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "23"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    V = z["cfg"]["vocab"]
    first = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(-1, V))
    last = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(-1, V))
    want = z["want"][2]
    assert rel_err(first, torch.stack([want[0], want[19], want[2]])) < TOL["float32"]
    assert rel_err(last, want[21:22]) < TOL["float32"]


# ---------------------------------------------------------------------------------------------
# configurations drawn at random
# ---------------------------------------------------------------------------------------------

def random_config(rng):
    """Any order of layers, any sizes."""
    layers = []
    for _ in range(rng.randint(3, 6)):
        kind = rng.random()
        if kind < 0.3:
            H, d = rng.choice([1, 2, 3, 5]), rng.choice([16, 24, 33, 64, 128])
            dims = rng.choice([0, d // 4 * 2, d // 2 * 2])
            mix = ret(H, d, rng.choice([20, 32, 64, 96]), [rng.choice([0.5, 0.9, 0.99, 0.9995]) for _ in range(H)],
                      (rng.choice([100.0, 1e4, 1e6]), dims) if dims else None)
        elif kind < 0.65:
            G = rng.choice([1, 2, 3])
            mix = delta(G * rng.choice([1, 2, 3]), G, rng.choice([16, 33, 64, 128]), rng.choice([20, 40, 64, 144]), rng.randint(1, 6))
        else:
            G, d = rng.choice([1, 2]), rng.choice([16, 32, 50, 64])
            dims = rng.choice([0, d // 4 * 2, d // 2 * 2])
            rot = (rng.choice([300.0, 1e4, 5e5]), dims) + rng.choice([(), ((4.0, 1.0, 4.0, 128),), ((16.0, 0.5, 3.0, 64),)]) if dims else None
            mix = par((G * rng.choice([1, 2, 4]), G, d, rng.choice([d, d, 8, 24]), rng.uniform(0.1, 0.4), rng.choice([None, 17, 40, 64, 100, 250]), rot),
                      (rng.choice([1, 2, 3]), rng.choice([16, 24, 64, 100]), rng.choice([17, 32, 80]), rng.choice([1.0, 8.0, 16.0])),
                      (rng.uniform(-1.5, 1.5), rng.uniform(0.3, 1.5)))
        f = None
        if rng.random() < 0.8:
            E = rng.choice([1, 2, 5, 8, 16])
            f = moe(E, rng.randint(1, min(4, E)), rng.choice([8, 16, 32]))
        layers.append(layer(mix, f))
    return model(rng.choice([97, 256, 500]), rng.choice([64, 96, 128, 160, 250]), rng.choice([1e-5, 1e-6]), layers,
                 scale=rng.choice([1.0, 4.0, 0.3]), pairs=rng.choice([None, (31, 5, 2), (400, 97, 13)]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(10))
def test_random_configurations(seed, dtype, tmp_path):
    """Whole prompts, a prompt with its last tokens one by one, and all of them in one batch that is decoded together."""
    from torchless_rs_amd.engine import Engine, SeqInput, load_model
    rng = random.Random(seed)
    cfg = random_config(rng)
    w = weights_for(cfg, 100 + seed, dtype, (rng.choice([4, 16, 33, 128]), rng.choice([2, 16, 40])))
    ps = some_prompts(cfg["vocab"], [1, 37, 150, 420], seed=seed)
    runs = [plain_run(w, cfg, p, dtype) for p in ps]
    loose = dict(tol=0.25, rms=5e-2)         # (rows behind a row that rounding has turned a little are a few; the mean square counts)
    if dtype == "float32":                   # some draw models that make rounding large: what 32 bits cost the plain implementation
        costs = [(rel_err(plain.forward(w, cfg, p, torch.float32)[m > MARGIN[dtype]], want[m > MARGIN[dtype]]))
                 for p, (want, m) in zip(ps, runs) if (m > MARGIN[dtype]).any()]
        loose = dict(tol=max(TOL[dtype], 4 * max(costs)), rms=max(RMS[dtype], 4 * max(costs)))
        assert loose["tol"] < 1e-3
    eng = Engine(load_model(write_model(str(tmp_path / "m"), cfg, w), dtype), max_tokens=64 * 30, max_slots=8)
    tails = [0, 5, 20, 33]
    heads = [len(p) - t for p, t in zip(ps, tails)]
    for p, h, (want, m) in zip(ps, heads, runs):
        s = eng.alloc()
        got = eng.step([SeqInput(s, p, list(range(len(p))))]).clone()
        eng.free(s)
        close(got, want, dtype, (seed, len(p), "whole"), m, **loose)
        s = eng.alloc()
        rows = [eng.step([SeqInput(s, p[:h], list(range(h)))]).clone()] + [eng.step([SeqInput(s, [t], [0])]).clone() for t in p[h:]]
        eng.free(s)
        close(torch.cat(rows), want, dtype, (seed, len(p), "then decoded"), m, **loose)
    slots = [eng.alloc() for _ in ps]
    lg = eng.step([SeqInput(s, p[:h], list(range(h))) for s, p, h in zip(slots, ps, heads)])
    got, at = [], 0
    for h in heads:
        got.append([lg[at:at + h].clone()])
        at += h
    for step in range(max(tails)):
        live = [i for i in range(len(ps)) if step < tails[i]]
        lg = eng.step([SeqInput(slots[i], [ps[i][heads[i] + step]], [0]) for i in live]).clone()
        for r, i in enumerate(live):
            got[i].append(lg[r:r + 1])
    for s in slots:
        eng.free(s)
    for i, (want, m) in enumerate(runs):
        close(torch.cat(got[i]), want, dtype, (seed, i, "together"), m, **loose)
    eng.close()
