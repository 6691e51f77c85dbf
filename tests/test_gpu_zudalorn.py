"""Zudalorn on the GPU against the plain implementation of `plain_zudalorn.py`: every new mechanism alone
(norms with one number, retention row by row and by chunks, the router with corrected choice scores, experts
behind it, xIELU, the pass that makes latents and rotated parts, products per head, attention over cached latents
and with values of another width than keys, with keys made to stand out at every window's edge, the whole
latent mixer over pages that are rings), then whole models of the tests' own sizes through the engine: whole
prompts, the stream after every layer, decoding token by token, portions down to two tokens, unequal batches,
slots, pages and states used again, long decoding, and greedy generation through the entry point."""
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

import plain_zudalorn as plain
from test_gpu_sozetar import some_prompts, write_model
from test_zudalorn_config import MIXED, dense, latent, layer, model, moe, ret
from util import rel_err, rms_err

pytestmark = pytest.mark.gpu
REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
TOL = {"float32": 3e-5, "bfloat16": 6e-2}
RMS = {"float32": 1e-5, "bfloat16": 2.5e-2}
# a model whose sublayers have a handful of channels divides them by root mean squares that may be near zero
FEW_CHANNELS = {"ones": 3.0}
# a router's choice made by less than this (the gap of two choice scores, or of two groups') may fall the other way
# under rounding (in bfloat16 every choice of these models is wider)
MARGIN = {"float32": 1e-5, "bfloat16": 1e-2}
F64 = torch.float64

# sizes that the matrix cores take: latents of 128, 256 and 512, 16 and more heads, values as wide as keys or not,
# retention heads of 64 to 256
CORES = model(256, 128, 1e-6, [
    layer(latent(16, 32, 32, 64, 128, 0.125, window=100, scaling=(4.0, 128.0, 16.0, 1.0)), moe(16, 2, 32, groups=(4, 2), shared=64)),
    layer(ret(2, 128, 128, [0.99, 0.875], rot=(10000.0, 128)), dense(256)),
    layer(latent(4, 64, 32, 64, 256, 0.1, window=129), moe(8, 4, 32, groups=(2, 1))),
    layer(ret(1, 256, 64, [0.998], rot=(1000.0, 64)), None),
    layer(latent(18, 128, 64, 128, 512, 0.07, base=500.0), dense(128)),
])
# what a model may happen to make 1 or leave out: one head, one expert, one group, groups of one expert, top = experts, a
# window of one (a position sees itself alone) and of two, no rotation, a latent of two channels, a decay of 0 and of 1.  (A
# sublayer of a single channel would be a sign behind its norm, which rounding turns: the kernels' own tests have that.)
ONES = model(96, 32, 1e-4, [
    layer(latent(1, 8, 2, 8, 2, 0.25, window=1), moe(1, 1, 16, groups=(1, 1), shared=8)),
    layer(ret(1, 4, 8, [0.5]), moe(4, 4, 8)),
    layer(latent(2, 1, 2, 4, 16, 0.35, window=2, scaling=(1.0, 10.0, 4.0, 0.5)), dense(8)),
    layer(ret(2, 8, 8, [0.0, 1.0], rot=(50.0, 2)), moe(5, 2, 8, groups=(5, 3))),
    layer(latent(1, 8, 8, 8, 8, 0.35), None),
])
# sizes that no kernel's fast way takes: an odd width and vocabulary, heads of 11 and 21, latents of 37, states of 13 x 7
ODD = model(131, 101, 1e-5, [
    layer(ret(3, 13, 7, [0.9, 0.8, 0.99], rot=(300.0, 6)), moe(6, 2, 11, groups=(3, 2), shared=10)),
    layer(latent(3, 11, 6, 21, 37, 0.29, window=33, scaling=(3.0, 40.0, 5.0, 1.5)), dense(77)),
    layer(ret(1, 20, 30, [0.97], rot=(20.0, 20)), None),
    layer(latent(5, 5, 10, 3, 9, 0.3, window=65), moe(9, 3, 10, groups=(3, 1))),
])
CONFIGS = {"mixed": MIXED, "cores": CORES, "ones": ONES, "odd": ODD}
LENGTHS = {"mixed": [1, 7, 23, 150], "cores": [5, 64, 129, 330], "ones": [2, 65, 130, 200], "odd": [4, 33, 67, 140]}
NAMES = list(CONFIGS)


def dev(t, dtype=None):
    return t.to("cuda", dtype) if dtype is not None else t.to("cuda")


def step_ctx(dtype, **kw):
    from torchless_rs_amd.parts.base import Workspace
    return types.SimpleNamespace(pending=None, prenormed=None, norm_ahead=None, row_factor=None, dtype=TORCH[dtype],
                                 workspace=Workspace(torch.device("cuda")), host={}, **kw)


def rotation_of(rot, interleaved):
    from torchless_rs_amd.kernels import ops
    if not rot or not rot["dims"]:
        return ops.NO_ROTATION
    f, mag = plain.frequencies(rot)
    return ops.Rotation(dev(f.float()), rot["dims"], interleaved, mag)


# ---------------------------------------------------------------------------------------------
# norms with one number
# ---------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [30, 101, 320, 2052, 8200])
def test_norms_with_one_number_for_all_channels(dtype, H):
    from torchless_rs_amd.parts.norms import RMSNorm
    g = torch.Generator().manual_seed(H)
    n = 5
    z, x = torch.randn(n, H, generator=g) * 3, torch.randn(n, H, generator=g)
    norms = []
    for i, num in enumerate((0.7, -1.3)):
        rn = RMSNorm(H, 1e-5 * (i + 1), name="", scalar=True)
        assert rn.weight_specs()[""].shape == ()
        rn.load({"": dev(torch.tensor(num))}, TORCH[dtype])
        norms.append((rn, num))
    (a, ga), (b, gb) = norms
    ctx = step_ctx(dtype)
    out = torch.empty(n, H, dtype=TORCH[dtype], device="cuda")
    a.forward(ctx, dev(z), out)
    tol = 1e-5 if dtype == "float32" else 1e-2
    want = plain.scalar_norm(z.double(), a.eps, ga)
    assert rel_err(out, want) < tol
    want_x = x.double() + want
    for then in (None, (b, out)):
        xs = dev(x.clone())
        ctx.prenormed = None
        a.add_to(ctx, dev(z.clone()), xs, then=then)
        assert rel_err(xs, want_x) < 1e-5
        if ctx.prenormed is not None:
            assert rel_err(out, plain.scalar_norm(want_x, b.eps, gb)) < tol


# ---------------------------------------------------------------------------------------------
# retention
# ---------------------------------------------------------------------------------------------

def retention_inputs(H, dk, dv, L, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(L, 2 * H * (dk + dv), generator=g).to(torch.bfloat16).double()      # (exact in both dtypes)


def plain_retention_rows(proj, H, dk, dv, rot, kscale, decay, eps, pos0=0):
    """The normed, gated heads [L, H*dv] and the last state of one sequence from zero."""
    L = proj.shape[0]
    pos = torch.arange(pos0, pos0 + L)
    q = plain.rotate(proj[:, :H * dk].reshape(L, H, dk), pos, rot, False)
    k = plain.rotate(proj[:, H * dk:2 * H * dk].reshape(L, H, dk), pos, rot, False) * kscale
    v = proj[:, 2 * H * dk:2 * H * dk + H * dv].reshape(L, H, dv)
    o, S = plain.retention_heads(q, k, v, decay)
    gate = proj[:, 2 * H * dk + H * dv:]
    return plain.rms(o, eps).reshape(L, H * dv) * gate * torch.sigmoid(gate), S


def retention_steps(way, dtype, H, dk, dv, rot, kscale, decay, eps, seqs, cuts, slots, n_slots=7):
    """Several sequences' rows (a list of [L, width]) in steps that bring `cuts[i]` rows of each that still has some, by
    `way` "scan" or "chunks"; the rows' results per sequence, and the states."""
    from torchless_rs_amd.kernels import ops
    from torchless_rs_amd.parts.base import Workspace
    from torchless_rs_amd.parts.retention import NO_DECAY_LEFT
    ws = Workspace(torch.device("cuda"))
    size = H * dk * dv
    state = torch.full((n_slots, -(-size // 4) * 4 + 4), float("nan"), device="cuda")[:, :size]      # strided rows
    for s in slots:
        state[s].zero_()
    d32 = dev(torch.tensor(decay))
    lg = dev(torch.tensor([math.log2(a) if a > 0 else NO_DECAY_LEFT for a in decay]))
    rotation = rotation_of(rot, False)
    done, outs, C = [0] * len(seqs), [[] for _ in seqs], ops.retention_chunk()
    for cut in cuts:
        live = [i for i in range(len(seqs)) if done[i] < len(seqs[i])]
        if not live:
            break
        take = [min(cut, len(seqs[i]) - done[i]) for i in live]
        proj = dev(torch.cat([seqs[i][done[i]:done[i] + m] for i, m in zip(live, take)]).float().contiguous())
        pos = dev(torch.cat([torch.arange(done[i], done[i] + m) for i, m in zip(live, take)]).to(torch.int32))
        cu = torch.tensor(np.concatenate([[0], np.cumsum(take)]), dtype=torch.int32, device="cuda")
        sl = torch.tensor([slots[i] for i in live], dtype=torch.int32, device="cuda")
        h = torch.empty(proj.shape[0], H * dv, dtype=TORCH[dtype], device="cuda")
        if way == "chunks":
            ops.retention_chunks(proj, pos, rotation, H, dk, dv, kscale, lg, eps, state, cu, sl, sum(-(-m // C) for m in take), ws, h)
        else:
            o = torch.empty(proj.shape[0], H * dv, device="cuda")
            ops.retention_scan(proj, pos, rotation, H, dk, dv, kscale, d32, state, cu, sl, o)
            ops.retention_norm_gate(o, proj[:, 2 * H * dk + H * dv:], H, eps, h)
        at = 0
        for i, m in zip(live, take):
            outs[i].append(h[at:at + m].clone())
            at += m
            done[i] += m
    return [torch.cat(o) for o in outs], state


SCAN_SHAPES = [(1, 1, 1, 0), (3, 13, 7, 6), (2, 33, 20, 0), (2, 64, 64, 64), (3, 32, 48, 16), (1, 200, 40, 200), (2, 512, 12, 32)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, dk, dv, dims", SCAN_SHAPES)
def test_retention_row_by_row_in_steps_of_any_size(dtype, H, dk, dv, dims):
    decay = [0.96875, 0.5, 0.999][:H]
    rot = {"base": 100.0, "dims": dims}
    seqs = [retention_inputs(H, dk, dv, L, seed=L) for L in (1, 40, 75)]
    slots = [5, 0, 3]
    want = [plain_retention_rows(s, H, dk, dv, rot, dk ** -0.5, decay, 1e-5) for s in seqs]
    tol = 1e-5 if dtype == "float32" else 6e-3
    for cuts in ([75], [1] * 5 + [33] + [2] * 30, [8, 9, 7, 64]):
        got, state = retention_steps("scan", dtype, H, dk, dv, rot, dk ** -0.5, decay, 1e-5, seqs, cuts, slots)
        for i in range(3):
            assert rel_err(got[i], want[i][0]) < tol, (cuts, i)
            assert rel_err(state[slots[i]].view(H, dk, dv), want[i][1]) < 1e-5, (cuts, i, "state")
        assert torch.isnan(state[[1, 2, 4, 6]]).all()           # nobody else's block was touched


@pytest.mark.parametrize("H, dk, dv", [(1, 8, 4), (3, 32, 48), (2, 64, 64), (2, 40, 100), (2, 128, 128), (1, 128, 256), (1, 256, 256), (2, 72, 20)])
def test_retention_by_chunks_in_steps_of_any_size(H, dk, dv):
    """Inputs that bfloat16 holds and a factor that is a power of two: what is left is the rounding inside, which the two
    terms of every decayed operand keep far below that of a single one (the state carries 16 bits at least)."""
    decay = [0.96875, 0.5, 0.9995][:H]
    lens = (1, 63, 257, 530)
    seqs = [retention_inputs(H, dk, dv, L, seed=3 * L) for L in lens]
    slots = [5, 0, 3, 6]
    want = [plain_retention_rows(s, H, dk, dv, None, 0.125, decay, 1e-5) for s in seqs]
    for cuts in ([530], [64, 192, 1, 256, 100], [2, 31, 300, 255], [256, 256, 256]):
        got, state = retention_steps("chunks", "bfloat16", H, dk, dv, None, 0.125, decay, 1e-5, seqs, cuts, slots)
        for i in range(len(lens)):
            assert rel_err(got[i], want[i][0]) < 8e-3, (cuts, i)
            assert rel_err(state[slots[i]].view(H, dk, dv), want[i][1]) < 2e-4, (cuts, i, "state")
        assert torch.isnan(state[[1, 2, 4]]).all()


@pytest.mark.parametrize("dims, base", [(64, 10000.0), (16, 50.0), (62, 1e6)])
def test_retention_by_chunks_with_a_rotation_and_mixed_with_single_rows(dims, base):
    H, dk, dv, decay, rot = 2, 64, 96, [0.99, 0.875], {"base": base, "dims": dims}
    seqs = [retention_inputs(H, dk, dv, L, seed=L) for L in (90, 400)]
    want = [plain_retention_rows(s, H, dk, dv, rot, 0.125, decay, 1e-5) for s in seqs]
    got, state = retention_steps("chunks", "bfloat16", H, dk, dv, rot, 0.125, decay, 1e-5, seqs, [1, 1, 80, 300, 18], [1, 4])
    for i in range(2):
        assert rel_err(got[i], want[i][0]) < 1.5e-2
        assert rel_err(state[[1, 4][i]].view(H, dk, dv), want[i][1]) < 6e-3


@pytest.mark.parametrize("way", ["scan", "chunks"])
def test_a_row_that_is_carried_far_and_one_that_is_forgotten_at_once(way):
    """Head 0 never forgets, head 1 keeps the present row alone, head 2 nearly never forgets: the loud first row still shows
    after 600 rows in heads 0 and 2, and nowhere in head 1, in steps of any size."""
    H, dk, dv, L = 3, 16, 16, 600
    decay = [1.0, 0.0, 0.9990234375]
    p = retention_inputs(H, dk, dv, L, seed=2) * 2.0 ** -6
    p[:, :H * dk:dk] = 1.0                               # channel 0 of q: every row looks for what row 0 left there
    p[:, H * dk:2 * H * dk:dk] = 0.0
    p[0, H * dk:2 * H * dk:dk] = 32.0                    # ... and row 0 alone writes it
    p[0, 2 * H * dk:2 * H * dk + H * dv] = 1.0
    p[:, 2 * H * dk + H * dv:] = 4.0
    want, S = plain_retention_rows(p, H, dk, dv, None, 1.0, decay, 1e-6)
    first = plain_retention_rows(torch.cat([p[:1] * 0, p[1:]]), H, dk, dv, None, 1.0, decay, 1e-6)[0]
    assert rel_err(first[-1, :dv], want[-1, :dv]) > 0.5 and rel_err(first[-1, 2 * dv:], want[-1, 2 * dv:]) > 0.5
    assert rel_err(first[-1, dv:2 * dv], want[-1, dv:2 * dv]) < 1e-12
    for cuts in ([600], [1] * 40 + [200, 360], [300, 300], [255, 2, 343]):
        got, state = retention_steps(way, "bfloat16", H, dk, dv, None, 1.0, decay, 1e-6, [p], cuts, [2])
        assert rel_err(got[0], want) < 8e-3, cuts
        assert rel_err(state[2].view(H, dk, dv), S) < 2e-4


# ---------------------------------------------------------------------------------------------
# feed-forwards
# ---------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, I", [(64, 96), (101, 77), (128, 256), (32, 1)])
def test_xielu_feed_forward(dtype, H, I):
    from torchless_rs_amd.parts.ffn_routed import PlainFeedForward
    cfg = model(8, H, 1e-5, [layer(ret(1, 1, 1, [0.5]), dense(I))])
    g = torch.Generator().manual_seed(I)
    for seed, pq in ((1, (0.3, -1.5)), (2, (-4.0, 3.0))):
        w = {k[3:]: v for k, v in plain.random_weights(cfg, seed, gain=3.0).items() if k.startswith("l0.mlp.")}
        w["mlp.act"] = torch.tensor(pq).to(torch.bfloat16)
        part = PlainFeedForward(H, I, activation="xielu")
        assert {k: tuple(v.shape) for k, v in part.weight_specs().items()} == {k: tuple(v.shape) for k, v in w.items()}
        part.load({k: dev(v if dtype == "bfloat16" else v.float()) for k, v in w.items()}, TORCH[dtype])
        for n in (1, 9, 40, 300):
            y = torch.randn(n, H, generator=g).to(TORCH[dtype])
            want = plain.dense_ff(y.double(), {k: v.double() for k, v in w.items()}, "mlp.")
            out = torch.empty(n, H, device="cuda")
            part.produce(step_ctx(dtype), dev(y), out)
            assert rel_err(out, want) < (2e-5 if dtype == "float32" else 2e-2), (n, pq)


@pytest.mark.parametrize("total", [8, 1000, 2 ** 20 + 8])
def test_activations_element_by_element(total):
    from torchless_rs_amd.kernels import ops
    g = torch.Generator().manual_seed(total)
    z = torch.randn(total, generator=g) * 3
    z[:4] = torch.tensor([0.0, -1e-4, 1e-4, -80.0])
    a, b = 1.3, 0.6
    x = z.double()
    want = {"xielu": torch.where(x > 0, a * x * x + x / 2, b * (torch.expm1(x.clamp(max=0)) - x) + x / 2), "relu": x.clamp(min=0),
            "relu2": x.clamp(min=0) ** 2}
    for name, w in want.items():
        c = {"a": a, "b": b} if name == "xielu" else None
        for ud, od, tol in ((torch.float32, torch.float32, 1e-6), (torch.float32, torch.bfloat16, 5e-3), (torch.bfloat16, torch.bfloat16, 2e-2)):
            out = torch.empty(total, dtype=od, device="cuda")
            ops.unary_act(dev(z, ud), name, out, c)
            assert rel_err(out, w) < tol, (name, ud, od)


ROUTERS = [(8, 2, 4, 2), (8, 2, None, None), (12, 3, 4, 1), (6, 6, 2, 2), (5, 2, 5, 3), (1, 1, 1, 1), (40, 7, 8, 3), (64, 4, 2, 1)]


@pytest.mark.parametrize("in_dtype", DTYPES)
@pytest.mark.parametrize("n", [3, 90])
@pytest.mark.parametrize("E, top, groups, keep", ROUTERS)
def test_the_router_with_corrected_choice_scores(in_dtype, n, E, top, groups, keep):
    """Corrections of both signs, large enough that choice scores are negative (a group that is not kept must not win with
    zeros); groups by their two largest (or their only) choice scores; weights without the correction, summing to one; the
    shared expert's own weight from one more row."""
    from torchless_rs_amd.kernels import ops
    g = torch.Generator().manual_seed(E * 10 + top)
    W = 48
    h = torch.randn(n, W, generator=g).to(TORCH[in_dtype])
    w = {"router": (torch.randn(E, W, generator=g) * 0.4).double(), "correction": (torch.randn(E, generator=g) - 1.5).double()}
    sg = torch.randn(1, W, generator=g) * 0.3
    weights, chosen = torch.empty(n, E, device="cuda"), torch.empty(n, top, dtype=torch.int32, device="cuda")
    shared = torch.empty(n, device="cuda")
    ops.route(dev(h), dev(torch.cat([w["router"].float(), sg])), groups or 0, keep or 0, top, weights, chosen, logistic=True,
              correction=dev(w["correction"].float()), two_largest=True, normalise_eps=1e-20, shared_weight=shared)
    r = {"experts": E, "top": top}
    if groups:
        r["groups"] = {"count": groups, "keep": keep}
    margins = []
    want = plain.route(h.double(), w, "", r, margins)
    sure = margins[0] > 1e-5
    assert sure.float().mean() > 0.9
    assert rel_err(weights[sure.cuda()], want[sure]) < 1e-5
    assert torch.allclose(weights.sum(dim=1), torch.ones(n, device="cuda"), atol=1e-5)
    picked = torch.gather(weights, 1, chosen.long())
    assert (picked > 0).all() and ((weights != 0).sum(dim=1) == top).all()
    assert rel_err(shared, torch.sigmoid(h.double() @ sg.double().T)[:, 0]) < 1e-5
    c = torch.gather(torch.sigmoid(h.double() @ w["router"].T) + w["correction"], 1, chosen.long().cpu())
    assert (c[:, :-1] >= c[:, 1:] - 1e-5).all()               # the best first, by the corrected scores


def test_a_correction_turns_choices_but_not_weights_and_a_group_wins_by_two():
    """Expert 0 scores highest and is alone in being corrected away; group 1 has the single largest choice score of the
    rest, group 0 the larger sum of two."""
    from torchless_rs_amd.kernels import ops
    h = torch.eye(1, 4)
    logits = torch.tensor([4.0, 1.0, 0.9, -3.0, 2.0, -3.0, -3.0, -3.0])
    router = torch.zeros(8, 4)
    router[:, 0] = logits
    corr = torch.tensor([-2.0, 0, 0, 0, 0, 0, 0, 0])
    out = torch.empty(1, 8, device="cuda")
    args = (dev(h), dev(router), 2, 1, 2, out, None)
    ops.route(*args, logistic=True, correction=dev(corr), two_largest=True, normalise_eps=0.0)
    s = torch.sigmoid(logits.double())
    assert rel_err(out[0], torch.tensor([0, s[1], s[2], 0, 0, 0, 0, 0]) / (s[1] + s[2])) < 1e-6
    ops.route(*args, logistic=True, correction=dev(corr), two_largest=False)
    assert out[0, 4] > 0 and out[0, 1] == 0 and abs(float(out[0, 4]) - float(s[4])) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, E, top, ff, groups, shared", [(64, 8, 2, 32, (4, 2), 48), (101, 6, 2, 11, (3, 2), 10), (32, 1, 1, 16, (1, 1), None),
                                                           (48, 10, 1, 8, None, 8), (40, 4, 4, 8, None, None)])
def test_experts_behind_corrected_scores_with_a_gated_shared_one(dtype, H, E, top, ff, groups, shared):
    """The chosen experts alone (few rows), all side by side (more rows) and, in bfloat16, over each expert's own rows."""
    from torchless_rs_amd.parts.ffn_routed import RoutedExperts
    mlp = moe(E, top, ff, groups=groups, shared=shared)
    cfg = model(8, H, 1e-5, [layer(ret(1, 1, 1, [0.5]), mlp)])
    w = {k[3:]: v for k, v in plain.random_weights(cfg, H + E, gain=2.0).items() if k.startswith("l0.mlp.")}
    part = RoutedExperts(H, E, top, ff, group_count=groups[0] if groups else None, group_keep=groups[1] if groups else None,
                         group_score="two_largest", shared_size=shared, score="sigmoid", correction=True, normalise_eps=1e-20,
                         gated=True, activation="silu", shared_gated=True)
    assert set(part.weight_specs()) == set(w)
    part.load({k: dev(v if dtype == "bfloat16" else v.float()) for k, v in w.items()}, TORCH[dtype])
    w = {k: v.double() for k, v in w.items()}
    g = torch.Generator().manual_seed(E)
    tol = 2e-5 if dtype == "float32" else 2.5e-2
    ways = set()
    for n in (1, 3, 40, 200):
        y = torch.randn(n, H, generator=g).to(TORCH[dtype])
        margins = []
        want = plain.routed_ff(y.double(), w, "mlp.", mlp, margins)
        sure = margins[0] > 1e-5
        out = torch.empty(n, H, device="cuda")
        ctx = step_ctx(dtype)
        ways.add("rows" if part.few_rows(dev(y)) else "wide")
        part.produce(ctx, dev(y), out)
        assert rel_err(out[sure.cuda()], want[sure]) < tol, (n, "stored")
        x0 = torch.randn(n, H, generator=g)
        x = dev(x0.clone())
        part.forward(ctx, dev(y), x)
        if ctx.pending is not None:
            x += ctx.pending.sum(dim=0)
        assert rel_err(x[sure.cuda()], (x0.double() + want)[sure]) < tol, (n, "added")
        if dtype == "bfloat16" and n == 200 and H % 8 == 0:
            part._grouped(ctx, dev(y), out, False)
            assert rel_err(out[sure.cuda()], want[sure]) < tol, (n, "expert by expert")
    assert ways == {"rows", "wide"}


# ---------------------------------------------------------------------------------------------
# attention over latents
# ---------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, dn, dr, R, scaling", [(3, 11, 6, 37, (3.0, 40.0, 5.0, 1.5)), (9, 32, 16, 128, None), (1, 8, 0, 2, None), (17, 128, 64, 512, (4.0, 4096.0, 32.0, 1.0))])
def test_the_pass_that_makes_latents_and_rotated_parts(dtype, H, dn, dr, R, scaling):
    """Into rows, and straight into pages whose other rows stay as they are."""
    from torchless_rs_amd.kernels import ops
    g = torch.Generator().manual_seed(R)
    pos = torch.tensor([0, 1, 63, 64, 65, 700, 129], dtype=torch.int32)
    n, eps, first = len(pos), 1e-3, H * (dn + dr)
    rot = {"base": 77.0, "dims": dr}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    proj, w = torch.randn(n, first + R + dr, generator=g) * 2, torch.randn(R, generator=g)
    p64 = proj.double()
    q = p64[:, :first].view(n, H, dn + dr)
    want_qr = plain.rotate(q[..., dn:], pos, rot, True) if dr else None
    want_c = plain.rms(p64[:, first:first + R], eps) * w.double()
    want_row = torch.cat([want_c, plain.rotate(p64[:, None, first + R:], pos, rot, True)[:, 0]], dim=1) if dr else want_c
    dt, tol = TORCH[dtype], 1e-4 if dtype == "float32" else 8e-3
    pd = dev(proj)
    ql = torch.full((n, H, R + dr), 7.0, dtype=dt, device="cuda")
    qn, c = torch.empty(n, H, dn, dtype=dt, device="cuda"), torch.empty(n, R, dtype=dt, device="cuda")
    rows = torch.empty(n, R + dr, dtype=dt, device="cuda")
    args = (pd[:, :first], pd[:, first:], dev(pos), rotation_of(rot, True), H, dn, dr, dev(w), eps)
    ops.latent_prepare(*args, qn, ql[:, :, R:], c, rows)
    assert rel_err(qn, q[..., :dn]) < tol and rel_err(c, want_c) < tol and rel_err(rows, want_row) < tol
    assert (ql[:, :, :R] == 7.0).all() and (not dr or rel_err(ql[:, :, R:], want_qr) < tol)
    ring = 3
    table = dev(torch.randperm(n * ring, generator=g).to(torch.int32).view(n, ring))
    pages = torch.full((n * ring, 64, R + dr), float("nan"), dtype=dt, device="cuda")
    ops.latent_prepare(*args, qn, ql[:, :, R:], None, None, table=table, ring_pages=ring, pages=pages)
    for i in range(n):
        page = int(table[i, (int(pos[i]) // 64) % ring])
        assert torch.equal(pages[page, int(pos[i]) % 64], rows[i])
        pages[page, int(pos[i]) % 64] = float("nan")
    assert torch.isnan(pages).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n, H, N, K", [(1, 3, 37, 11), (5, 16, 128, 32), (40, 2, 64, 256), (17, 18, 512, 128), (8, 4, 20, 512), (3, 1, 1, 8)])
def test_products_per_head(dtype, n, H, N, K):
    from torchless_rs_amd.kernels import ops
    g = torch.Generator().manual_seed(N)
    x, w = torch.randn(n, H, K, generator=g).to(TORCH[dtype]), torch.randn(H, N, K, generator=g).to(TORCH[dtype])
    wide = torch.full((n, H, N + 5), 3.0, dtype=TORCH[dtype], device="cuda")
    ops.head_products(dev(x), dev(w), wide[:, :, :N])
    want = torch.einsum("nhk,hjk->nhj", x.double(), w.double())
    assert rel_err(wide[:, :, :N], want) < (1e-5 if dtype == "float32" else 6e-3) and (wide[:, :, N:] == 3.0).all()


def loud_rows(L, D, H, edges, seed):
    """Rows [L, D] and queries [H, D]: every row's score is about 0 but for the rows `edges`, which every query scores at
    +16 over D's scale; c (the values) differs everywhere."""
    g = torch.Generator().manual_seed(seed)
    rows, q = torch.randn(L, D, generator=g) * 0.3, torch.randn(H, D, generator=g) * 0.1
    rows[:, D - 1] = 0.0
    q[:, D - 1] = 4.0
    for e in edges:
        if 0 <= e < L:
            rows[e, D - 1] = 4.0
    return rows, q


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, R, dr", [(1, 2, 2), (3, 37, 6), (16, 64, 16), (5, 96, 8), (17, 128, 64), (20, 256, 32), (4, 240, 16), (33, 512, 64), (2, 504, 8), (2, 520, 8)])
@pytest.mark.parametrize("window", [None, 1, 2, 63, 64, 65, 130])
def test_single_tokens_over_cached_latents(dtype, H, R, dr, window):
    """Three sequences of unequal lengths; the loud rows are the last inside the window and the first outside (and row 0
    without one): a row that is one off shows at once.  Pages of nobody and rows behind the query's own hold NaN."""
    from torchless_rs_amd.kernels import ops
    D, dt = R + dr, TORCH[dtype]
    lens = [1, 64, 300]
    ring = -(-window // 64) if window else 1 << 24
    n_seq = [min(-(-L // 64), ring) for L in lens]
    width = max(n_seq)
    g = torch.Generator().manual_seed(R)
    order = torch.randperm(sum(n_seq) + 2, generator=g).tolist()
    pages = torch.full((len(order), 64, D), float("nan"), dtype=dt, device="cuda")
    table = torch.zeros(3, width, dtype=torch.int32)
    q, want = torch.empty(3, H, D), []
    for b, L in enumerate(lens):
        mine = [order.pop() for _ in range(n_seq[b])]
        table[b, :n_seq[b]] = torch.tensor(mine, dtype=torch.int32)
        p = L - 1
        edges = [p - window + 1, p - window] if window else [0]
        rows, q[b] = loud_rows(L, D, H, edges, seed=b + L)
        rows = rows.to(dt)
        for j in range(max(0, L - ring * 64), L):
            pages[mine[(j // 64) % ring], j % 64] = dev(rows[j])
        lo = max(0, p - window + 1) if window else 0
        a = torch.softmax(q[b].to(dt).double() @ rows[lo:].double().T, dim=-1)
        want.append(a @ rows[lo:, :R].double())
    pos = torch.tensor([L - 1 for L in lens], dtype=torch.int32, device="cuda")
    ctx = step_ctx(dtype, row_pos=pos)
    out = torch.empty(3, H, R, dtype=dt, device="cuda")
    ops.latent_attention(dev(q, dt), pages, dev(table), ring, ctx, dr, window, 1.0, out)
    assert rel_err(out, torch.stack(want)) < (2e-5 if dtype == "float32" else 1.2e-2)


@pytest.mark.parametrize("splits", [1, 2, 3, 9, 40])
@pytest.mark.parametrize("blocks, H, R, dr", [(1, 6, 128, 16), (1, 16, 510, 66), (1, 33, 504, 8), (2, 6, 512, 64), (2, 48, 510, 66)])
def test_splits_of_the_cached_latents(splits, blocks, H, R, dr, monkeypatch):
    """A loud row in the first page, one in the last, and long runs without; more splits than pages leave some empty.
    One and two blocks of 16 heads a workgroup."""
    from torchless_rs_amd.kernels import ops
    monkeypatch.setattr(ops, "latent_splits", lambda *a: (blocks, splits))
    L = 1000
    D, n = R + dr, 16
    rows, q = loud_rows(L, D, H, [3, L - 2], seed=1)
    rows, q = rows.bfloat16(), q.bfloat16()
    pages = torch.full((n, 64, D), float("nan"), dtype=torch.bfloat16)
    for j in range(L):
        pages[n - 1 - j // 64, j % 64] = rows[j]
    table = torch.arange(n - 1, -1, -1, dtype=torch.int32).view(1, n)
    for window in (None, 200):
        lo = L - window if window else 0
        want = torch.softmax(q.double() @ rows[lo:].double().T, dim=-1) @ rows[lo:, :R].double()
        out = torch.empty(1, H, R, dtype=torch.bfloat16, device="cuda")
        ctx = step_ctx("bfloat16", row_pos=torch.tensor([L - 1], dtype=torch.int32, device="cuda"))
        ops.latent_attention(dev(q[None].contiguous()), dev(pages), dev(table), 1 << 24, ctx, dr, window, 1.0, out)
        assert rel_err(out[0], want) < 1e-2


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dk, dv", [(10, 7), (16, 8), (48, 72), (40, 100), (64, 64), (96, 64), (136, 128), (192, 128), (160, 192), (256, 200)])
@pytest.mark.parametrize("window", [None, 1, 63, 64, 65, 200])
def test_keys_and_values_of_unequal_width_from_pages_and_from_the_step(dtype, dk, dv, window):
    """Unequal sequences, part of each in pages that live for the step; the loud keys are those just inside and just outside
    the last rows' windows, position 0, and both sides of the border between pages and new rows."""
    from torchless_rs_amd.kernels import ops
    H, dt = 3, TORCH[dtype]
    before, new = [0, 70, 128, 129], [150, 2, 130, 75]
    g = torch.Generator().manual_seed(dk)
    offs, cols = ops.aligned_columns(before, new)
    i32 = dict(dtype=torch.int32, device="cuda")
    ring = -(-window // 64) if window else 1 << 24
    held = [min(-(-c // 64), ring) for c in before]
    off = np.concatenate([[0], np.cumsum(held)])
    pages = torch.full((max(1, off[-1]), H * 64 * (dk + dv)), float("nan"), dtype=dt)
    table = torch.zeros(4, max(1, max(held)), dtype=torch.int32)
    qs, ks, vs, want = [], [], [], []
    for b, (c, m) in enumerate(zip(before, new)):
        L = c + m
        k, v, q = (torch.randn(L, H, d, generator=g) for d in (dk, dv, dk))
        k, q = k * 0.2, q * 0.05
        k[..., 0] = 0.0
        q[..., 0] = 4.0
        for e in [0, c - 1, c] + ([L - 1 - window, L - window, c - window] if window else []):
            if 0 <= e < L:
                k[e, :, 0] = 4.0
        k, v, q = k.to(dt), v.to(dt), q.to(dt)
        table[b, :held[b]] = torch.arange(off[b], off[b + 1], dtype=torch.int32)
        for j in range(max(0, c - ring * 64), c):
            page = pages[off[b] + (j // 64) % ring]
            page[:H * 64 * dk].view(H, 64, dk)[:, j % 64] = k[j]
            page[H * 64 * dk:].view(H, dv, 64)[:, :, j % 64] = v[j]
        s = torch.einsum("ihd,jhd->hij", q.double(), k.double())
        s = s.masked_fill(~plain.window_mask(torch.arange(L), window)[None], -math.inf)[:, c:]
        want.append(torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v.double()))
        qs.append(q[c:]), ks.append(k[c:]), vs.append(v[c:])
    cu = np.concatenate([[0], np.cumsum(new)])
    ctx = step_ctx(dtype, row_pos=torch.cat([torch.arange(c, c + m) for c, m in zip(before, new)]).to(**i32),
                   row_seq=torch.repeat_interleave(torch.arange(4), torch.tensor(new)).to(**i32),
                   cu_seqlens=torch.tensor(cu, **i32), len_before=torch.tensor(before, **i32), tile_off=torch.tensor(offs, **i32),
                   len_after=torch.tensor([c + m for c, m in zip(before, new)], **i32))
    ctx.host.update(n_new=np.asarray(new), len_before=np.asarray(before), aligned_cols=cols)
    out = torch.empty(sum(new), H, dv, dtype=dt, device="cuda")
    ops.attend_heads(ctx, dev(torch.cat(qs)), dev(torch.cat(ks)), dev(torch.cat(vs)), dev(pages), dev(table), ring, window, 1.0, out)
    assert rel_err(out, torch.cat(want)) < (2e-5 if dtype == "float32" else 1.2e-2)


class LatentSequences:
    """The cache of one latent mixer for several sequences, driven as the engine drives it: steps of any size, pages of 64
    in rings when there is a window, NaN wherever nothing was written."""

    def __init__(self, dtype, D, window, n_seqs, room=800):
        from torchless_rs_amd.cache.cache import NO_RING
        from torchless_rs_amd.parts.base import Workspace
        self.dt, self.ring = TORCH[dtype], -(-window // 64) if window else NO_RING
        per = min(-(-room // 64), self.ring)
        order = torch.randperm(n_seqs * per + 3, generator=torch.Generator().manual_seed(D))
        self.table = order[:n_seqs * per].view(n_seqs, per).to(torch.int32)
        self.pages = torch.full((n_seqs * per + 3, 64 * D), float("nan"), dtype=self.dt, device="cuda")
        self.length = [0] * n_seqs
        self.ws = Workspace(torch.device("cuda"))

    def step(self, seqs, take):
        from torchless_rs_amd.kernels import ops
        i32 = dict(dtype=torch.int32, device="cuda")
        before = [self.length[s] for s in seqs]
        after = [c + m for c, m in zip(before, take)]
        offs, cols = ops.aligned_columns(before, take)
        group = types.SimpleNamespace(storage=[self.pages], ring_pages=self.ring,
                                      pages_needed=lambda n: min(-(-n // 64), self.ring))
        ctx = types.SimpleNamespace(
            row_seq=torch.repeat_interleave(torch.arange(len(seqs)), torch.tensor(take)).to(**i32),
            row_pos=torch.cat([torch.arange(c, a) for c, a in zip(before, after)]).to(**i32),
            cu_seqlens=torch.tensor(np.concatenate([[0], np.cumsum(take)]), **i32), len_before=torch.tensor(before, **i32),
            len_after=torch.tensor(after, **i32), tile_off=torch.tensor(offs, **i32), all_single=all(m == 1 for m in take),
            workspace=self.ws, dtype=self.dt, tables={0: dev(self.table[seqs].contiguous())}, pending=None,
            host={"n_new": np.asarray(take), "len_before": np.asarray(before), "aligned_cols": cols})
        for s, a in zip(seqs, after):
            self.length[s] = a
        return ctx, types.SimpleNamespace(kv_group=group, kv_layer=0, kv_group_index=0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("q_rank", [None, 24])
@pytest.mark.parametrize("H, dn, dr, dv, R", [(3, 11, 6, 21, 37), (16, 32, 16, 48, 128), (2, 64, 32, 64, 256), (1, 8, 0, 8, 16)])
@pytest.mark.parametrize("window", [None, 1, 65, 130])
def test_the_latent_mixer_in_steps_of_any_size(dtype, q_rank, H, dn, dr, dv, R, window):
    """Whole prompts, portions from two rows up that start and end at pages' and windows' edges, single tokens, and
    sequences that bring unequal numbers of rows, all over the same pages; with and without a latent of the queries."""
    from torchless_rs_amd.parts.attention_latent_cache import LatentCacheAttentionMixer
    from torchless_rs_amd.parts.base import PartSpec
    W, eps, scale = 64, 1e-5, 1.5 / math.sqrt(dn + dr)
    _, m = latent(H, dn, dr, dv, R, scale, window=window, base=100.0, scaling=(4.0, 64.0, 8.0, 1.0) if dr else None)
    g = torch.Generator().manual_seed(H + R)
    shapes = {"dkv": (R + dr, W), "uk": (H * dn, R), "uv": (H * dv, R), "o": (W, H * dv)}
    shapes.update({"dq": (q_rank, W), "uq": (H * (dn + dr), q_rank)} if q_rank else {"q": (H * (dn + dr), W)})
    w = {"mix." + k: (torch.randn(s, generator=g) / math.sqrt(s[1])).to(torch.bfloat16) for k, s in shapes.items()}
    w["mix.dkv.norm"] = (1 + 0.3 * torch.randn(R, generator=g)).to(torch.bfloat16)
    if q_rank:
        w["mix.dq.norm"] = (1 + 0.3 * torch.randn(q_rank, generator=g)).to(torch.bfloat16)
    position = PartSpec("rotary", {"head_dim": dr, "theta": 100.0, "rotary_dim": dr, "interleaved": True,
                                   "scaling": m["rot"]["scaling"]}) if dr else None
    part = LatentCacheAttentionMixer(W, H, dn, dv, R, scale, eps, rot_dim=dr, position=position, window=window, q_rank=q_rank)
    assert {k: tuple(v.shape) for k, v in part.weight_specs().items()} == {k: tuple(v.shape) for k, v in w.items()}
    part.load({k: dev(v if dtype == "bfloat16" else v.float()) for k, v in w.items()}, TORCH[dtype])
    lens = [300, 131]
    hs = [torch.randn(L, W, generator=g).to(TORCH[dtype]) for L in lens]
    w64 = {k: v.double() for k, v in w.items()}
    if q_rank:      # the plain mixer projects h itself: hand it the product of the two, row by row
        def want_of(h):
            a = plain.rms(h @ w64["mix.dq"].T, eps) * w64["mix.dq.norm"]
            both = torch.cat([h, a], dim=1)
            pad = {"mix.q": torch.cat([torch.zeros(H * (dn + dr), W, dtype=F64), w64["mix.uq"]], dim=1),
                   "mix.dkv": torch.cat([w64["mix.dkv"], torch.zeros(R + dr, q_rank, dtype=F64)], dim=1)}
            return plain.latent_attention(both, dict(w64, **pad), "mix.", m, torch.arange(len(h)), eps)
    else:
        def want_of(h):
            return plain.latent_attention(h, w64, "mix.", m, torch.arange(len(h)), eps)
    want = [want_of(h.double()) for h in hs]
    tol = 3e-5 if dtype == "float32" else 2e-2
    for cuts in ([(300, 131)], [(64, 1), (1, 63), (2, 2), (63, 64), (65, 1), (105, 0)], [(130, 2)] + [(1, 1)] * 40 + [(2, 3)] * 5 + [(120, 74)]):
        seqs = LatentSequences(dtype, R + dr, window, 2)
        outs = [[], []]
        for cut in cuts:
            live = [s for s in range(2) if seqs.length[s] < lens[s] and cut[s]]
            take = [min(cut[s], lens[s] - seqs.length[s]) for s in live]
            y = torch.cat([hs[s][seqs.length[s]:seqs.length[s] + t] for s, t in zip(live, take)])
            ctx, run = seqs.step(live, take)
            out = torch.empty(y.shape[0], W, device="cuda")
            part.produce(ctx, run, dev(y), out)
            at = 0
            for s, t in zip(live, take):
                outs[s].append(out[at:at + t].clone())
                at += t
        for s in range(2):
            got = torch.cat(outs[s])
            assert rel_err(got, want[s][:len(got)]) < tol, (cuts[:3], s)


# ---------------------------------------------------------------------------------------------
# whole models through the engine
# ---------------------------------------------------------------------------------------------

def plain_run(w, cfg, ids):
    """Logits and, per row, the smallest gap by which a router chose at that row or before it (retention carries a
    choice's outcome on)."""
    margins = []
    lg = plain.forward(w, cfg, ids, margins=margins)
    m = torch.stack(margins).min(dim=0).values if margins else torch.ones(len(ids), dtype=F64)
    return lg, m


def weights_for(cfg, seed, dtype):
    """For the bfloat16 runs the corrections lie more than a score's whole range apart (a choice that rounding turns changes the keys
    and states of every row behind it, and one of some hundred rows would always be that close): the choice is then the
    same for every row, with weights that are not.  The float32 runs choose row by row, and so do the routers' own tests."""
    w = plain.random_weights(cfg, seed=seed)
    if dtype == "bfloat16":
        g = torch.Generator().manual_seed(seed)
        for k in w:
            if k.endswith(".correction"):
                w[k] = (-3.0 * 2.0 ** torch.randperm(w[k].numel(), generator=g)).to(w[k].dtype)      # (sums of two differ too)
    return w


@pytest.fixture(scope="module")
def zoo(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("zudalorn")
    out = {}
    for i, name in enumerate(NAMES):
        cfg = copy.deepcopy(CONFIGS[name])
        ps = some_prompts(cfg["vocab"], LENGTHS[name], seed=51 + i)
        for dtype in DTYPES:
            w = weights_for(cfg, 70 + i, dtype)
            runs = [plain_run(w, cfg, p) for p in ps]
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
    for g in eng.cache.groups:              # stale rows and states must never be read: make them NaN
        g.storage.fill_(float("nan"))
    for t in eng.cache.state.values():
        t.fill_(float("nan"))
    return eng


def close(got, want, dtype, what, margin=None, tol=None, rms=None):
    """Rows whose routers chose by a wide enough margin must agree (a choice made by a hair may fall the other way under
    rounding, and then the row is another function's)."""
    loose = FEW_CHANNELS.get(what[0] if isinstance(what, tuple) else what, 1.0) if dtype == "bfloat16" else 1.0
    tol, rms = (tol or TOL[dtype]) * loose, rms if rms is False else (rms or RMS[dtype]) * loose
    got = got.detach().double().cpu()
    assert torch.isfinite(got).all(), what
    if margin is not None:
        sure = margin > MARGIN[dtype]
        assert sure.all() if dtype == "bfloat16" else int(sure.sum()) * 20 >= len(sure) * 19 or len(sure) < 20, (what, "too few sure rows")
        got, want = got[sure], want[sure]
    if not len(got):
        return
    assert rel_err(got, want) < tol, (what, rel_err(got, want))
    if rms is not False:
        assert rms_err(got, want) < rms, (what, rms_err(got, want))


def test_the_right_parts_and_caches_are_chosen(zoo):
    from torchless_rs_amd.kernels import ops
    from torchless_rs_amd.parts.attention_latent_cache import LatentCacheAttentionMixer
    from torchless_rs_amd.parts.block import SandwichNormBlock
    from torchless_rs_amd.parts.ffn_routed import PlainFeedForward, RoutedExperts
    from torchless_rs_amd.parts.retention import RetentionMixer
    eng = engine_for(zoo, "cores", "bfloat16")
    blocks = eng.model.blocks
    assert all(isinstance(b, SandwichNormBlock) and b.mixer_out_norm.scalar for b in blocks)
    assert [type(b.mixer) for b in blocks] == [LatentCacheAttentionMixer, RetentionMixer] * 2 + [LatentCacheAttentionMixer]
    assert [type(b.ffn) for b in blocks] == [RoutedExperts, PlainFeedForward, RoutedExperts, type(None), PlainFeedForward]
    assert sorted(eng.cache.state) == [1, 3] and eng.cache.state[1].dtype == torch.float32
    assert [g.request.value_dim for g in eng.cache.groups] == [0, 0, 0]
    assert [g.storage.shape[2] for g in eng.cache.groups] == [64 * 160, 64 * 288, 64 * 576]
    assert [g.ring_pages for g in eng.cache.groups][:2] == [2, 3]
    assert all(ops.latents_on_matrix_cores(torch.bfloat16, b.mixer.R, b.mixer.dr) for b in blocks if isinstance(b.mixer, LatentCacheAttentionMixer))
    assert not ops.latents_on_matrix_cores(torch.float32, 512, 64) and not ops.wide_on_matrix_cores(torch.float32, 64, 64)


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
    close(lg[:k], z["want"][3][80:], dtype, (name, "goes on beside others"), z["margin"][3][80:])
    close(lg[k:k + len(q)], z["want"][2], dtype, (name, "begins beside others"), z["margin"][2])
    close(lg[k + len(q):], z["want"][1][-1:], dtype, (name, "a single token beside others"), z["margin"][1][-1:])
    assert not eng.cache.length


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_long_decoding_past_every_window(zoo, name, dtype):
    """A short prompt, then 300 tokens one by one (through captured graphs): every window passes over decoded tokens, the
    rings of pages wrap, the recurrent state is carried 300 times."""
    from torchless_rs_amd.engine import SeqInput
    eng, z = engine_for(zoo, name, dtype), zoo[name, dtype]
    ids = some_prompts(z["cfg"]["vocab"], [310], seed=78)[0]
    want, m = plain_run(z["w"], z["cfg"], ids)
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
    """The same prompt's shape three times, then with cached rows before it, then again: replays beside eager steps, each
    against the plain logits."""
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


def test_a_long_prompt_goes_by_chunks_and_many_rows_expert_by_expert(zoo, monkeypatch):
    from torchless_rs_amd.engine import SeqInput
    from torchless_rs_amd.kernels import ops
    from torchless_rs_amd.parts import ffn_routed
    monkeypatch.setattr(ffn_routed, "GROUPED_ROWS_PER_EXPERT", 1)
    calls, chunks = [], []
    inner = ffn_routed.RoutedExperts._grouped
    monkeypatch.setattr(ffn_routed.RoutedExperts, "_grouped", lambda self, *a: (calls.append(a[1].shape[0]), inner(self, *a))[1])
    by_chunks = ops.retention_chunks
    monkeypatch.setattr(ops, "retention_chunks", lambda *a: (chunks.append(a[12]), by_chunks(*a))[1])
    eng, z = engine_for(zoo, "cores", "bfloat16"), zoo["cores", "bfloat16"]
    p, q = z["prompts"][3], z["prompts"][2]
    s = eng.alloc()
    got = eng.step([SeqInput(s, p, list(range(len(p))))]).clone()
    eng.free(s)
    assert calls == [len(p)] * 2 and chunks == [2, 2], (calls, chunks)
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
        if rng.random() < 0.5:
            H, d = rng.choice([1, 2, 3, 5]), rng.choice([8, 16, 24, 33, 64, 128])
            dims = rng.choice([0, d // 4 * 2, d // 2 * 2])
            mix = ret(H, d, rng.choice([8, 20, 32, 64, 96]), [rng.choice([0.5, 0.9, 0.99, 0.9995]) for _ in range(H)],
                      rot=(rng.choice([100.0, 1e4, 1e6]), dims) if dims else None)
        else:
            dr = rng.choice([4, 8, 16, 32])
            mix = latent(rng.choice([1, 3, 4, 8, 20]), rng.choice([8, 16, 24, 64]), dr, rng.choice([8, 16, 40, 64, 100]),
                         rng.choice([16, 48, 64, 136, 256]), rng.uniform(0.1, 0.4), window=rng.choice([None, 17, 40, 64, 100, 200]),
                         base=rng.choice([300.0, 1e4, 5e5]),
                         scaling=rng.choice([None, (4.0, 128.0, 16.0, 1.0), (40.0, 64.0, 32.0, 1.0), (2.0, 1000.0, 4.0, 2.0)]))
        f = None
        r = rng.random()
        if r < 0.4:
            f = dense(rng.choice([16, 40, 96, 200]))
        elif r < 0.85:
            E = rng.choice([1, 2, 4, 6, 8, 16])
            G = rng.choice([g for g in (1, 2, 4) if E % g == 0])
            keep = rng.randint(1, G)
            top = rng.randint(1, min(4, keep * (E // G)))
            f = moe(E, top, rng.choice([8, 16, 32]), groups=(G, keep) if rng.random() < 0.7 else None,
                    shared=rng.choice([None, 8, 32, 50]))
        layers.append(layer(mix, f))
    return model(rng.choice([97, 256, 500]), rng.choice([64, 96, 128, 160, 250]), rng.choice([1e-5, 1e-6]), layers)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(8))
def test_random_configurations(seed, dtype, tmp_path):
    """Whole prompts, a prompt with its last tokens one by one, and all of them in one batch that is decoded together."""
    from torchless_rs_amd.engine import Engine, SeqInput, load_model
    loose = {} if dtype == "float32" else dict(tol=0.15, rms=5e-2)       # (some draw heads of few channels)
    cfg = random_config(random.Random(seed))
    w = weights_for(cfg, 100 + seed, dtype)
    ps = some_prompts(cfg["vocab"], [1, 37, 150, 420], seed=seed)
    runs = [plain_run(w, cfg, p) for p in ps]
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
