"""Decode and prefill throughput of the Mistral-7B-v0.1 shape on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--context 8192] [--layers L]
                    [--shape 7b-v0.1|7b-v0.3|nemo-12b] [--only decode|prefill] [--prefill-tokens T]
                    [--no-points] [--no-kernels] [--no-workloads] [--no-tiled-copies]

One JSON line: decoded tokens a second of the default run (batch 8 at the
context length of the configuration), the prefill of one 2,048-token prompt,
the decode step's share of the HBM roofline, decoding at batch 1 and 64
("points"), the step's kernels one by one with their own shares of the HBM
roofline ("kernels"), the baseline's configurations as it words them, run
through the generation loop ("workloads"), and what a plain read and a chain
of MFMAs reach on the machine ("ceilings").  Weights are random (seeded),
token ids synthetic.  The context is built by a real prefill of synthetic
prompts.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

HBM_PEAK_GBS = 8000.0                 # MI355X, published
PEAK_TFLOPS = {"bf16": 2500.0, "fp32": 157.3}

# Mistral-7B-v0.1 shape: the third configuration of the baseline, and the default
SHAPE = dict(num_hidden_layers=32, hidden_size=4096, num_attention_heads=32, num_key_value_heads=8,
             head_dim=128, intermediate_size=14336, vocab_size=32000, rope_theta=10000.0,
             sliding_window=4096, rms_norm_eps=1e-5)
# the baseline's other shapes of the same architecture, for --shape
SHAPES = {
    "7b-v0.1": ("Mistral-7B-v0.1 shape", SHAPE),
    "7b-v0.3": ("Mistral-7B-v0.3 shape", dict(SHAPE, vocab_size=32768, rope_theta=1e6, sliding_window=None)),
    "nemo-12b": ("Mistral-NeMo-12B shape", dict(SHAPE, num_hidden_layers=40, hidden_size=5120, vocab_size=131072,
                                                 rope_theta=1e6, sliding_window=None)),
}


# Layer sizes that resemble real models, for --only designs: both designs are built with these
DESIGN_SIZES = {
    "2b": dict(width=2048, heads=32, kv_heads=8, dim=64, ff=8192, window=1024, vocab=32000),
    "7b": dict(width=4096, heads=32, kv_heads=8, dim=128, ff=14336, window=4096, vocab=32000),
    "12b": dict(width=5120, heads=32, kv_heads=8, dim=128, ff=14336, window=None, vocab=131072),
}


def design_configs(z: dict, layers: int, share_from=None):
    """config.json of a Sozetar and of a Mistral model with the layer sizes `z`.  `share_from`: the
    Sozetar layers behind that index read its keys and values instead of making their own."""
    def mixer(i):
        m = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["dim"],
             "scale": z["dim"] ** -0.5, "q_temp": {"coef": 0.25, "every": 256}}
        if z["window"]:
            m["mask"] = {"size": z["window"]}
        if share_from is not None and i > share_from:
            m["kv_from"] = share_from
        return m
    soz = {"architecture": "Sozetar", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-6},
           "layers": [{"type": "attention", "mixer": mixer(i), "mlp": {"kind": "dense", "ff": z["ff"]}}
                      for i in range(layers)]}
    mis = dict(architectures=["MistralForCausalLM"], num_hidden_layers=layers, hidden_size=z["width"],
               num_attention_heads=z["heads"], num_key_value_heads=z["kv_heads"], head_dim=z["dim"],
               intermediate_size=z["ff"], vocab_size=z["vocab"], rope_theta=10000.0, sliding_window=z["window"],
               rms_norm_eps=1e-5)
    return soz, mis


def fanitar_config(z: dict, layers: int):
    """config.json of a Fanitar model with the layer sizes `z`: layers out of latents and differential
    layers in turn.  The differential layers have half the heads with two maps each and values of two
    maps' width, so that every projection is as large as the other designs'; the latents are 3/8 and
    1/8 of the width."""
    def mixer(i):
        if i % 2 == 0:
            m = {"heads": z["heads"], "dim": z["dim"], "vdim": z["dim"], "q_rank": 3 * z["width"] // 8,
                 "kv_rank": z["width"] // 8, "scale": z["dim"] ** -0.5}
            if z["window"]:
                m["mask"] = {"size": z["window"]}
            return "latent_attention", m
        return "attention", {"heads": z["heads"] // 2, "kv_heads": z["kv_heads"] // 2, "dim": z["dim"], "vdim": 2 * z["dim"],
                             "scale": z["dim"] ** -0.5, "diff": 0.5, "rot": {"base": 10000.0, "dims": z["dim"]}}
    return {"architecture": "Fanitar", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-6},
            "embedding": {"scale": 1.0}, "logit_scale": 1.0,
            "layers": [{"type": mixer(i)[0], "mixer": mixer(i)[1], "mlp": {"kind": "dense", "ff": z["ff"], "limit": 7.0}}
                       for i in range(layers)]}


def fanitar_counts(z: dict, layers: int, B: int, C: int, T: int):
    """(weight elements of the layers' products, bytes of keys and values that a decode step reads, multiply-adds
    times two of a prompt's attention) of `fanitar_config(z, layers)`.  The layers out of latents keep keys and
    values per head (every head its own), the differential ones one key of two maps and one value per KV head;
    a differential head's two maps are counted with the d channels each that they have."""
    H, I, nq, nkv, d = z["width"], z["ff"], z["heads"], z["kv_heads"], z["dim"]
    qr, kvr = 3 * H // 8, H // 8
    w = kv = att = 0
    for i in range(layers):
        w += 3 * I * H
        if i % 2 == 0:
            held = min(C, z["window"]) if z["window"] else C
            w += qr * H + nq * d * qr + kvr * H + 2 * nq * d * kvr + 2 * nq * d * H
            kv += B * held * nq * 2 * d * 2
            att += 4 * nq * d * sum(min(p + 1, z["window"] or T) for p in range(T))
        else:
            w += 2 * nq * d * H + 2 * nkv * d * H
            kv += B * C * (nkv // 2) * 4 * d * 2
            att += (nq // 2) * 2 * (2 * d + 2 * 2 * d) * T * (T + 1) // 2
    return w, kv, att


def nepisun_layers(z: dict, layers: int):
    """The layers of `nepisun_config(z, layers)` as (mixer kind, feed-forward kind): state-space layers and the two
    kinds of attention in turn, the first feed-forward dense, the others routed."""
    kinds = ["mamba2", "mamba2", "attention_2", "attention"]
    return [(kinds[i % 4], "dense" if i % 4 == 0 else "moe") for i in range(layers)]


def nepisun_sizes(z: dict):
    """Sizes of the Nepisun layers at the layer sizes `z`: a state-space mixer of twice the width in heads of 64
    with states of 128 rows; 16 experts of a quarter of the dense feed-forward's hidden size of which a token uses
    4, beside a shared one of half of it: a token multiplies as much as in the dense feed-forward."""
    return dict(ssm_heads=2 * z["width"] // 64, ssm_dv=64, state=128, groups=8, conv=4, experts=16, top=4,
                expert_ff=z["ff"] // 4, shared_ff=z["ff"] // 2, keep_first=64)


def nepisun_config(z: dict, layers: int):
    """config.json of a Nepisun model with the layer sizes `z` (see `nepisun_layers`, `nepisun_sizes`)."""
    n = nepisun_sizes(z)
    out = []
    for mix, ff in nepisun_layers(z, layers):
        if mix == "mamba2":
            m = {"heads": n["ssm_heads"], "vdim": n["ssm_dv"], "state": n["state"], "groups": n["groups"], "conv": n["conv"],
                 "norm_groups": n["groups"]}
        else:
            m = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["dim"], "scale": z["dim"] ** -0.5,
                 "rot": {"base": 10000.0, "dims": z["dim"]}, "v_mix": True}
            if mix == "attention_2" and z["window"]:
                m["mask"] = {"size": z["window"], "keep_first": n["keep_first"]}
        mlp = {"kind": "dense", "ff": z["ff"]} if ff == "dense" else {
            "kind": "moe", "router": {"experts": n["experts"], "top": n["top"], "groups": {"count": 4, "keep": 2}},
            "expert": {"ff": n["expert_ff"]}, "shared": {"ff": n["shared_ff"]}}
        out.append({"type": mix, "mixer": m, "mlp": mlp})
    return {"architecture": "Nepisun", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-6}, "layers": out}


def nepisun_counts(z: dict, layers: int, B: int, C: int, T: int):
    """(weight elements that a prompt's products multiply a row by, bytes of keys, values and recurrent state that a
    decode step reads and writes, multiply-adds times two of a prompt's attention and recurrence, weight elements that
    a decode step of B rows must read) of `nepisun_config(z, layers)`.  A routed feed-forward multiplies a row by its
    `top` experts and the shared one; a decode step reads the experts that B rows can choose at most."""
    H, I, nq, nkv, d = z["width"], z["ff"], z["heads"], z["kv_heads"], z["dim"]
    n = nepisun_sizes(z)
    inner, GN = n["ssm_heads"] * n["ssm_dv"], n["groups"] * n["state"]
    w = w_read = kv = att = 0
    for mix, ff in nepisun_layers(z, layers):
        if mix == "mamba2":
            m = (2 * inner + 2 * GN + n["ssm_heads"]) * H + H * inner
            kv += B * n["ssm_heads"] * n["state"] * n["ssm_dv"] * 4 * 2
            att += 4 * T * n["ssm_heads"] * n["state"] * n["ssm_dv"]
        else:
            m = 2 * nq * d * H + 2 * nkv * d * H + (nq * d * H if mix == "attention" else 0)
            reach = (z["window"] + n["keep_first"]) if (mix == "attention_2" and z["window"]) else None
            kv += B * (min(C, reach) if reach else C) * nkv * 2 * d * 2
            att += 4 * nq * d * sum(min(p + 1, reach or T) for p in range(T))
        w += m
        w_read += m
        if ff == "dense":
            w += 3 * I * H
            w_read += 3 * I * H
        else:
            w += 2 * H * (n["top"] * n["expert_ff"] + n["shared_ff"]) + n["experts"] * H
            w_read += 2 * H * (min(n["experts"], B * n["top"]) * n["expert_ff"] + n["shared_ff"]) + n["experts"] * H
    return w, kv, att, w_read


def giforax_layers(layers: int):
    """The mixers of `giforax_config(z, layers)`: attention with keys of its own, attention that reads the first
    layer's keys, a gated recurrence, attention, and so on; every layer has a routed feed-forward."""
    kinds = ["attention", "reader", "mingru", "attention"]
    return [kinds[i % 4] if i else "attention" for i in range(layers)]


def giforax_sizes(z: dict):
    """Sizes of the Giforax layers at the layer sizes `z`: a recurrence as wide as the model; 16 gated experts of an
    eighth of the dense feed-forward's hidden size of which a token uses 4, beside a shared one of half of it: a
    token multiplies as much as in the dense gated feed-forward.  Chunks as long as the other designs' window."""
    return dict(gru=z["width"], experts=16, top=4, expert_ff=z["ff"] // 8, shared_ff=z["ff"] // 2, chunk=z["window"])


def giforax_config(z: dict, layers: int):
    """config.json of a Giforax model with the layer sizes `z` (see `giforax_layers`, `giforax_sizes`)."""
    n = giforax_sizes(z)
    out = []
    for mix in giforax_layers(layers):
        if mix == "mingru":
            kind, m = "mingru", {"width": n["gru"]}
        else:
            kind = "attention"
            m = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["dim"], "scale": z["dim"] ** -0.5,
                 "rot": {"base": 10000.0, "dims": z["dim"] // 2}}
            if n["chunk"]:
                m["mask"] = {"size": n["chunk"]}
            if mix == "reader":
                m["kv_from"] = 0
        mlp = {"kind": "moe", "router": {"experts": n["experts"], "top": n["top"]},
               "expert": {"ff": n["expert_ff"], "limit": 7.0}, "shared": {"ff": n["shared_ff"], "limit": 7.0}}
        out.append({"type": kind, "mixer": m, "mlp": mlp})
    return {"architecture": "Giforax", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-6},
            "embedding": {"scale": 1.0}, "layers": out}


def giforax_counts(z: dict, layers: int, B: int, C: int, T: int):
    """(weight elements that a prompt's products multiply a row by, bytes of keys, values and recurrent state that a
    decode step reads and writes, multiply-adds times two of a prompt's attention, weight elements that a decode step
    of B rows must read) of `giforax_config(z, layers)`.  A position sees the keys of its own chunk alone; a routed
    feed-forward multiplies a row by its `top` experts and the shared one, and a decode step reads the experts that B
    rows can choose at most."""
    H, nq, nkv, d = z["width"], z["heads"], z["kv_heads"], z["dim"]
    n = giforax_sizes(z)
    chunk = n["chunk"]
    w = w_read = kv = att = 0
    for mix in giforax_layers(layers):
        if mix == "mingru":
            m = 4 * n["gru"] * H
            kv += B * n["gru"] * 4 * 2
        else:
            m = 2 * nq * d * H + nq * H + (2 * nkv * d * H if mix == "attention" else 0)
            seen = ((C - 1) % chunk + 1) if chunk else C
            kv += B * seen * nkv * 2 * d * 2
            att += 4 * nq * d * sum((p % chunk if chunk else p) + 1 for p in range(T))
        w += m + 3 * H * (n["top"] * n["expert_ff"] + n["shared_ff"]) + n["experts"] * H
        w_read += m + 3 * H * (min(n["experts"], B * n["top"]) * n["expert_ff"] + n["shared_ff"]) + n["experts"] * H
    return w, kv, att, w_read


def zudalorn_layers(layers: int):
    """(mixer, feed-forward) of `zudalorn_config(z, layers)`: both mixers with both feed-forwards in every four layers."""
    kinds = [("retention", "dense"), ("latent_attention", "moe"), ("retention", "moe"), ("latent_attention", "dense")]
    return [kinds[i % 4] for i in range(layers)]


def zudalorn_sizes(z: dict):
    """Sizes of the Zudalorn layers at the layer sizes `z`: as many heads of the same size in both mixers, latents of four
    heads' channels with half a head rotated beside them; an ungated feed-forward half as wide again as the gated one; 16
    gated experts of an eighth of its hidden size of which a token uses 4, beside a shared one of half of it: a token
    multiplies as much as in the dense gated feed-forward either way."""
    return dict(rank=4 * z["dim"], rot=z["dim"] // 2, dense_ff=3 * z["ff"] // 2, experts=16, top=4, expert_ff=z["ff"] // 8,
                shared_ff=z["ff"] // 2)


def zudalorn_config(z: dict, layers: int):
    """config.json of a Zudalorn model with the layer sizes `z` (see `zudalorn_layers`, `zudalorn_sizes`)."""
    n = zudalorn_sizes(z)
    out = []
    for mix, ff in zudalorn_layers(layers):
        if mix == "retention":
            m = {"heads": z["heads"], "dim": z["dim"], "vdim": z["dim"], "rot": {"base": 10000.0, "dims": z["dim"]},
                 "decay": [1.0 - 2.0 ** (-5.0 - 7.0 * h / max(1, z["heads"] - 1)) for h in range(z["heads"])]}
        else:
            m = {"heads": z["heads"], "dim": z["dim"], "rot_dim": n["rot"], "vdim": z["dim"], "kv_rank": n["rank"],
                 "scale": (z["dim"] + n["rot"]) ** -0.5,
                 "rot": {"base": 10000.0, "dims": n["rot"], "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
            if z["window"]:
                m["mask"] = {"size": z["window"]}
        mlp = {"kind": "dense", "ff": n["dense_ff"]} if ff == "dense" else {
            "kind": "moe", "router": {"experts": n["experts"], "top": n["top"], "groups": {"count": 4, "keep": 2}},
            "expert": {"ff": n["expert_ff"]}, "shared": {"ff": n["shared_ff"]}}
        out.append({"type": mix, "mixer": m, "mlp": mlp})
    return {"architecture": "Zudalorn", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-6}, "layers": out}


def zudalorn_counts(z: dict, layers: int, B: int, C: int, T: int):
    """(weight elements that a prompt's products multiply a row by, bytes of cached latents and recurrent state that a
    decode step reads and writes, multiply-adds times two of a prompt's attention and recurrence, weight elements that
    a decode step of B rows must read) of `zudalorn_config(z, layers)`.  A prompt makes keys and values per head of its
    latents; a decode step reads the latents as they are."""
    H, nq, d = z["width"], z["heads"], z["dim"]
    n = zudalorn_sizes(z)
    w = w_read = kv = att = 0
    for mix, ff in zudalorn_layers(layers):
        if mix == "retention":
            m = 5 * nq * d * H
            kv += B * nq * d * d * 4 * 2
            att += 4 * T * nq * d * d
        else:
            m = nq * (d + n["rot"]) * H + (n["rank"] + n["rot"]) * H + 2 * nq * d * n["rank"] + nq * d * H
            kv += B * (min(C, z["window"]) if z["window"] else C) * (n["rank"] + n["rot"]) * 2
            att += 2 * nq * (2 * d + n["rot"]) * sum(min(p + 1, z["window"] or T) for p in range(T))
        w += m
        w_read += m
        if ff == "dense":
            w += 2 * H * n["dense_ff"]
            w_read += 2 * H * n["dense_ff"]
        else:
            w += 3 * H * (n["top"] * n["expert_ff"] + n["shared_ff"]) + n["experts"] * H
            w_read += 3 * H * (min(n["experts"], B * n["top"]) * n["expert_ff"] + n["shared_ff"]) + n["experts"] * H
    return w, kv, att, w_read


def zifetar_layers(layers: int):
    """The mixers of `zifetar_config(z, layers)`: all three in every four layers, each with a routed feed-forward."""
    kinds = ["parallel", "channel_delta", "retention", "parallel"]
    return [kinds[i % 4] for i in range(layers)]


def zifetar_sizes(z: dict):
    """Sizes of the Zifetar layers at the layer sizes `z`: attention as the other designs have it beside a linear attention of
    half as many heads; a delta rule and retention with as many heads as the attention; 16 gated experts of a quarter of the
    dense feed-forward's hidden size of which a token uses 4: a token multiplies as much as in the dense gated one.  Chunks as
    long as the other designs' window."""
    return dict(lin_heads=z["heads"] // 2, inner=16, experts=16, top=4, expert_ff=z["ff"] // 4, chunk=z["window"])


def zifetar_config(z: dict, layers: int):
    """config.json of a Zifetar model with the layer sizes `z` (see `zifetar_layers`, `zifetar_sizes`)."""
    n, d = zifetar_sizes(z), z["dim"]
    out = []
    for mix in zifetar_layers(layers):
        if mix == "channel_delta":
            m = {"heads": z["heads"], "kv_heads": z["heads"], "dim": d, "vdim": d, "conv": 4}
        elif mix == "retention":
            m = {"heads": z["heads"], "dim": d, "vdim": d, "rot": {"base": 10000.0, "dims": d},
                 "decay": [1.0 - 2.0 ** (-5.0 - 7.0 * h / max(1, z["heads"] - 1)) for h in range(z["heads"])]}
        else:
            left = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": d, "vdim": d, "scale": d ** -0.5,
                    "rot": {"base": 500000.0, "dims": d, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
            if n["chunk"]:
                left["mask"] = {"size": n["chunk"]}
            m = {"left": left, "right": {"heads": n["lin_heads"], "dim": d, "vdim": d, "tau": 16.0}, "left_scale": 0.7,
                 "right_scale": 0.7}
        out.append({"type": mix, "mixer": m, "mlp": {"kind": "moe", "router": {"experts": n["experts"], "top": n["top"]},
                                                     "expert": {"ff": n["expert_ff"]}}})
    return {"architecture": "Zifetar", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-6},
            "embedding": {"scale": 1.0, "bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 1}}, "layers": out}


def zifetar_counts(z: dict, layers: int, B: int, C: int, T: int):
    """(weight elements that a prompt's products multiply a row by, bytes of keys, values and recurrent state that a
    decode step reads and writes, multiply-adds times two of a prompt's attention and recurrences, weight elements that a
    decode step of B rows must read) of `zifetar_config(z, layers)`.  A position sees the keys of its own chunk alone; a
    routed feed-forward multiplies a row by its `top` experts, and a decode step reads the experts that B rows can choose at
    most.  A recurrence counts as its row-by-row form: two products with the state a row, three by the delta rule."""
    H, nq, nkv, d = z["width"], z["heads"], z["kv_heads"], z["dim"]
    n = zifetar_sizes(z)
    chunk, nl = n["chunk"], n["lin_heads"]
    w = w_read = kv = att = 0
    for mix in zifetar_layers(layers):
        if mix == "channel_delta":
            m = 4 * nq * d * H + nq * H + 2 * d * H + 2 * nq * d * d
            kv += B * (nq * d * d + 3 * 3 * nq * d) * 4 * 2
            att += 6 * T * nq * d * d
        elif mix == "retention":
            m = 5 * nq * d * H
            kv += B * nq * d * d * 4 * 2
            att += 4 * T * nq * d * d
        else:
            m = 2 * nq * d * H + 2 * nkv * d * H + 5 * nl * d * H + n["inner"] * (H + nl * d)
            seen = ((C - 1) % chunk + 1) if chunk else C
            kv += B * (seen * nkv * 2 * d * 2 + nl * d * d * 4 * 2)
            att += 4 * nq * d * sum((p % chunk if chunk else p) + 1 for p in range(T)) + 4 * T * nl * d * d
        w += m + 3 * H * n["top"] * n["expert_ff"] + n["experts"] * H
        w_read += m + 3 * H * min(n["experts"], B * n["top"]) * n["expert_ff"] + n["experts"] * H
    return w, kv, att, w_read


def bench_designs(args) -> int:
    """Prefill (one prompt of --prefill-tokens in one step) and decode (--batch sequences at --context
    positions, one token a step through captured graphs) of the designs at equal layer sizes,
    random weights, bfloat16.  The bytes a decode step must read (every weight once, the live keys
    and values) over its time is its share of the HBM roofline; a prefill's products and causal
    attention over its time its share of the matrix cores' peak."""
    import torch
    from torchless_rs_amd import config_from_dict
    from torchless_rs_amd.engine import Engine, SeqInput, model_from_tensors
    from torchless_rs_amd.kernels.page import PAGE, round_up
    from torchless_rs_amd.models import model_spec_for
    from torchless_rs_amd.weights import random_tensors
    dev = "cuda:0"
    L = args.layers or 4
    B, C, T = args.batch, min(args.context, 4096), args.prefill_tokens
    gen = torch.Generator().manual_seed(11)
    out = {"metric": "designs_side_by_side", "dtype": "bf16", "data": "synthetic", "layers": L, "batch": B,
           "context": C, "prefill_tokens": T, "steps": args.steps, "warmup": args.warmup, "sizes": {}}

    def measure(cfgd, z, shared_layers=0, counts=None):
        cfg = config_from_dict(cfgd)
        tensors = random_tensors(model_spec_for(cfg).weight_specs(), seed=5, std=0.02, dtype=torch.bfloat16, device=dev)
        model = model_from_tensors(cfg, tensors, "bfloat16", dev)
        del tensors
        V = z["vocab"]
        held = min(C, z["window"]) if z["window"] else C
        room = C if counts is not None else held          # (a design whose layers differ: some keep every position)
        eng = Engine(model, max_tokens=max(B * (round_up(room) + PAGE), round_up(T) + PAGE), max_slots=max(B, 1),
                     freeze_gc=False)
        # prefill
        ids = torch.randint(0, V, (T,), generator=gen).tolist()
        times = []
        for i in range(2 + 3):
            s = eng.alloc()
            torch.cuda.synchronize()
            t = time.perf_counter()
            eng.step([SeqInput(s, ids, [T - 1])])
            torch.cuda.synchronize()
            times.append(time.perf_counter() - t)
            eng.free(s)
        pre = min(times[2:])
        # decode
        slots = [eng.alloc() for _ in range(B)]
        plen = max(1, C - args.steps - args.warmup - 1)
        for s in slots:
            p = torch.randint(0, V, (plen,), generator=gen).tolist()
            for c0 in range(0, plen, 2048):
                eng.step([SeqInput(s, p[c0:c0 + 2048], [])])
        for _ in range(args.warmup + 2):                      # (the second step of a shape captures its graph)
            eng.step([SeqInput(s, [7], [0]) for s in slots])
        torch.cuda.synchronize()
        t = time.perf_counter()
        for _ in range(args.steps):
            eng.step([SeqInput(s, [7], [0]) for s in slots])
        torch.cuda.synchronize()
        dec = (time.perf_counter() - t) / args.steps
        for s in slots:
            eng.free(s)
        eng.close()
        H, I, nq, nkv, d = z["width"], z["ff"], z["heads"], z["kv_heads"], z["dim"]
        own = L - shared_layers
        w_elems = L * (2 * nq * d * H + 3 * I * H) + own * 2 * nkv * d * H + V * H      # (biases, norms, gates: noise)
        kv_bytes = B * held * 2 * nkv * d * 2 * L           # every layer reads its keys and values, shared or not
        flops = 2 * T * (w_elems - V * H) + 2 * V * H + L * 4 * nq * d * sum(min(p + 1, z["window"] or T) for p in range(T))
        if counts is not None:
            w_elems, kv_bytes, att = counts[0] + V * H, counts[1], counts[2]
            flops = 2 * T * counts[0] + 2 * V * H + att
            if len(counts) > 3:                               # (what a decode step reads is not what a row multiplies)
                w_elems = counts[3] + V * H
        return {"prefill_ms": round(pre * 1e3, 3), "prefill_tok_s": round(T / pre),
                "prefill_frac_of_2.5_pflops": round(flops / pre / 2.5e15, 3),
                "decode_ms": round(dec * 1e3, 3), "decode_tok_s": round(B / dec),
                "decode_frac_of_8_tbs": round((2 * w_elems + kv_bytes) / dec / 8e12, 3)}

    for name in [n for n in args.design_sizes.split(",") if n]:
        z = DESIGN_SIZES[name]
        soz, mis = design_configs(z, L)
        which = [n for n in args.design_names.split(",") if n]
        row = {}
        if "fanitar" in which:
            row["fanitar"] = measure(fanitar_config(z, L), z, counts=fanitar_counts(z, L, B, C, T))
        if "nepisun" in which:
            row["nepisun"] = measure(nepisun_config(z, L), z, counts=nepisun_counts(z, L, B, C, T))
        if "giforax" in which:
            row["giforax"] = measure(giforax_config(z, L), z, counts=giforax_counts(z, L, B, C, T))
        if "zudalorn" in which:
            row["zudalorn"] = measure(zudalorn_config(z, L), z, counts=zudalorn_counts(z, L, B, C, T))
        if "zifetar" in which:
            row["zifetar"] = measure(zifetar_config(z, L), z, counts=zifetar_counts(z, L, B, C, T))
        if "sozetar" in which:
            row["sozetar"] = measure(soz, z)
        if "mistral" in which:
            row["mistral"] = measure(mis, z)
        if L > 2 and "sozetar" in which:
            row["sozetar_sharing_keys"] = measure(design_configs(z, L, share_from=L // 2 - 1)[0], z, L - L // 2)
        out["sizes"][name] = dict(z, **row)
        print(f"[bench] {name}: {json.dumps(row)}", file=sys.stderr, flush=True)
    print(json.dumps(out), flush=True)
    return 0


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=32)
    ap.add_argument("--warmup", type=int, default=4)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=8192)
    ap.add_argument("--shape", choices=sorted(SHAPES), default="7b-v0.1")
    ap.add_argument("--layers", type=int, default=None, help="fewer layers than the shape has")
    ap.add_argument("--prefill-tokens", type=int, default=2048)
    ap.add_argument("--no-points", action="store_true", help="skip batch 1 and 64")
    ap.add_argument("--no-kernels", action="store_true", help="skip the timing of the step's kernels one by one")
    ap.add_argument("--no-workloads", action="store_true", help="skip the baseline's configurations as it words them")
    ap.add_argument("--no-tiled-copies", action="store_true",
                    help="keep no second copies of q|k|v, o and down in the layout that single-token steps stream")
    ap.add_argument("--workload", choices=["baseline"], default="baseline",
                    help="the baseline's configurations as it words them (unequal prompt lengths drawn from a seed, "
                         "256/128/128 new tokens, temperature 0.7 for the NeMo shape) run through the generation "
                         "loop, under 'workloads' (the default; --no-workloads skips them)")
    ap.add_argument("--only", choices=["prefill", "decode", "pipes", "designs"], default=None,
                    help="measure one phase only and print its line to stderr (for profiling); pipes: whether a "
                         "SIMD's matrix and vector pipes overlap (ops.measure_pipes); designs: prefill and decode of "
                         "the Fanitar, Sozetar, Nepisun, Giforax, Zudalorn and Zifetar designs beside the Mistral design at equal layer sizes (--design-sizes, "
                         "--layers, --batch, --context, --prefill-tokens apply)")
    ap.add_argument("--design-names", default="fanitar,sozetar,mistral",
                    help="with --only designs: which designs to run (of fanitar, sozetar, nepisun, giforax, zudalorn, zifetar, mistral)")
    ap.add_argument("--design-sizes", default="2b,7b,12b",
                    help="with --only designs: which layer sizes to run (of %s)" % ",".join(sorted(DESIGN_SIZES)))
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py measures one GPU; --gpus {args.gpus} is not served")
        return 2

    import torch
    if args.only == "pipes":
        from torchless_rs_amd.kernels import ops as _o
        print(json.dumps({"pipes_ns_per_iteration": _o.measure_pipes("cuda:0")}), flush=True)
        return 0
    if args.only == "designs":
        return bench_designs(args)
    from torchless_rs_amd import SamplingConfig, config_from_dict
    from torchless_rs_amd.engine import Engine, SeqInput, model_from_tensors
    from torchless_rs_amd.engine.generate import BatchRun
    from torchless_rs_amd.kernels.page import PAGE, round_up
    from torchless_rs_amd.models import model_spec_for
    from torchless_rs_amd.sampling.sampler import Sampler
    from torchless_rs_amd.weights import random_tensors

    shape_name, shape = SHAPES[args.shape]
    if args.layers is None:
        args.layers = shape["num_hidden_layers"]
    cfgd = dict(shape, architectures=["MistralForCausalLM"], num_hidden_layers=args.layers)
    cfg = config_from_dict(cfgd)
    dev = "cuda:0"
    t0 = time.time()
    tensors = random_tensors(model_spec_for(cfg).weight_specs(), seed=5, std=0.02,
                             dtype=torch.bfloat16, device=dev)
    model = model_from_tensors(cfg, tensors, "bfloat16", dev, tiled_copies=not args.no_tiled_copies)
    del tensors
    torch.cuda.synchronize()
    resident_gib = round(torch.cuda.memory_allocated() / 2 ** 30, 2)     # weights and their tiled copies
    print(f"[bench] weights ready in {time.time() - t0:.1f} s", file=sys.stderr, flush=True)

    L, H, I, V = args.layers, cfg.hidden_size, cfg.intermediate_size, cfg.vocab_size
    nq, nkv, d, W = cfg.num_attention_heads, cfg.num_key_value_heads, cfg.head_dim, cfg.sliding_window
    per_layer = (nq + 2 * nkv) * d * H + H * nq * d + 3 * I * H
    weight_bytes = 2 * (L * per_layer + V * H)          # every matrix once; one embedding row is noise
    kv_per_token = 2 * nkv * d * 2 * L                  # K and V, bf16, all layers
    sampler = Sampler(SamplingConfig.greedy(), dev)
    gen = torch.Generator().manual_seed(11)

    def run_decode(batch: int, context: int, steps: int, warmup: int, engine=None, then=None):
        """Prefill `batch` prompts of `context - steps - warmup` tokens, then time `steps` decode
        steps (model step + greedy sampling).  `then(engine, slots)`: called after the timed steps
        while the sequences are still held."""
        held = min(context, W) if W else context
        eng = engine or Engine(model, max_tokens=batch * (round_up(held) + PAGE), max_slots=batch, freeze_gc=True)
        plen = max(1, context - steps - warmup - 1)
        slots = [eng.alloc() for _ in range(batch)]
        chunk = 2048
        for s in slots:                                  # prompt by prompt, in chunks
            ids = torch.randint(0, V, (plen,), generator=gen).tolist()
            for c0 in range(0, plen, chunk):
                part = ids[c0:c0 + chunk]
                last = c0 + chunk >= plen
                lg = eng.step([SeqInput(s, part, [len(part) - 1] if last else [])])
        # every sequence goes on with the same first token; from here the steps are the generation
        # loop's own (`BatchRun.advance`: the next step is launched with the drawn tokens still on
        # the device, then the host reads the tokens of the step before)
        first = sampler.sample(lg, [0], [0]) * batch
        lg = eng.step([SeqInput(s, [t], [0]) for s, t in zip(slots, first)])
        run = BatchRun(eng, sampler, accept=lambda i, t: False, max_tokens=1 << 30, run_ahead=True)
        run.resume(list(range(batch)), lg, slots=slots)
        for _ in range(warmup):
            run.advance()
        torch.cuda.synchronize()
        t = time.perf_counter()
        for _ in range(steps):
            run.advance()
        torch.cuda.synchronize()
        dt = time.perf_counter() - t
        ctx_mid = plen + warmup + steps // 2
        extra = then(eng, [run.slots[i] for i in range(batch)]) if then is not None else None
        run.release()
        if engine is None:
            eng.close()
        return (dt / steps, ctx_mid) if then is None else (dt / steps, ctx_mid, extra)

    def kernels_one_by_one(eng, slots):
        """The kernels of one decode step, each kind by itself: one more step is run with every call
        into the kernels' Python face noted (function and arguments, layer after layer), then the calls
        of each kind are captured as a graph of their own (every layer's launch of that kernel, each on
        its own weights and cache, so that nothing is warm that the step would not find warm) and the
        graph is timed with events.  Bytes are what the kernel has to read once: its weight, or the
        keys and values of the live sequences."""
        from torchless_rs_amd.kernels import ops as K
        names = ("embed", "rmsnorm", "add_rmsnorm", "qkv_rope_commit", "rope_commit", "attention", "gemm_bf16_norm",
                 "gemm_bf16", "gemm_mid_bf16", "gemm", "gemm_library", "add_partials", "gather_rows", "silu_mul_pairs")
        real = {n: getattr(K, n) for n in names}
        tape = []
        depth = [0]

        def noted(name):
            def call(*a, **k):
                if depth[0] == 0:               # (a face that calls another face counts once)
                    tape.append((name, a, k))
                depth[0] += 1
                try:
                    return real[name](*a, **k)
                finally:
                    depth[0] -= 1
            return call

        use_graphs, eng.use_graphs = eng.use_graphs, False
        for n in names:
            setattr(K, n, noted(n))
        try:
            ctx, want_rows, n_want = eng.build_context([SeqInput(s, [0], [0]) for s in slots])
            eng.model.forward(ctx, eng.runs, want_rows, n_want)
        finally:
            for n, f in real.items():
                setattr(K, n, f)
            eng.use_graphs = use_graphs
        torch.cuda.synchronize()
        held_rows = sum(min(int(n), W) if W else int(n) for n in ctx.host["len_after"])

        def kind_and_bytes(name, a, k):
            if name == "attention":
                return "attention", held_rows * 2 * nkv * d * 2
            w = next((t for t in a[:3] if isinstance(t, torch.Tensor) and t.dim() == 2 and t.dtype == torch.bfloat16
                      and t.shape[0] > 64), None)
            if name in ("qkv_rope_commit", "gemm_bf16_norm", "gemm_bf16", "gemm_mid_bf16", "gemm", "gemm_library") and w is not None:
                label = {(nq + 2 * nkv) * d: "qkv", 2 * I: "gate_up", V: "head"}.get(w.shape[0])
                if label is None:
                    label = "o" if w.shape[1] == nq * d else "down"
                if name == "qkv_rope_commit":
                    label = "qkv_rope_commit"
                return label, w.numel() * 2
            return name, 0

        kinds = {}
        for name, a, k in tape:
            kind, nbytes = kind_and_bytes(name, a, k)
            kinds.setdefault(kind, {"calls": [], "bytes": 0})
            kinds[kind]["calls"].append((real[name], a, k))
            kinds[kind]["bytes"] += nbytes
        out, total = {}, 0.0
        side = torch.cuda.Stream()
        for kind, rec in kinds.items():
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph, stream=side):
                for f, a, k in rec["calls"]:
                    f(*a, **k)
            torch.cuda.synchronize()
            best = float("inf")
            for _ in range(5):
                e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
                e0.record()
                graph.replay()
                e1.record()
                e1.synchronize()
                best = min(best, e0.elapsed_time(e1) * 1e3)
            n = len(rec["calls"])
            out[f"{kind}_us"] = round(best / n, 2)
            out[f"{kind}_calls"] = n
            if rec["bytes"]:
                out[f"{kind}_frac"] = round(rec["bytes"] / (best * 1e-6) / 1e9 / HBM_PEAK_GBS, 4)
            total += best
            del graph
        out["sum_us"] = round(total, 1)
        return out

    def run_workload(mdl, mcfg, n_layers, batch, lo, hi, new_tokens, temperature, seed):
        """`batch` requests with prompt lengths uniform in [lo, hi] and `new_tokens` new tokens each,
        through `generate_until_eos` as a user would call it: prompts in one step, then one token a
        step.  The prefill ends and decoding begins when the host holds the first token."""
        from torchless_rs_amd import generate_until_eos
        g = torch.Generator().manual_seed(seed)
        lens = torch.randint(lo, hi + 1, (batch,), generator=g).tolist()
        prompts = [torch.randint(0, mcfg.vocab_size, (n,), generator=g).tolist() for n in lens]
        win = mcfg.sliding_window
        held = [min(n + new_tokens, win) if win else n + new_tokens for n in lens]
        eng = Engine(mdl, max_tokens=sum(round_up(h) + PAGE for h in held), max_slots=batch, freeze_gc=True)
        scfg = SamplingConfig(temperature=temperature, seed=seed) if temperature > 0 else SamplingConfig.greedy()
        stamps = []

        def on_token(i, t):
            if not stamps:
                torch.cuda.synchronize()
                stamps.append(time.perf_counter())

        torch.cuda.synchronize()
        t0 = time.perf_counter()
        out = generate_until_eos(eng, prompts, scfg, max_tokens=new_tokens, on_token=on_token)
        torch.cuda.synchronize()
        t2 = time.perf_counter()
        eng.close()
        assert all(len(r.tokens) == new_tokens for r in out)
        t_pre, t_dec = stamps[0] - t0, t2 - stamps[0]
        per_l = ((mcfg.num_attention_heads + 2 * mcfg.num_key_value_heads) * mcfg.head_dim * mcfg.hidden_size
                 + mcfg.hidden_size * mcfg.num_attention_heads * mcfg.head_dim
                 + 3 * mcfg.intermediate_size * mcfg.hidden_size)
        w_bytes = 2 * (n_layers * per_l + mcfg.vocab_size * mcfg.hidden_size)
        kv_tok = 2 * mcfg.num_key_value_heads * mcfg.head_dim * 2 * n_layers
        steps = new_tokens - 1                           # the first token comes out of the prompts' step
        ctx = [n + new_tokens / 2 for n in lens]
        step_bytes = w_bytes + sum((min(c, win) if win else c) for c in ctx) * kv_tok
        gbs = step_bytes * steps / t_dec / 1e9
        return {"batch": batch, "prompt_tokens": sum(lens), "new_tokens": new_tokens, "temperature": temperature,
                "prefill_tok_s": round(sum(lens) / t_pre, 1), "prefill_ms": round(t_pre * 1e3, 1),
                "decode_tok_s": round(batch * steps / t_dec, 1), "decode_ms_per_step": round(t_dec / steps * 1e3, 3),
                "roofline_frac": round(gbs / HBM_PEAK_GBS, 4), "achieved_GBs": round(gbs, 1)}

    if args.only == "decode":
        sec, _ = run_decode(args.batch, args.context, args.steps, args.warmup)
        print(f"[bench] decode b{args.batch}: {args.batch / sec:.1f} tok/s, {sec * 1e3:.3f} ms/step",
              file=sys.stderr, flush=True)
        return 0

    # prefill of one prompt
    T = args.prefill_tokens
    eng = Engine(model, max_tokens=T + PAGE, max_slots=1, freeze_gc=True)
    ids = torch.randint(0, V, (T,), generator=gen).tolist()
    pre_ms = []
    for it in range(2):
        s = eng.alloc()
        torch.cuda.synchronize()
        t = time.perf_counter()
        eng.step([SeqInput(s, ids, [T - 1])])
        torch.cuda.synchronize()
        pre_ms.append((time.perf_counter() - t) * 1e3)
        eng.free(s)
    eng.close()
    pre = min(pre_ms)
    attn_flops = sum(4 * nq * d * min(p + 1, W or (p + 1)) for p in range(T)) * L
    pre_flops = 2 * T * (L * per_layer) + 2 * V * H + attn_flops
    prefill = {"value": round(T / (pre / 1e3), 1), "tokens": T, "ms": round(pre, 3),
               "frac": round(pre_flops / (pre / 1e3) / (PEAK_TFLOPS["bf16"] * 1e12), 4)}
    print(f"[bench] prefill {prefill}", file=sys.stderr, flush=True)
    if args.only == "prefill":
        return 0

    if args.no_kernels:
        (sec, ctx_mid), kernels = run_decode(args.batch, args.context, args.steps, args.warmup), {}
    else:
        sec, ctx_mid, kernels = run_decode(args.batch, args.context, args.steps, args.warmup, then=kernels_one_by_one)
        kernels["step_us"] = round(sec * 1e6, 1)
        print(f"[bench] kernels of the step one by one {kernels}", file=sys.stderr, flush=True)
    held = min(ctx_mid, W) if W else ctx_mid
    step_bytes = weight_bytes + args.batch * held * kv_per_token
    achieved = step_bytes / sec / 1e9
    value = args.batch / sec
    print(f"[bench] decode b{args.batch}: {value:.1f} tok/s, {sec * 1e3:.3f} ms/step", file=sys.stderr,
          flush=True)
    points = {}
    if not args.no_points:
        for b in (1, 64):
            s_b, _ = run_decode(b, args.context, max(32, args.steps), 4)
            points[f"decode_b{b}"] = round(b / s_b, 1)
            print(f"[bench] decode b{b}: {b / s_b:.1f} tok/s", file=sys.stderr, flush=True)

    workloads = {}
    if args.workload == "baseline" and not args.no_workloads:
        if args.shape == "7b-v0.1":                     # the model that is loaded: prompts U[128, 2048], 256 new tokens
            for b in (1, 8, 64):
                workloads[f"7b-v0.1_b{b}"] = run_workload(model, cfg, L, b, 128, 2048, 256, 0.0, seed=5)
                print(f"[bench] workload 7b-v0.1 b{b}: {workloads[f'7b-v0.1_b{b}']}", file=sys.stderr, flush=True)
        del model
        torch.cuda.empty_cache()
        for key, b, lo, hi, new, temp, seed in (("7b-v0.3", 8, 1024, 16384, 128, 0.0, 6),
                                                ("nemo-12b", 16, 256, 8192, 128, 0.7, 7)):
            wcfg = config_from_dict(dict(SHAPES[key][1], architectures=["MistralForCausalLM"]))
            wt = random_tensors(model_spec_for(wcfg).weight_specs(), seed=seed, std=0.02, dtype=torch.bfloat16, device=dev)
            wm = model_from_tensors(wcfg, wt, "bfloat16", dev, tiled_copies=not args.no_tiled_copies)
            del wt
            workloads[f"{key}_b{b}"] = run_workload(wm, wcfg, wcfg.num_hidden_layers, b, lo, hi, new, temp, seed)
            print(f"[bench] workload {key} b{b}: {workloads[f'{key}_b{b}']}", file=sys.stderr, flush=True)
            del wm
            torch.cuda.empty_cache()
        model = None

    # what the simplest kernels get here: a plain read of 8 GiB, independent MFMAs on registers
    from torchless_rs_amd.kernels import ops as _ops
    del model
    torch.cuda.empty_cache()
    ceilings = _ops.measure_ceilings(dev)
    print(f"[bench] measured ceilings {ceilings}", file=sys.stderr, flush=True)
    ceilings["decode_frac_of_read"] = round(achieved / ceilings["hbm_read_GBs"], 4)
    ceilings["prefill_frac_of_mfma"] = round(pre_flops / (pre / 1e3) / (ceilings["mfma_bf16_TFLOPs"] * 1e12), 4)
    out = {
        "metric": f"decode tok/s at batch {args.batch} ({shape_name}), with prefill tok/s at "
                  f"{args.prefill_tokens:,} tokens",
        "value": round(value, 1), "unit": "tokens/s", "n_gpus": 1, "steps": args.steps,
        "warmup": args.warmup, "ms_per_step": round(sec * 1e3, 4), "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16",
        "data": "synthetic: random weights N(0,0.02) seed 5, uniform random token ids",
        "config": {"model": shape_name, "layers": L, "layers_of_config": shape["num_hidden_layers"],
                   "hidden_size": H, "heads": nq, "kv_heads": nkv, "head_dim": d,
                   "intermediate_size": I, "vocab_size": V, "sliding_window": W,
                   "rope_theta": cfg.rope_theta, "rms_norm_eps": cfg.rms_norm_eps,
                   "global_batch": args.batch, "seq_len": args.context, "parallelism": "none",
                   "sampling": "greedy", "tiled_weight_copies": not args.no_tiled_copies,
                   "weights_resident_gib": resident_gib},
        "prefill": prefill,
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBS,
                     "unit": "GB/s", "frac": round(achieved / HBM_PEAK_GBS, 4)},
        "points": points,
        "ceilings": ceilings,
    }
    if kernels:
        out["kernels"] = kernels
    if workloads:
        # flat: decoded and prefilled tokens a second and the decode steps' share of the HBM roofline
        out["workloads"] = {f"{k}_{f}": v[f] for k, v in workloads.items()
                            for f in ("decode_tok_s", "prefill_tok_s", "roofline_frac")}
        out["workload_details"] = workloads
    print(json.dumps(out), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
