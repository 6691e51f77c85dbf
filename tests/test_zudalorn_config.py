"""Zudalorn's configuration and model spec (no GPU): every key read, what is refused, which parts
and which cache a layer asks for, the stretched frequencies.  The builders below are shared with the
GPU tests."""
import copy
import math

import pytest
import torch

import plain_zudalorn as plain
from torchless_rs_amd.config.base import ConfigError, config_from_dict
from torchless_rs_amd.models import model_spec_for


def latent(heads, dim, rot_dim, vdim, rank, scale, window=None, base=10000.0, scaling=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if window:
        m["mask"] = {"size": window}
    return "latent_attention", m


def ret(heads, dim, vdim, decay, rot=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    return "retention", m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, groups=None, shared=None):
    m = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if groups:
        m["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def model(vocab, width, eps, layers):
    return {"architecture": "Zudalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# both mixers and both feed-forwards, windows below and above a page, a layer without a feed-forward, values wider and
# narrower than keys, a rotation of part of a retention head, plain and stretched frequencies
MIXED = model(200, 96, 1e-5, [
    layer(ret(3, 32, 48, [0.9, 0.99, 0.999], rot=(10000.0, 16)), moe(8, 2, 32, groups=(4, 2), shared=48)),
    layer(latent(4, 24, 8, 16, 64, 0.2, window=70, scaling=(4.0, 256.0, 32.0, 1.0)), dense(160)),
    layer(ret(2, 64, 64, [0.96875, 0.5], rot=(500.0, 64))),
    layer(latent(3, 16, 16, 32, 40, 0.25, window=33, base=300.0, scaling=(16.0, 64.0, 8.0, 2.0)), moe(6, 3, 16, shared=32)),
    layer(latent(2, 32, 16, 32, 32, 0.18), dense(96)),
])


def test_every_key_is_read_and_written_back():
    cfg = config_from_dict(copy.deepcopy(MIXED))
    assert cfg.architecture == "Zudalorn" and cfg.vocab_size == 200 and cfg.hidden_size == 96 and cfg.norm_eps == 1e-5
    r, a = cfg.layers[0].mixer, cfg.layers[1].mixer
    assert (r.heads, r.dim, r.vdim, r.decay, r.rot_base, r.rot_dims) == (3, 32, 48, [0.9, 0.99, 0.999], 10000.0, 16)
    assert (a.heads, a.dim, a.rot_dim, a.vdim, a.kv_rank, a.scale, a.rot_base, a.window) == (4, 24, 8, 16, 64, 0.2, 10000.0, 70)
    assert (a.scaling.factor, a.scaling.original, a.scaling.fast, a.scaling.slow) == (4.0, 256.0, 32.0, 1.0)
    assert cfg.layers[4].mixer.window is None and cfg.layers[4].mixer.scaling is None and cfg.layers[2].mlp is None
    f = cfg.layers[0].mlp
    assert (f.experts, f.top, f.ff, f.groups, f.keep, f.shared_ff) == (8, 2, 32, 4, 2, 48)
    assert cfg.layers[3].mlp.groups is None and cfg.layers[1].mlp.ff == 160
    assert cfg.to_dict() == MIXED and config_from_dict(cfg.to_dict()).to_dict() == MIXED


@pytest.mark.parametrize("change, text", [
    (lambda d: d["layers"][0]["mixer"]["decay"].pop(), "decay"),
    (lambda d: d["layers"][0]["mixer"]["decay"].__setitem__(0, -0.5), "decay"),
    (lambda d: d["layers"][0]["mixer"].update(dim=600), "not served"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=34), "rotated"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=5), "rotated"),
    (lambda d: d["layers"][1]["mixer"].update(rot_dim=10), "rot_dim"),
    (lambda d: d["layers"][1]["mixer"].pop("rot"), "rot_dim"),
    (lambda d: d["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda d: d["layers"][1]["mixer"].update(dim=300), "not served"),
    (lambda d: d["layers"][1]["mixer"].update(kv_rank=2000), "not served"),
    (lambda d: d["layers"][1]["mixer"]["mask"].update(size=0), ">= 1"),
    (lambda d: d["layers"][1]["mixer"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda d: d["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0), "factor"),
    (lambda d: d["layers"][1].update(type="attention"), "no mixer"),
    (lambda d: d["layers"][1]["mlp"].update(kind="gated"), "no feed-forward"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=9), "experts"),
    (lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(count=3), "groups"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=5), "groups"),
    (lambda d: d["layers"][0]["mlp"].pop("expert"), "expert"),
    (lambda d: d.pop("norm"), "norm"),
    (lambda d: d.update(layers=[]), "layers"),
])
def test_what_is_refused(change, text):
    d = copy.deepcopy(MIXED)
    change(d)
    with pytest.raises(ConfigError) as e:
        config_from_dict(d)
    assert text in str(e.value), str(e.value)


def test_the_spec_names_every_tensor_and_part():
    cfg = config_from_dict(copy.deepcopy(MIXED))
    spec = model_spec_for(cfg)
    got = {k: tuple(v.shape) for k, v in spec.weight_specs().items()}
    assert got == {k: tuple(v) for k, v in plain.tensor_shapes(MIXED).items()}
    assert [l.mixer.kind for l in spec.layers] == ["retention", "latent_cache_attention", "retention"] + ["latent_cache_attention"] * 2
    assert [l.ffn.kind if l.ffn else None for l in spec.layers] == ["routed_experts", "plain", None, "routed_experts", "plain"]
    assert all(l.block.kind == "sandwich_norm" and l.mixer_norm.params["scalar"] for l in spec.layers)
    p = spec.layers[1].mixer.params["position"].params
    assert p["interleaved"] and p["rotary_dim"] == 8 and p["scaling"]["original"] == 256.0
    assert not spec.layers[0].mixer.params["position"].params["interleaved"]
    f = spec.layers[0].ffn.params
    assert f["correction"] and f["group_score"] == "two_largest" and f["normalise_eps"] == 1e-20 and f["shared_gated"]


def test_the_cache_that_the_layers_ask_for():
    """A latent layer keeps a latent and a rotated part a position, in a ring of its window's pages; retention one float32
    state a head and sequence."""
    from torchless_rs_amd.engine.model import Model
    cfg = config_from_dict(copy.deepcopy(MIXED))
    kv, st = Model(model_spec_for(cfg), cfg, torch.bfloat16, "cpu").cache_requests()
    assert sorted(kv) == [1, 3, 4] and sorted(st) == [0, 2]
    assert [(kv[i].n_kv_heads, kv[i].head_dim, kv[i].value_dim, kv[i].window) for i in (1, 3, 4)] == \
        [(1, 72, 0, 70), (1, 56, 0, 33), (1, 48, 0, None)]
    assert st[0].shape == (3 * 32 * 48,) and st[2].shape == (2 * 64 * 64,) and st[0].dtype == torch.float32


@pytest.mark.parametrize("base, dims, scaling", [
    (10000.0, 64, (4.0, 4096.0, 32.0, 1.0)), (20000.0, 8, (16.0, 64.0, 8.0, 2.0)), (500.0, 2, (2.0, 100.0, 1.0, 1.0)),
    (1e6, 128, (32.0, 8192.0, 32.0, 1.0)), (300.0, 16, (1.0, 10.0, 4.0, 0.5)), (10000.0, 32, (8.0, 2.0, 32.0, 1.0))])
def test_stretched_frequencies(base, dims, scaling):
    """Quick pairs as they were, slow ones divided, a ramp between (steep where both ends fall on one pair); the factor on
    cosines and sines."""
    from torchless_rs_amd.parts.position import Rotary
    sc = dict(zip(("factor", "original", "fast", "slow"), scaling))
    part = Rotary(dims, base, dims, True, scaling=sc)
    f, mag = plain.frequencies({"base": base, "dims": dims, "scaling": sc})
    assert torch.allclose(part.inv_freq_host().double(), f, rtol=2e-7, atol=0)
    assert math.isclose(part.magnitude, mag, rel_tol=1e-12) and part.rotation("cpu").magnitude == part.magnitude
    bare, one = plain.frequencies({"base": base, "dims": dims})
    assert one == 1.0 and torch.allclose(Rotary(dims, base, dims).inv_freq_host().double(), bare, rtol=2e-7, atol=0)
    assert ((f <= bare * (1 + 1e-12)) & (f >= bare / sc["factor"] * (1 - 1e-12))).all()


def test_a_ramp_has_pairs_on_both_sides_and_between():
    f, _ = plain.frequencies({"base": 10000.0, "dims": 64, "scaling": dict(factor=4.0, original=4096.0, fast=32.0, slow=1.0)})
    bare, _ = plain.frequencies({"base": 10000.0, "dims": 64})
    ratio = f / bare
    assert ratio[0] == 1.0 and math.isclose(ratio[-1], 0.25) and ((ratio > 0.26) & (ratio < 0.99)).any()


def test_kernels_without_a_factor_on_the_rotation_refuse_one():
    from torchless_rs_amd.kernels import ops
    rot = ops.Rotation(torch.ones(4), 8, False, 1.2)
    with pytest.raises(ops.KernelError):
        ops._rotation(rot, 16, "a kernel")


@pytest.mark.parametrize("bad", [dict(factor=2.0), dict(factor=2.0, original=10.0, fast=-1.0, slow=1.0)])
def test_a_scaling_that_is_no_scaling(bad):
    from torchless_rs_amd.parts.position import Rotary
    with pytest.raises(ValueError):
        Rotary(8, 100.0, scaling=bad)


def test_parts_that_are_refused():
    from torchless_rs_amd.parts.attention_latent_cache import LatentCacheAttentionMixer
    from torchless_rs_amd.parts.ffn_routed import RoutedExperts
    from torchless_rs_amd.parts.retention import RetentionMixer
    with pytest.raises(ValueError):
        RetentionMixer(8, 2, 4, [0.5], 1e-5)
    with pytest.raises(ValueError):
        LatentCacheAttentionMixer(8, 2, 4, 4, 16, 0.5, 1e-5, rot_dim=3)
    with pytest.raises(ValueError):
        RoutedExperts(8, 4, 2, 4, gated=True, activation="silu", activation_constants={"limit": 1.0})
    with pytest.raises(ValueError):
        RoutedExperts(8, 4, 2, 4, group_score="mean")
    with pytest.raises(ValueError):
        RoutedExperts(8, 4, 2, 4, activation="xielu")


def test_retention_written_as_a_sum_over_all_rows():
    """The plain recurrence against its closed form, sum_j decay^(i-j) (k_j . q_i) v_j."""
    g = torch.Generator().manual_seed(0)
    T, H, d, dv = 9, 2, 3, 4
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=torch.float64) for n in (d, d, dv))
    decay = torch.tensor([0.9, 0.0], dtype=torch.float64)
    o, _ = plain.retention_heads(q, k, v, decay)
    i = torch.arange(T)
    for h in range(H):
        D = torch.where(i[:, None] >= i[None], decay[h] ** (i[:, None] - i[None]).clamp(min=0), torch.zeros(()).double())
        assert torch.allclose(o[:, h], ((q[:, h] @ k[:, h].T) * D) @ v[:, h])
