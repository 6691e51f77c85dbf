"""Zudalorn as a list of parts.

A decoder-only model whose layers norm a sublayer on both sides, every norm a root mean square
with one number for all channels, x += g1b rms(mixer(g1 rms(x))); x += g2b rms(ffn(g2 rms(x)))
(`sandwich_norm` of `rmsnorm` with `scalar`, the feed-forward optional).  The mixer is, layer by
layer as config.json lists them, one of

* `latent_attention`: attention whose cache keeps a latent and one rotated key part per position
  (`latent_cache_attention`), its rotation stretched for long contexts, with a sliding window;
* `retention`: linear attention with a fixed decay per head and a state per sequence (`retention`).

The feed-forward is one layer with the xIELU activation (`plain`) or a routed mixture of small gated
experts, chosen by groups with a correction on the scores, with a shared expert behind a gate
(`routed_experts` with those terms).  Tensor names: `embed`, `l<i>.norm1` .. `l<i>.norm2b`,
`l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`, `head`.  Every size comes from the configuration, layer by
layer.
"""
from __future__ import annotations

from ..config.base import register_architecture
from ..config.zudalorn import NAME, ZudalornAttention, ZudalornConfig, ZudalornDense
from ..parts.base import LayerSpec, ModelSpec, PartSpec, Run

# what keeps the sum of the chosen experts' scores from being zero
ROUTER_SUM_EPS = 1e-20


def _rotary(head_dim, base, dims, scaling, interleaved) -> PartSpec:
    if not dims or base is None:
        return PartSpec("none")
    return PartSpec("rotary", {"head_dim": head_dim, "theta": base, "rotary_dim": dims, "interleaved": interleaved,
                               "scaling": None if scaling is None else scaling.to_dict()})


def zudalorn_spec(cfg: ZudalornConfig) -> ModelSpec:
    H = cfg.hidden_size
    norm = PartSpec("rmsnorm", {"size": H, "eps": cfg.norm_eps, "name": "", "scalar": True})
    layers = []
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        if isinstance(m, ZudalornAttention):
            mixer = PartSpec("latent_cache_attention", {
                "hidden_size": H, "n_heads": m.heads, "head_dim": m.dim, "rot_dim": m.rot_dim, "v_head_dim": m.vdim,
                "kv_rank": m.kv_rank, "scale": m.scale, "norm_eps": cfg.norm_eps, "window": m.window,
                "position": _rotary(m.rot_dim, m.rot_base, m.rot_dim, m.scaling, True), "prefix": "mix."})
        else:
            mixer = PartSpec("retention", {
                "hidden_size": H, "n_heads": m.heads, "head_dim": m.dim, "v_head_dim": m.vdim, "decay": m.decay,
                "norm_eps": cfg.norm_eps, "position": _rotary(m.dim, m.rot_base, m.rot_dims, m.scaling, False),
                "prefix": "mix."})
        ffn = None
        f = layer.mlp
        if isinstance(f, ZudalornDense):
            ffn = PartSpec("plain", {"hidden_size": H, "intermediate_size": f.ff, "activation": "xielu", "prefix": "mlp."})
        elif f is not None:
            ffn = PartSpec("routed_experts", {
                "hidden_size": H, "n_experts": f.experts, "top": f.top, "expert_size": f.ff, "group_count": f.groups,
                "group_keep": f.keep, "group_score": "two_largest", "shared_size": f.shared_ff, "score": "sigmoid",
                "correction": True, "normalise_eps": ROUTER_SUM_EPS, "gated": True, "activation": "silu",
                "shared_gated": True, "prefix": "mlp."})
        layers.append(LayerSpec(prefix=f"l{i}.", mixer=mixer, ffn=ffn, mixer_norm=norm,
                                ffn_norm=norm if ffn is not None else None, mixer_out_norm=norm,
                                ffn_out_norm=norm if ffn is not None else None,
                                block=PartSpec("sandwich_norm", {"names": ("norm1", "norm1b", "norm2", "norm2b")})))
    return ModelSpec(
        hidden_size=H, vocab_size=cfg.vocab_size,
        embedding=PartSpec("tokens", {"vocab_size": cfg.vocab_size, "hidden_size": H, "name": "embed"}),
        embedding_prefix="",
        layers=layers, schedule=[Run(i) for i in range(len(layers))],
        final_norm=norm, final_norm_prefix="final.norm",
        head=PartSpec("linear", {"vocab_size": cfg.vocab_size, "hidden_size": H, "name": "head"}),
        head_prefix="",
    )


register_architecture(NAME, ZudalornConfig, zudalorn_spec)
