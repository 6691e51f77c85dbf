"""Zifetar as a list of parts.

A decoder-only model whose embedding is a token's row times a factor plus a row that the pair of the
previous and the present token picks, normed (`token_pairs`), and whose layers norm a sublayer on both
sides, x += N1b(mixer(N1(x))); x += N2b(ffn(N2(x))), every norm a root mean square whose weight is stored as
its difference from one (`sandwich_norm` of `rmsnorm` with `around_zero`, the feed-forward optional).
The mixer is, layer by layer as config.json lists them, one of

* `channel_delta`: a delta rule with a decay per head and key channel behind short convolutions, its read-out
  normed per head and gated (`channel_linear` with those terms);
* `retention`: linear attention with a fixed decay per head (`retention`);
* `parallel`: attention in chunks of positions (`headwise_attention`: biases, a norm of q and k per head, a
  rotation stretched by wavelength) beside a linear attention with a decay per key channel (`channel_linear`),
  each with a factor (`parallel`).

The feed-forward is a routed mixture of gated experts weighted by a softmax over the chosen ones' logits
(`routed_experts` with those terms).  Tensor names: `embed`, `bigram`, `embed.norm`, `l<i>.norm1` ..
`l<i>.norm2b`, `l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`, `head`.  Every size comes from the configuration,
layer by layer, or, for the inner sizes of two-step projections, from the tensors.
"""
from __future__ import annotations

from ..config.base import register_architecture
from ..config.zifetar import NAME, ZifetarConfig, ZifetarDelta, ZifetarRetention
from ..parts.base import LayerSpec, ModelSpec, PartSpec, Run

UNIT_EPS = 1e-6          # beside the sum of squares of a head of q or k that is made a unit vector


def _rotary(rot, dim) -> PartSpec:
    if rot is None or not rot.dims:
        return PartSpec("none")
    return PartSpec("rotary", {"head_dim": dim, "theta": rot.base, "rotary_dim": rot.dims, "scaling": rot.scaling})


def zifetar_spec(cfg: ZifetarConfig) -> ModelSpec:
    H, eps = cfg.hidden_size, cfg.norm_eps
    norm = PartSpec("rmsnorm", {"size": H, "eps": eps, "name": "", "around_zero": True})
    layers = []
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        if isinstance(m, ZifetarDelta):
            mixer = PartSpec("channel_linear", {
                "hidden_size": H, "n_heads": m.heads, "n_kv_heads": m.kv_heads, "head_dim": m.dim, "v_head_dim": m.vdim,
                "norm_eps": eps, "conv_taps": m.conv, "unit_eps": UNIT_EPS, "decay": "softplus", "delta": True,
                "gate": "logistic", "inner": m.dim, "prefix": "mix."})
        elif isinstance(m, ZifetarRetention):
            mixer = PartSpec("retention", {
                "hidden_size": H, "n_heads": m.heads, "head_dim": m.dim, "v_head_dim": m.vdim, "decay": m.decay,
                "norm_eps": eps, "position": _rotary(m.rot, m.dim), "prefix": "mix."})
        else:
            a, b = m.left, m.right
            left = PartSpec("headwise_attention", {
                "hidden_size": H, "n_heads": a.heads, "n_kv_heads": a.kv_heads, "head_dim": a.dim, "v_head_dim": a.vdim,
                "position": _rotary(a.rot, a.dim), "scale": a.scale, "bias": True, "o_bias": False, "head_norm_eps": eps,
                "chunk": a.chunk, "prefix": "mix.left."})
            right = PartSpec("channel_linear", {
                "hidden_size": H, "n_heads": b.heads, "head_dim": b.dim, "v_head_dim": b.vdim, "norm_eps": eps,
                "decay": "logistic", "tau": b.tau, "gate": "silu", "names": {"decay_bias": "a2.b"}, "prefix": "mix.right."})
            mixer = PartSpec("parallel", {"left": left, "right": right, "left_scale": m.left_scale, "right_scale": m.right_scale})
        ffn = None
        f = layer.mlp
        if f is not None:
            # a softmax over all experts divided by the chosen ones' share is the softmax over the chosen ones
            ffn = PartSpec("routed_experts", {
                "hidden_size": H, "n_experts": f.experts, "top": f.top, "expert_size": f.ff, "score": "softmax",
                "normalise_eps": 0.0, "router_bias": True, "gated": True, "activation": "silu", "prefix": "mlp."})
        layers.append(LayerSpec(prefix=f"l{i}.", mixer=mixer, ffn=ffn, mixer_norm=norm,
                                ffn_norm=norm if ffn is not None else None, mixer_out_norm=norm,
                                ffn_out_norm=norm if ffn is not None else None,
                                block=PartSpec("sandwich_norm", {"names": ("norm1", "norm1b", "norm2", "norm2b")})))
    table = {"vocab_size": cfg.vocab_size, "hidden_size": H, "name": "embed", "scale": cfg.embedding_scale, "norm": norm,
             "norm_prefix": "embed.norm"}
    pairs = cfg.bigram
    if pairs is not None:
        table.update(buckets=pairs.buckets, mul_prev=pairs.mul_prev, mul_cur=pairs.mul_cur, pair_name="bigram")
    return ModelSpec(
        hidden_size=H, vocab_size=cfg.vocab_size, embedding=PartSpec("token_pairs", table), embedding_prefix="",
        layers=layers, schedule=[Run(i) for i in range(len(layers))],
        final_norm=norm, final_norm_prefix="final.norm",
        head=PartSpec("linear", {"vocab_size": cfg.vocab_size, "hidden_size": H, "name": "head"}),
        head_prefix="",
    )


register_architecture(NAME, ZifetarConfig, zifetar_spec)
