"""`ZifetarConfig`: the config.json of a Zifetar model, typed.

The file names its design in `architecture`, the sizes `vocab` and `width`, `norm.eps`, `embedding` =
{`scale`, `bigram`} and `layers`, a list with one entry per layer.  `bigram` = {`buckets`, `mul_prev`,
`mul_cur`} (absent: no table of token pairs).  A layer's entry has `type` (which mixer), `mixer` (its sizes
and constants) and `mlp` (the feed-forward, or null for a layer without one); every entry is read on
its own, so layers may differ in every size.

Mixer `channel_delta`: `heads`, `kv_heads` (heads of q and k), `dim`, `vdim`, `conv` (taps of the short convolution).
Mixer `retention`: `heads`, `dim`, `vdim`, `decay` (a number per head), `rot` (absent: no rotation).
Mixer `parallel`: `left_scale`, `right_scale`, `left` = {`heads`, `kv_heads`, `dim`, `vdim`, `scale` (the factor on
a score), `rot`, `mask.size` (the chunk; absent: every earlier position is seen)} and `right` = {`heads`, `dim`,
`vdim`, `tau`}.
`rot` = {`base`, `dims`, `scaling`}, `scaling` = {`factor`, `low`, `high`, `original`} (absent: plain frequencies).
Feed-forward `moe`: `router` = {`experts`, `top`}, `expert.ff`.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Union

from .base import ConfigError, ModelConfig, take_float, take_int, take_obj

MAX_HEAD_DIM = 256          # the largest head the attention kernels and the delta rule's take
MAX_RETENTION_DIM = 512     # the largest key size of a retention head
MAX_TAPS = 8                # the longest short convolution
MAX_EXPERTS = 1024
NAME = "Zifetar"


def _at(where, take, *args, **kw):
    try:
        return take(*args, **kw)
    except ConfigError as e:
        raise ConfigError(f"{e} (in {where})") from None


def _sizes(m: Dict[str, Any], names, where: str) -> Dict[str, int]:
    return {k: _at(where, take_int, m, k, required=True, minimum=1) for k in names}


def _heads(n: Dict[str, int], where: str, most: int = MAX_HEAD_DIM) -> Dict[str, int]:
    if n["dim"] > most or n["vdim"] > MAX_HEAD_DIM:
        raise ConfigError(f"config.json: {where}: heads of {n['dim']} and {n['vdim']} are not served (up to {most} and {MAX_HEAD_DIM})")
    if "kv_heads" in n and n["heads"] % n["kv_heads"]:
        raise ConfigError(f"config.json: {where}: {n['heads']} heads are not a multiple of {n['kv_heads']}")
    return n


@dataclass
class ZifetarRotation:
    base: float
    dims: int
    scaling: Optional[Dict[str, float]] = None

    @classmethod
    def from_mixer(cls, m: Dict[str, Any], dim: int, where: str) -> Optional["ZifetarRotation"]:
        rot = take_obj(m, "rot", where)
        if rot is None:
            return None
        dims = _at(where, take_int, rot, "dims", default=dim, minimum=0)
        if dims % 2 or dims > dim:
            raise ConfigError(f"config.json: {where}: {dims} rotated channels of {dim} (even, at most as many)")
        sc = take_obj(rot, "scaling", where)
        if sc is not None:
            sc = {k: _at(where, take_float, sc, k, required=True, positive=True) for k in ("factor", "low", "high", "original")}
            if sc["high"] < sc["low"]:
                raise ConfigError(f"config.json: {where}: rot.scaling: high {sc['high']} is below low {sc['low']}")
        return cls(_at(where, take_float, rot, "base", required=True, positive=True), dims, sc)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            d["scaling"] = dict(self.scaling)
        return d


@dataclass
class ZifetarDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZifetarDelta":
        n = _heads(_sizes(m, ("heads", "kv_heads", "dim", "vdim", "conv"), where), where)
        if n["conv"] > MAX_TAPS:
            raise ConfigError(f"config.json: {where}: a convolution of {n['conv']} taps is not served (up to {MAX_TAPS})")
        return cls(**n)

    def to_dict(self) -> Dict[str, Any]:
        return {k: getattr(self, k) for k in ("heads", "kv_heads", "dim", "vdim", "conv")}


@dataclass
class ZifetarRetention:
    heads: int
    dim: int
    vdim: int
    decay: List[float]
    rot: Optional[ZifetarRotation] = None

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZifetarRetention":
        n = _heads(_sizes(m, ("heads", "dim", "vdim"), where), where, MAX_RETENTION_DIM)
        decay = m.get("decay")
        if (not isinstance(decay, list) or len(decay) != n["heads"]
                or any(isinstance(a, bool) or not isinstance(a, (int, float)) or not 0 <= a for a in decay)):
            raise ConfigError(f"config.json: {where}: 'decay' must list {n['heads']} numbers, none below 0")
        return cls(decay=[float(a) for a in decay], rot=ZifetarRotation.from_mixer(m, n["dim"], where), **n)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass
class ZifetarAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[ZifetarRotation] = None
    chunk: Optional[int] = None

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZifetarAttention":
        n = _heads(_sizes(m, ("heads", "kv_heads", "dim", "vdim"), where), where)
        mask = take_obj(m, "mask", where)
        return cls(scale=_at(where, take_float, m, "scale", required=True), rot=ZifetarRotation.from_mixer(m, n["dim"], where),
                   chunk=None if mask is None else _at(where, take_int, mask, "size", required=True, minimum=1), **n)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        if self.chunk is not None:
            d["mask"] = {"size": self.chunk}
        return d


@dataclass
class ZifetarLinear:
    heads: int
    dim: int
    vdim: int
    tau: float

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZifetarLinear":
        return cls(tau=_at(where, take_float, m, "tau", required=True, positive=True),
                   **_heads(_sizes(m, ("heads", "dim", "vdim"), where), where))

    def to_dict(self) -> Dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}


@dataclass
class ZifetarParallel:
    left: ZifetarAttention
    right: ZifetarLinear
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZifetarParallel":
        return cls(ZifetarAttention.from_dict(take_obj(m, "left", where, required=True), where + ", left"),
                   ZifetarLinear.from_dict(take_obj(m, "right", where, required=True), where + ", right"),
                   *(_at(where, take_float, m, k, required=True) for k in ("left_scale", "right_scale")))

    def to_dict(self) -> Dict[str, Any]:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


@dataclass
class ZifetarExperts:
    experts: int
    top: int
    ff: int

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZifetarExperts":
        router = take_obj(m, "router", where, required=True)
        n = _sizes(router, ("experts", "top"), where)
        if n["experts"] > MAX_EXPERTS or n["top"] > n["experts"]:
            raise ConfigError(f"config.json: {where}: {n['top']} of {n['experts']} experts (at most {MAX_EXPERTS}, top within them)")
        return cls(ff=_at(where, take_int, take_obj(m, "expert", where, required=True), "ff", required=True, minimum=1), **n)

    def to_dict(self) -> Dict[str, Any]:
        return {"kind": "moe", "router": {"experts": self.experts, "top": self.top}, "expert": {"ff": self.ff}}


MIXERS = {"channel_delta": ZifetarDelta, "retention": ZifetarRetention, "parallel": ZifetarParallel}
FEED_FORWARDS = {"moe": ZifetarExperts}


@dataclass
class ZifetarLayer:
    type: str
    mixer: Union[ZifetarDelta, ZifetarRetention, ZifetarParallel]
    mlp: Optional[ZifetarExperts] = None

    def to_dict(self) -> Dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass
class ZifetarBigram:
    buckets: int
    mul_prev: int
    mul_cur: int

    def to_dict(self) -> Dict[str, Any]:
        return {"buckets": self.buckets, "mul_prev": self.mul_prev, "mul_cur": self.mul_cur}


@dataclass
class ZifetarConfig(ModelConfig):
    vocab_size: int = 0
    hidden_size: int = 0
    norm_eps: float = 1e-5
    embedding_scale: float = 1.0
    bigram: Optional[ZifetarBigram] = None
    layers: List[ZifetarLayer] = field(default_factory=list)
    eos_token_ids: List[int] = field(default_factory=list)
    max_position_embeddings: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "ZifetarConfig":
        norm = take_obj(d, "norm", "the model", required=True)
        emb = take_obj(d, "embedding", "the model") or {}
        pair = take_obj(emb, "bigram", "the embedding")
        if pair is not None:
            pair = ZifetarBigram(*(_at("the embedding's bigram", take_int, pair, k, required=True, minimum=low)
                                   for k, low in (("buckets", 1), ("mul_prev", 0), ("mul_cur", 0))))
            if pair.buckets >= 2 ** 31:
                raise ConfigError(f"config.json: the embedding's bigram: {pair.buckets} buckets")
        entries = d.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers: List[ZifetarLayer] = []
        for i, e in enumerate(entries):
            where = f"layer {i}"
            if not isinstance(e, dict):
                raise ConfigError(f"config.json: {where} must be an object")
            kind = e.get("type")
            if kind not in MIXERS:
                raise ConfigError(f"config.json: {where}: no mixer of type {kind!r}; there are {sorted(MIXERS)}")
            mixer = MIXERS[kind].from_dict(take_obj(e, "mixer", where, required=True), where)
            mlp = take_obj(e, "mlp", where)
            if mlp is not None:
                ff = mlp.get("kind")
                if ff not in FEED_FORWARDS:
                    raise ConfigError(f"config.json: {where}: no feed-forward of kind {ff!r}; there are {sorted(FEED_FORWARDS)}")
                mlp = FEED_FORWARDS[ff].from_dict(mlp, where)
            layers.append(ZifetarLayer(type=kind, mixer=mixer, mlp=mlp))
        known = {"architecture", "architectures", "vocab", "width", "norm", "embedding", "layers", "eos_token_id",
                 "max_position_embeddings", "torch_dtype"}
        eos = d.get("eos_token_id")
        eos_ids = [eos] if isinstance(eos, int) and not isinstance(eos, bool) else list(eos or [])
        return cls(architecture=NAME, extra={k: v for k, v in d.items() if k not in known},
                   vocab_size=take_int(d, "vocab", required=True, minimum=1),
                   hidden_size=take_int(d, "width", required=True, minimum=1),
                   norm_eps=take_float(norm, "eps", required=True, positive=True),
                   embedding_scale=_at("the embedding", take_float, emb, "scale", default=1.0), bigram=pair, layers=layers,
                   eos_token_ids=eos_ids,
                   max_position_embeddings=take_int(d, "max_position_embeddings", default=None, allow_none=True,
                                                    minimum=1))

    def to_dict(self) -> Dict[str, Any]:
        emb: Dict[str, Any] = {"scale": self.embedding_scale}
        if self.bigram is not None:
            emb["bigram"] = self.bigram.to_dict()
        d: Dict[str, Any] = {"architecture": NAME, "vocab": self.vocab_size, "width": self.hidden_size,
                             "norm": {"eps": self.norm_eps}, "embedding": emb, "layers": [l.to_dict() for l in self.layers]}
        if self.eos_token_ids:
            d["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        if self.max_position_embeddings is not None:
            d["max_position_embeddings"] = self.max_position_embeddings
        d.update(self.extra)
        return d
