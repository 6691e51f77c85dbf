"""`ZudalornConfig`: the config.json of a Zudalorn model, typed.

The file names its design in `architecture`, the sizes `vocab` and `width`, `norm.eps` and
`layers`, a list with one entry per layer.  A layer's entry has `type` (which mixer), `mixer` (its
sizes and constants) and `mlp` (the feed-forward, or null for a layer without one); every entry is
read on its own, so layers may differ in every size.

Mixer `latent_attention`: `heads`, `dim` and `rot_dim` (the unrotated and the rotated query and key
channels of a head), `vdim` (value channels of a head), `kv_rank` (channels of the latent), `scale`
(the factor on a score), `rot` = {`base`, `dims` (equal to rot_dim), `scaling`}, `scaling` =
{`factor`, `original`, `fast`, `slow`} (absent: plain frequencies), `mask.size` (the sliding window;
absent: every earlier position is seen).
Mixer `retention`: `heads`, `dim`, `vdim`, `decay` (a number per head), `rot` = {`base`, `dims`}
(absent: no rotation).
Feed-forward `dense`: `ff`.  Feed-forward `moe`: `router` = {`experts`, `top`, `groups` =
{`count`, `keep`} (absent: no groups)}, `expert.ff`, `shared.ff` (absent: no shared expert).
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Union

from .base import ConfigError, ModelConfig, take_float, take_int, take_obj

MAX_HEAD_DIM = 256          # the largest head the attention kernels take (dim + rot_dim, vdim)
MAX_LATENT = 1024           # the largest latent with its rotated part
MAX_RETENTION_DIM = 512     # the largest key size of a retention head
MAX_EXPERTS = 1024
NAME = "Zudalorn"


def _at(where, take, *args, **kw):
    try:
        return take(*args, **kw)
    except ConfigError as e:
        raise ConfigError(f"{e} (in {where})") from None


@dataclass
class YarnScaling:
    """The stretch of a rotation's slow pairs: see `parts.position.Rotary`."""
    factor: float
    original: float
    fast: float
    slow: float

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "YarnScaling":
        return cls(**{k: _at(where, take_float, d, k, required=True, positive=True)
                      for k in ("factor", "original", "fast", "slow")})

    def to_dict(self) -> Dict[str, Any]:
        return {"factor": self.factor, "original": self.original, "fast": self.fast, "slow": self.slow}


def _rotation(m: Dict[str, Any], most: int, where: str):
    """(base, dims, scaling) of a mixer's `rot`, dims at most `most`; (None, 0, None) without one."""
    rot = take_obj(m, "rot", where)
    if rot is None:
        return None, 0, None
    base = _at(where, take_float, rot, "base", required=True, positive=True)
    dims = _at(where, take_int, rot, "dims", default=most, minimum=0)
    if dims % 2 or dims > most:
        raise ConfigError(f"config.json: {where}: {dims} rotated channels of {most} (even, at most as many)")
    scaling = take_obj(rot, "scaling", where)
    return base, dims, None if scaling is None else YarnScaling.from_dict(scaling, where)


def _rotation_dict(base, dims, scaling) -> Dict[str, Any]:
    d: Dict[str, Any] = {"base": base, "dims": dims}
    if scaling is not None:
        d["scaling"] = scaling.to_dict()
    return d


@dataclass
class ZudalornAttention:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: Optional[float] = None
    scaling: Optional[YarnScaling] = None
    window: Optional[int] = None

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZudalornAttention":
        n = {k: _at(where, take_int, m, k, required=True, minimum=0 if k == "rot_dim" else 1)
             for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank")}
        if max(n["dim"] + n["rot_dim"], n["vdim"]) > MAX_HEAD_DIM:
            raise ConfigError(f"config.json: {where}: head sizes {n['dim']} + {n['rot_dim']} / {n['vdim']} are not served "
                              f"(up to {MAX_HEAD_DIM})")
        if n["kv_rank"] + n["rot_dim"] > MAX_LATENT:
            raise ConfigError(f"config.json: {where}: a latent of {n['kv_rank']} + {n['rot_dim']} channels is not served "
                              f"(up to {MAX_LATENT})")
        base, dims, scaling = _rotation(m, n["rot_dim"], where)
        if dims != n["rot_dim"]:
            raise ConfigError(f"config.json: {where}: rot.dims {dims} is not rot_dim {n['rot_dim']}")
        mask = take_obj(m, "mask", where)
        return cls(scale=_at(where, take_float, m, "scale", required=True), rot_base=base, scaling=scaling,
                   window=None if mask is None else _at(where, take_int, mask, "size", required=True, minimum=1), **n)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim,
                             "kv_rank": self.kv_rank, "scale": self.scale}
        if self.rot_base is not None:
            d["rot"] = _rotation_dict(self.rot_base, self.rot_dim, self.scaling)
        if self.window is not None:
            d["mask"] = {"size": self.window}
        return d


@dataclass
class ZudalornRetention:
    heads: int
    dim: int
    vdim: int
    decay: List[float]
    rot_base: Optional[float] = None
    rot_dims: int = 0
    scaling: Optional[YarnScaling] = None

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZudalornRetention":
        heads, dim, vdim = (_at(where, take_int, m, k, required=True, minimum=1) for k in ("heads", "dim", "vdim"))
        if dim > MAX_RETENTION_DIM:
            raise ConfigError(f"config.json: {where}: a retention head of {dim} is not served (up to {MAX_RETENTION_DIM})")
        decay = m.get("decay")
        if (not isinstance(decay, list) or len(decay) != heads
                or any(isinstance(a, bool) or not isinstance(a, (int, float)) or not 0 <= a for a in decay)):
            raise ConfigError(f"config.json: {where}: 'decay' must list {heads} numbers, none below 0")
        base, dims, scaling = _rotation(m, dim, where)
        return cls(heads=heads, dim=dim, vdim=vdim, decay=[float(a) for a in decay], rot_base=base if dims else None,
                   rot_dims=dims, scaling=scaling if dims else None)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}
        if self.rot_dims:
            d["rot"] = _rotation_dict(self.rot_base, self.rot_dims, self.scaling)
        return d


@dataclass
class ZudalornDense:
    ff: int

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZudalornDense":
        return cls(ff=_at(where, take_int, m, "ff", required=True, minimum=1))

    def to_dict(self) -> Dict[str, Any]:
        return {"kind": "dense", "ff": self.ff}


@dataclass
class ZudalornExperts:
    experts: int
    top: int
    ff: int
    groups: Optional[int] = None
    keep: Optional[int] = None
    shared_ff: Optional[int] = None

    @classmethod
    def from_dict(cls, m: Dict[str, Any], where: str) -> "ZudalornExperts":
        router = take_obj(m, "router", where, required=True)
        expert = take_obj(m, "expert", where, required=True)
        shared = take_obj(m, "shared", where)
        experts = _at(where, take_int, router, "experts", required=True, minimum=1)
        top = _at(where, take_int, router, "top", required=True, minimum=1)
        if experts > MAX_EXPERTS or top > experts:
            raise ConfigError(f"config.json: {where}: {top} of {experts} experts (at most {MAX_EXPERTS}, top within them)")
        groups = take_obj(router, "groups", where)
        count = keep = None
        if groups is not None:
            count = _at(where, take_int, groups, "count", required=True, minimum=1)
            keep = _at(where, take_int, groups, "keep", required=True, minimum=1)
            if experts % count or keep > count or keep * (experts // count) < top:
                raise ConfigError(f"config.json: {where}: {experts} experts in {count} groups of which {keep} are kept "
                                  f"cannot give {top}")
        return cls(experts=experts, top=top, ff=_at(where, take_int, expert, "ff", required=True, minimum=1),
                   groups=count, keep=keep,
                   shared_ff=None if shared is None else _at(where, take_int, shared, "ff", required=True, minimum=1))

    def to_dict(self) -> Dict[str, Any]:
        r: Dict[str, Any] = {"experts": self.experts, "top": self.top}
        if self.groups is not None:
            r["groups"] = {"count": self.groups, "keep": self.keep}
        d: Dict[str, Any] = {"kind": "moe", "router": r, "expert": {"ff": self.ff}}
        if self.shared_ff is not None:
            d["shared"] = {"ff": self.shared_ff}
        return d


MIXERS = {"latent_attention": ZudalornAttention, "retention": ZudalornRetention}
FEED_FORWARDS = {"dense": ZudalornDense, "moe": ZudalornExperts}


@dataclass
class ZudalornLayer:
    type: str
    mixer: Union[ZudalornAttention, ZudalornRetention]
    mlp: Optional[Union[ZudalornDense, ZudalornExperts]] = None

    def to_dict(self) -> Dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass
class ZudalornConfig(ModelConfig):
    vocab_size: int = 0
    hidden_size: int = 0
    norm_eps: float = 1e-5
    layers: List[ZudalornLayer] = field(default_factory=list)
    eos_token_ids: List[int] = field(default_factory=list)
    max_position_embeddings: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "ZudalornConfig":
        norm = take_obj(d, "norm", "the model", required=True)
        entries = d.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers: List[ZudalornLayer] = []
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
            layers.append(ZudalornLayer(type=kind, mixer=mixer, mlp=mlp))
        known = {"architecture", "architectures", "vocab", "width", "norm", "layers", "eos_token_id",
                 "max_position_embeddings", "torch_dtype"}
        eos = d.get("eos_token_id")
        eos_ids = [eos] if isinstance(eos, int) and not isinstance(eos, bool) else list(eos or [])
        return cls(architecture=NAME, extra={k: v for k, v in d.items() if k not in known},
                   vocab_size=take_int(d, "vocab", required=True, minimum=1),
                   hidden_size=take_int(d, "width", required=True, minimum=1),
                   norm_eps=take_float(norm, "eps", required=True, positive=True), layers=layers, eos_token_ids=eos_ids,
                   max_position_embeddings=take_int(d, "max_position_embeddings", default=None, allow_none=True,
                                                    minimum=1))

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"architecture": NAME, "vocab": self.vocab_size, "width": self.hidden_size,
                             "norm": {"eps": self.norm_eps}, "layers": [l.to_dict() for l in self.layers]}
        if self.eos_token_ids:
            d["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        if self.max_position_embeddings is not None:
            d["max_position_embeddings"] = self.max_position_embeddings
        d.update(self.extra)
        return d
