"""Typed configuration of the Nidasun decoder, read from config.json.

The file lists the layers one by one; each names its mixer (``type``), the mixer's sizes and
constants (``mixer``) and its feed-forward (``mlp``, or null for a layer without one):

    {"architecture": "Nidasun", "vocab": V, "width": D, "streams": S, "norm": {"eps": e},
     "loop": {"start": a, "stop": b, "times": n},
     "layers": [{"type": "attention",
                 "mixer": {"heads": H, "kv_heads": G, "dim": dk, "vdim": dv, "scale": s, "mask": {"size": chunk},
                           "rot": {"base": b, "dims": n}},
                 "mlp": {"kind": "moe", "expert": {"ff": F},
                         "router": {"experts": E, "top": k, "scale": r, "groups": {"count": g, "keep": m}}}},
                {"type": "lightning", "mixer": {"heads": H, "dim": dk, "vdim": dv, "decay": [one a head]}, "mlp": null},
                {"type": "parallel",
                 "mixer": {"left": {as attention, "mask": {"size": window},
                                    "rot": {"base": b, "dims": n, "scaling": {"factor": f}}},
                           "right": {"width": W, "blocks": B, "conv": taps}, "left_scale": a, "right_scale": b},
                 "mlp": {"kind": "dense", "ff": F}}, ...]}

Every size and constant of the model is read here and handed to the parts as a parameter.  A key
that is missing or of the wrong kind is reported by its path (``layers[3].mixer.left.heads``).  Layers
a to b - 1 run n times in a row; without ``loop`` every layer runs once.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Mapping, Optional, Tuple

from .base import ConfigError, read_key, token_id_list
from .dudatar import LoopConfig, _at, _obj

MIXERS = ("attention", "lightning", "parallel")
FEED_FORWARDS = ("dense", "moe")


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int                   # how many numbers of a head turn
    factor: float = 0.0         # what every frequency is divided by (0: as it is)


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int                    # query/key numbers per head
    vdim: int                   # value numbers per head
    scale: float
    mask: int                   # positions of a chunk, or of a window in a parallel layer
    rot: RotationConfig


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]    # one a head


@dataclass(frozen=True)
class RecurrenceConfig:
    width: int
    blocks: int
    conv: int                   # taps of the convolution over time


@dataclass(frozen=True)
class ParallelConfig:
    left: AttentionConfig
    right: RecurrenceConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class DenseFFConfig:
    ff: int
    kind: str = "dense"


@dataclass(frozen=True)
class MoEFFConfig:
    ff: int
    experts: int
    top: int
    scale: float
    groups: int = 1
    keep: int = 1
    kind: str = "moe"


@dataclass(frozen=True)
class NidasunLayer:
    type: str
    mixer: object               # AttentionConfig, LightningConfig or ParallelConfig
    mlp: object                 # DenseFFConfig, MoEFFConfig or None


def _attention(mx: Mapping, mp: str) -> AttentionConfig:
    heads, dim = _at(mp, read_key, mx, "heads", int), _at(mp, read_key, mx, "dim", int)
    mask, rot, rp = _obj(mx, "mask", mp + "."), _obj(mx, "rot", mp + "."), mp + ".rot"
    scaling = _obj(rot, "scaling", rp + ".", optional=True)
    factor = 0.0 if scaling is None else _at(rp + ".scaling", read_key, scaling, "factor", float)
    return AttentionConfig(
        heads=heads, kv_heads=_at(mp, read_key, mx, "kv_heads", int, heads), dim=dim, vdim=_at(mp, read_key, mx, "vdim", int, dim),
        scale=_at(mp, read_key, mx, "scale", float), mask=_at(mp + ".mask", read_key, mask, "size", int),
        rot=RotationConfig(base=_at(rp, read_key, rot, "base", float), dims=_at(rp, read_key, rot, "dims", int, dim), factor=factor))


def _lightning(mx: Mapping, mp: str) -> LightningConfig:
    dim, decay = _at(mp, read_key, mx, "dim", int), mx.get("decay")
    if not isinstance(decay, (list, tuple)) or not all(isinstance(d, (int, float)) and not isinstance(d, bool) for d in decay):
        raise ConfigError(f"missing/invalid config key: {mp}.decay (want a list of numbers)")
    return LightningConfig(heads=_at(mp, read_key, mx, "heads", int), dim=dim, vdim=_at(mp, read_key, mx, "vdim", int, dim),
                           decay=tuple(float(d) for d in decay))


def _mixer(kind: str, mx: Mapping, mp: str):
    if kind == "attention":
        return _attention(mx, mp)
    if kind == "lightning":
        return _lightning(mx, mp)
    right, rp = _obj(mx, "right", mp + "."), mp + ".right"
    return ParallelConfig(
        left=_attention(_obj(mx, "left", mp + "."), mp + ".left"),
        right=RecurrenceConfig(*(_at(rp, read_key, right, k, int) for k in ("width", "blocks", "conv"))),
        left_scale=_at(mp, read_key, mx, "left_scale", float), right_scale=_at(mp, read_key, mx, "right_scale", float))


def _feed_forward(mlp: Mapping, fp: str):
    kind = _at(fp, read_key, mlp, "kind", str, "dense")
    if kind == "dense":
        return DenseFFConfig(ff=_at(fp, read_key, mlp, "ff", int))
    if kind != "moe":
        raise ConfigError(f"unknown feed-forward kind: {fp}.kind = {kind!r} (known: {', '.join(FEED_FORWARDS)})")
    router, rp = _obj(mlp, "router", fp + "."), fp + ".router"
    groups = _obj(router, "groups", rp + ".", optional=True)
    count = keep = 1
    if groups is not None:
        count, keep = (_at(rp + ".groups", read_key, groups, k, int) for k in ("count", "keep"))
    return MoEFFConfig(ff=_at(fp + ".expert", read_key, _obj(mlp, "expert", fp + "."), "ff", int),
                       experts=_at(rp, read_key, router, "experts", int), top=_at(rp, read_key, router, "top", int),
                       scale=_at(rp, read_key, router, "scale", float), groups=count, keep=keep)


@dataclass(frozen=True)
class NidasunConfig:
    architecture: str
    vocab: int
    width: int
    streams: int
    norm_eps: float
    layers: Tuple[NidasunLayer, ...]
    loop: Optional[LoopConfig] = None
    eos_token_ids: Tuple[int, ...] = ()
    extra: Mapping[str, Any] = field(default_factory=dict, compare=False)

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "NidasunConfig":
        norm, loop = _obj(d, "norm", ""), _obj(d, "loop", "", optional=True)
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
            raise ConfigError("missing/invalid config key: layers (want a list of layers)")
        layers = []
        for i, layer in enumerate(raw_layers):
            path = f"layers[{i}]"
            if not isinstance(layer, Mapping):
                raise ConfigError(f"missing/invalid config key: {path} (want an object)")
            kind = _at(path, read_key, layer, "type", str)
            if kind not in MIXERS:
                raise ConfigError(f"unknown layer type: {path}.type = {kind!r} (known: {', '.join(MIXERS)})")
            mlp = _obj(layer, "mlp", path + ".", optional=True)
            layers.append(NidasunLayer(kind, _mixer(kind, _obj(layer, "mixer", path + "."), path + ".mixer"),
                                       None if mlp is None else _feed_forward(mlp, path + ".mlp")))
        known = {"architecture", "architectures", "vocab", "width", "streams", "norm", "layers", "loop", "eos_token_id"}
        cfg = cls(
            architecture="Nidasun",
            vocab=read_key(d, "vocab", int), width=read_key(d, "width", int), streams=read_key(d, "streams", int, 1),
            norm_eps=_at("norm", read_key, norm, "eps", float),
            layers=tuple(layers),
            loop=None if loop is None else LoopConfig(*(_at("loop", read_key, loop, k, int) for k in ("start", "stop", "times"))),
            eos_token_ids=token_id_list(d.get("eos_token_id"), "eos_token_id"),
            extra={k: v for k, v in d.items() if k not in known})
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0 or self.streams <= 0:
            raise ConfigError("vocab, width and streams must be positive")
        if self.norm_eps < 0:
            raise ConfigError("norm.eps must not be negative")

        def positive(path, s, keys):
            for key in keys:
                if getattr(s, key) <= 0:
                    raise ConfigError(f"{path}.{key} must be positive")
        for i, layer in enumerate(self.layers):
            m, path = layer.mixer, f"layers[{i}].mixer"
            attention, ap = None, path
            if isinstance(m, AttentionConfig):
                attention = m
            elif isinstance(m, ParallelConfig):
                attention, ap = m.left, path + ".left"
                positive(path + ".right", m.right, ("width", "blocks", "conv"))
                if m.right.width % m.right.blocks:
                    raise ConfigError(f"{path}.right: {m.right.blocks} blocks do not divide a width of {m.right.width}")
            else:
                positive(path, m, ("heads", "dim", "vdim"))
                if len(m.decay) != m.heads:
                    raise ConfigError(f"{path}.decay: {len(m.decay)} numbers for {m.heads} heads")
                if not all(0.0 <= d <= 1.0 for d in m.decay):
                    raise ConfigError(f"{path}.decay: a decay lies between 0 and 1")
            if attention is not None:
                positive(ap, attention, ("heads", "kv_heads", "dim", "vdim"))
                rot = attention.rot
                if attention.mask <= 0:
                    raise ConfigError(f"{ap}.mask.size must be positive")
                if attention.heads % attention.kv_heads:
                    raise ConfigError(f"{ap}: {attention.heads} heads are not a multiple of {attention.kv_heads} kv_heads")
                if rot.dims < 0 or rot.dims % 2 or rot.dims > attention.dim:
                    raise ConfigError(f"{ap}.rot.dims = {rot.dims} must be even and at most {attention.dim}")
                if rot.dims and rot.base <= 0:
                    raise ConfigError(f"{ap}.rot.base must be positive")
                if rot.factor < 0:
                    raise ConfigError(f"{ap}.rot.scaling.factor must be positive")
            f, fp = layer.mlp, f"layers[{i}].mlp"
            if f is not None:
                if f.ff <= 0:
                    raise ConfigError(f"{fp}: the feed-forward's ff must be positive")
                if isinstance(f, MoEFFConfig):
                    positive(fp + ".router", f, ("experts", "top", "groups", "keep"))
                    if f.top > f.experts:
                        raise ConfigError(f"{fp}.router: {f.top} choices of {f.experts} experts")
                    if f.experts % f.groups or f.keep > f.groups:
                        raise ConfigError(f"{fp}.router.groups: {f.keep} of {f.groups} groups do not fit {f.experts} experts")
                    if f.keep * (f.experts // f.groups) < f.top:
                        raise ConfigError(f"{fp}.router.groups: {f.keep} groups of {f.experts // f.groups} experts hold fewer than "
                                          f"the {f.top} a token takes")
        if self.loop is not None:
            lp = self.loop
            if not 0 <= lp.start < lp.stop <= len(self.layers):
                raise ConfigError(f"loop: start = {lp.start} and stop = {lp.stop} do not name a run of the {len(self.layers)} layers")
            if lp.times <= 0:
                raise ConfigError("loop.times must be positive")

    def to_dict(self) -> dict:
        def attention(a):
            rot = {"base": a.rot.base, "dims": a.rot.dims}
            if a.rot.factor:
                rot["scaling"] = {"factor": a.rot.factor}
            return {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale,
                    "mask": {"size": a.mask}, "rot": rot}

        def mixer(m):
            if isinstance(m, AttentionConfig):
                return attention(m)
            if isinstance(m, LightningConfig):
                return {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": list(m.decay)}
            return {"left": attention(m.left), "left_scale": m.left_scale, "right_scale": m.right_scale,
                    "right": {"width": m.right.width, "blocks": m.right.blocks, "conv": m.right.conv}}

        def feed_forward(f):
            if f is None:
                return None
            if isinstance(f, DenseFFConfig):
                return {"kind": "dense", "ff": f.ff}
            return {"kind": "moe", "expert": {"ff": f.ff},
                    "router": {"experts": f.experts, "top": f.top, "scale": f.scale, "groups": {"count": f.groups, "keep": f.keep}}}
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "streams": self.streams,
             "norm": {"eps": self.norm_eps},
             "layers": [{"type": x.type, "mixer": mixer(x.mixer), "mlp": feed_forward(x.mlp)} for x in self.layers]}
        if self.loop is not None:
            d["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        if self.eos_token_ids:
            d["eos_token_id"] = list(self.eos_token_ids)
        d.update(self.extra)
        return d
