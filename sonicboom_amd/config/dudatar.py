"""Typed configuration of the Dudatar decoder, read from config.json.

The file lists the layers one by one; each names its mixer (``type``), the mixer's sizes and
constants (``mixer``) and its feed-forward (``mlp``, or null for a layer without one):

    {"architecture": "Dudatar", "vocab": V, "width": D, "logit_softcap": c, "norm": {"eps": e},
     "loop": {"start": a, "stop": b, "times": n},
     "layers": [{"type": "parallel",
                 "mixer": {"left": {"heads": H, "kv_heads": G, "dim": dk, "vdim": dv, "scale": s,
                                    "rot": {"base": b, "dims": n}},
                           "right": {"heads": H, "dim": dk, "vdim": dv, "decay": [one a head],
                                     "rot": {"base": b, "dims": n}}},
                 "mlp": {"kind": "dense", "ff": F}},
                {"type": "gla", "mixer": {"heads": H, "dim": dk, "vdim": dv, "tau": t, "rank": r}, "mlp": null}, ...]}

Every size and constant of the model is read here and handed to the parts as a parameter.  A key
that is missing or of the wrong kind is reported by its path (``layers[3].mixer.left.heads``).  Layers
a to b - 1 run n times in a row; without ``loop`` every layer runs once.  ``rank``, the inner size of the
decays' projection, may be left to the file's tensors.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Mapping, Optional, Tuple

from .base import ConfigError, read_key, token_id_list

MIXERS = ("parallel", "gla")
FEED_FORWARDS = ("dense",)


def _at(path: str, fn, *a):
    """``fn(*a)`` with the path of the object in front of the key a ConfigError names."""
    try:
        return fn(*a)
    except ConfigError as e:
        raise ConfigError(str(e).replace("config key: ", f"config key: {path}.", 1)) from None


def _obj(d: Mapping, key: str, path: str, optional: bool = False):
    v = d.get(key)
    if v is None and optional:
        return None
    if not isinstance(v, Mapping):
        raise ConfigError(f"missing/invalid config key: {path}{key} (want an object)")
    return v


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int                   # how many numbers of a head turn


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int                    # query/key numbers per head
    vdim: int                   # value numbers per head
    scale: float
    rot: RotationConfig


@dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]    # one a head
    rot: RotationConfig


@dataclass(frozen=True)
class ParallelConfig:
    left: AttentionConfig
    right: RetentionConfig


@dataclass(frozen=True)
class GLAConfig:
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int = -1              # -1: what the file's tensors have


@dataclass(frozen=True)
class DenseFFConfig:
    ff: int
    kind: str = "dense"


@dataclass(frozen=True)
class DudatarLayer:
    type: str
    mixer: object               # ParallelConfig or GLAConfig
    mlp: Optional[DenseFFConfig]


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


def _rotation(mx: Mapping, mp: str, dim: int) -> RotationConfig:
    rot = _obj(mx, "rot", mp + ".")
    return RotationConfig(base=_at(mp + ".rot", read_key, rot, "base", float),
                          dims=_at(mp + ".rot", read_key, rot, "dims", int, dim))


def _attention(mx: Mapping, mp: str) -> AttentionConfig:
    heads, dim = _at(mp, read_key, mx, "heads", int), _at(mp, read_key, mx, "dim", int)
    return AttentionConfig(heads=heads, kv_heads=_at(mp, read_key, mx, "kv_heads", int, heads), dim=dim,
                           vdim=_at(mp, read_key, mx, "vdim", int, dim), scale=_at(mp, read_key, mx, "scale", float),
                           rot=_rotation(mx, mp, dim))


def _retention(mx: Mapping, mp: str) -> RetentionConfig:
    dim, decay = _at(mp, read_key, mx, "dim", int), mx.get("decay")
    if not isinstance(decay, (list, tuple)) or not all(isinstance(d, (int, float)) and not isinstance(d, bool) for d in decay):
        raise ConfigError(f"missing/invalid config key: {mp}.decay (want a list of numbers)")
    return RetentionConfig(heads=_at(mp, read_key, mx, "heads", int), dim=dim, vdim=_at(mp, read_key, mx, "vdim", int, dim),
                           decay=tuple(float(d) for d in decay), rot=_rotation(mx, mp, dim))


@dataclass(frozen=True)
class DudatarConfig:
    architecture: str
    vocab: int
    width: int
    logit_softcap: float        # 0: logits as they are
    norm_eps: float
    layers: Tuple[DudatarLayer, ...]
    loop: Optional[LoopConfig] = None
    eos_token_ids: Tuple[int, ...] = ()
    extra: Mapping[str, Any] = field(default_factory=dict, compare=False)

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "DudatarConfig":
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
            mx, mp = _obj(layer, "mixer", path + "."), path + ".mixer"
            if kind == "parallel":
                mixer = ParallelConfig(left=_attention(_obj(mx, "left", mp + "."), mp + ".left"),
                                       right=_retention(_obj(mx, "right", mp + "."), mp + ".right"))
            elif kind == "gla":
                dim = _at(mp, read_key, mx, "dim", int)
                mixer = GLAConfig(heads=_at(mp, read_key, mx, "heads", int), dim=dim, vdim=_at(mp, read_key, mx, "vdim", int, dim),
                                  tau=_at(mp, read_key, mx, "tau", float), rank=_at(mp, read_key, mx, "rank", int, -1))
            else:
                raise ConfigError(f"unknown layer type: {path}.type = {kind!r} (known: {', '.join(MIXERS)})")
            mlp, fp = _obj(layer, "mlp", path + ".", optional=True), path + ".mlp"
            ff = None
            if mlp is not None:
                ff_kind = _at(fp, read_key, mlp, "kind", str, "dense")
                if ff_kind not in FEED_FORWARDS:
                    raise ConfigError(f"unknown feed-forward kind: {fp}.kind = {ff_kind!r} "
                                      f"(known: {', '.join(FEED_FORWARDS)})")
                ff = DenseFFConfig(ff=_at(fp, read_key, mlp, "ff", int))
            layers.append(DudatarLayer(kind, mixer, ff))
        known = {"architecture", "architectures", "vocab", "width", "logit_softcap", "norm", "layers", "loop", "eos_token_id"}
        cfg = cls(
            architecture="Dudatar",
            vocab=read_key(d, "vocab", int), width=read_key(d, "width", int),
            logit_softcap=read_key(d, "logit_softcap", float, 0.0),
            norm_eps=_at("norm", read_key, norm, "eps", float),
            layers=tuple(layers),
            loop=None if loop is None else LoopConfig(*(_at("loop", read_key, loop, k, int) for k in ("start", "stop", "times"))),
            eos_token_ids=token_id_list(d.get("eos_token_id"), "eos_token_id"),
            extra={k: v for k, v in d.items() if k not in known})
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError("vocab and width must be positive")
        if self.norm_eps < 0 or self.logit_softcap < 0:
            raise ConfigError("norm.eps and logit_softcap must not be negative")
        for i, layer in enumerate(self.layers):
            m, path = layer.mixer, f"layers[{i}].mixer"
            sides = [(path + ".left", m.left, ("heads", "kv_heads", "dim", "vdim")),
                     (path + ".right", m.right, ("heads", "dim", "vdim"))] if isinstance(m, ParallelConfig) \
                else [(path, m, ("heads", "dim", "vdim"))]
            for sp, s, keys in sides:
                for key in keys:
                    if getattr(s, key) <= 0:
                        raise ConfigError(f"{sp}.{key} must be positive")
                rot = getattr(s, "rot", None)
                if rot is not None and (rot.dims < 0 or rot.dims % 2 or rot.dims > s.dim):
                    raise ConfigError(f"{sp}.rot.dims = {rot.dims} must be even and at most {s.dim}")
                if rot is not None and rot.dims and rot.base <= 0:
                    raise ConfigError(f"{sp}.rot.base must be positive")
            if isinstance(m, GLAConfig):
                if m.tau <= 0:
                    raise ConfigError(f"{path}.tau must be positive")
                if m.rank == 0 or m.rank < -1:
                    raise ConfigError(f"{path}.rank must be positive")
            else:
                if m.left.heads % m.left.kv_heads:
                    raise ConfigError(f"{path}.left: {m.left.heads} heads are not a multiple of {m.left.kv_heads} kv_heads")
                if len(m.right.decay) != m.right.heads:
                    raise ConfigError(f"{path}.right.decay: {len(m.right.decay)} numbers for {m.right.heads} heads")
                if not all(0.0 <= d <= 1.0 for d in m.right.decay):
                    raise ConfigError(f"{path}.right.decay: a decay lies between 0 and 1")
            if layer.mlp is not None and layer.mlp.ff <= 0:
                raise ConfigError(f"layers[{i}].mlp.ff must be positive")
        if self.loop is not None:
            lp = self.loop
            if not 0 <= lp.start < lp.stop <= len(self.layers):
                raise ConfigError(f"loop: start = {lp.start} and stop = {lp.stop} do not name a run of the {len(self.layers)} layers")
            if lp.times <= 0:
                raise ConfigError("loop.times must be positive")

    def to_dict(self) -> dict:
        def rotation(r):
            return {"base": r.base, "dims": r.dims}
        layers = []
        for layer in self.layers:
            m = layer.mixer
            if isinstance(m, ParallelConfig):
                a, b = m.left, m.right
                mx = {"left": {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale,
                               "rot": rotation(a.rot)},
                      "right": {"heads": b.heads, "dim": b.dim, "vdim": b.vdim, "decay": list(b.decay), "rot": rotation(b.rot)}}
            else:
                mx = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "tau": m.tau}
                if m.rank > 0:
                    mx["rank"] = m.rank
            layers.append({"type": layer.type, "mixer": mx,
                           "mlp": None if layer.mlp is None else {"kind": layer.mlp.kind, "ff": layer.mlp.ff}})
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "logit_softcap": self.logit_softcap,
             "norm": {"eps": self.norm_eps}, "layers": layers}
        if self.loop is not None:
            d["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        if self.eos_token_ids:
            d["eos_token_id"] = list(self.eos_token_ids)
        d.update(self.extra)
        return d
