"""Configuration of the Notadra decoder, from its config.json.

A Notadra model is a list of attention layers with RMS norms on both sides of every sublayer, whose gains are stored as
distances from one.  Queries, keys and values have biases; the first elements of a head turn in halves, with frequencies
stretched for long contexts; scores are scaled and capped, and the softmax has a sink of score 0.  A layer may read the
keys and values of an earlier one instead of making its own.  Feed-forwards are mixtures of squared-ReLU experts with a
sigmoid router over groups.  The embedding adds a row for the pair of the token before and the token.  config.json
names the design in ``"architecture"`` and gives every size and constant:

    vocab, width, norm: {eps}, logit_scale, embedding: {bigram: {buckets, mul_prev, mul_cur}},
    layers: [{type: "attention",
              mixer: {heads, kv_heads, dim, vdim, scale, softcap, kv_from,
                      rot: {dims, base, scaling: {factor, original, fast, slow}}},
              mlp: {kind: "moe", expert: {ff}, router: {experts, top, groups: {count, keep}}} or null}, ...]

Optional keys that are absent or null mean that the mechanism is not there (``softcap``, ``kv_from``, ``rot``,
``rot.scaling``, ``groups``, ``bigram``).  ``max_positions`` is no key of the design; where it is given it is the default length
of a cache that is given none.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import ClassVar, Optional

from ..errors import ConfigError, UnsupportedError
from .base import ModelConfig, f32, whole

DEFAULT_MAX_POSITIONS = 1 << 20


def _section(raw, key: str, where: str) -> dict:
    v = raw.get(key) if isinstance(raw, dict) else None
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: {key!r} must be an object, got {v!r}")
    return v


def _number(raw: dict, key: str, where: str) -> float:
    """A number as config.json has it: what is computed from it once, on the host, is computed in 64-bit."""
    v = raw.get(key)
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"config key {where + '.' + key!r}: expected a number, got {v!r}")
    return float(v)


@dataclass(frozen=True)
class StretchedRotation:
    """Frequencies for contexts ``factor`` times as long as ``original``: pairs that turn more than ``fast`` times in the
    original context keep theirs, pairs that turn less than ``slow`` times turn ``factor`` times slower, with a ramp between."""
    factor: float
    original: float
    fast: float
    slow: float

    @classmethod
    def read(cls, raw: dict, where: str) -> "StretchedRotation":
        s = cls(*(_number(raw, key, where) for key in ("factor", "original", "fast", "slow")))
        if min(s.factor, s.original, s.fast, s.slow) <= 0:
            raise ConfigError(f"{where}: factor, original, fast and slow must be positive")
        return s

    def to_dict(self) -> dict:
        return {"factor": self.factor, "original": self.original, "fast": self.fast, "slow": self.slow}


@dataclass(frozen=True)
class SharedAttentionSizes:
    heads: int
    kv_heads: int
    dim: int                          # size of a query or key head
    vdim: int                         # size of a value head
    scale: float                      # factor on q . k
    softcap: Optional[float]          # scores are capped at +- softcap; None: they are not
    rot_dims: int                     # the first rot_dims elements of a head turn, i with i + rot_dims / 2
    rot_base: float
    scaling: Optional[StretchedRotation]
    kv_from: Optional[int]            # the layer whose keys and values this one reads; None: its own

    @classmethod
    def read(cls, m: dict, where: str) -> "SharedAttentionSizes":
        for key in ("heads", "dim", "scale"):
            if key not in m:
                raise ConfigError(f"{where}: an attention mixer needs {key!r}")
        heads = whole(m["heads"], where + ".heads", 1)
        kv = whole(m.get("kv_heads", heads), where + ".kv_heads", 1)
        if heads % kv:
            raise ConfigError(f"{where}: {heads} heads not divisible by {kv} kv heads")
        dim = whole(m["dim"], where + ".dim", 1)
        rot_dims, rot_base, scaling = 0, 10000.0, None
        if m.get("rot") is not None:
            rot = _section(m, "rot", where)
            rot_dims = whole(rot.get("dims"), where + ".rot.dims", 0)
            rot_base = _number(rot, "base", where + ".rot")
            if rot_dims % 2 or rot_dims > dim:
                raise ConfigError(f"{where}.rot.dims {rot_dims} must be even and at most the head size {dim}")
            if rot.get("scaling") is not None:
                scaling = StretchedRotation.read(_section(rot, "scaling", where + ".rot"), where + ".rot.scaling")
            if rot_dims and (not rot_base > 0 or (scaling is not None and rot_base == 1.0)):
                raise ConfigError(f"{where}.rot.base {rot_base} must be positive, and not 1 where the frequencies are stretched")
        scale = f32(m["scale"], where + ".scale")
        if not scale > 0:
            raise ConfigError(f"{where}.scale {scale} must be positive")
        cap = None
        if m.get("softcap"):
            cap = f32(m["softcap"], where + ".softcap")
            if not cap > 0:
                raise ConfigError(f"{where}.softcap {cap} must be positive")
        kv_from = None if m.get("kv_from") is None else whole(m["kv_from"], where + ".kv_from", 0)
        vdim = dim if m.get("vdim") is None else whole(m["vdim"], where + ".vdim", 1)
        return cls(heads, kv, dim, vdim, scale, cap, rot_dims, rot_base, scaling, kv_from)

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.softcap is not None:
            out["softcap"] = self.softcap
        if self.rot_dims:
            out["rot"] = {"dims": self.rot_dims, "base": self.rot_base}
            if self.scaling is not None:
                out["rot"]["scaling"] = self.scaling.to_dict()
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class RoutedExpertsSizes:
    experts: int
    top: int
    ff: int                           # width of one expert
    groups: int = 1                   # the experts form this many equal groups of neighbours
    keep: int = 1                     # of which the best `keep` can be chosen from

    @classmethod
    def read(cls, mlp: dict, where: str) -> "RoutedExpertsSizes":
        if mlp.get("kind") != "moe":
            raise UnsupportedError(f"{where}: feed-forward kind {mlp.get('kind')!r} is not 'moe'")
        expert, router = _section(mlp, "expert", where), _section(mlp, "router", where)
        experts = whole(router.get("experts"), where + ".router.experts", 1)
        top = whole(router.get("top"), where + ".router.top", 1)
        groups = keep = 1
        if router.get("groups") is not None:
            g = _section(router, "groups", where + ".router")
            groups = whole(g.get("count", 1), where + ".router.groups.count", 1)
            keep = whole(g.get("keep", groups), where + ".router.groups.keep", 1)
        if experts % groups or keep > groups:
            raise ConfigError(f"{where}.router: {experts} experts in {groups} groups of which {keep} stay")
        if top > keep * (experts // groups):
            raise ConfigError(f"{where}.router: the {top} best of the {keep * (experts // groups)} experts of {keep} groups")
        return cls(experts, top, whole(expert.get("ff"), where + ".expert.ff", 1), groups, keep)

    def to_dict(self) -> dict:
        return {"kind": "moe", "expert": {"ff": self.ff},
                "router": {"experts": self.experts, "top": self.top, "groups": {"count": self.groups, "keep": self.keep}}}


@dataclass(frozen=True)
class NotadraLayer:
    type: str                                     # "attention"
    mixer: SharedAttentionSizes
    mlp: Optional[RoutedExpertsSizes] = None      # None: the layer has no feed-forward

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class BigramSizes:
    buckets: int
    mul_prev: int
    mul_cur: int

    def to_dict(self) -> dict:
        return {"buckets": self.buckets, "mul_prev": self.mul_prev, "mul_cur": self.mul_cur}


@dataclass(frozen=True)
class NotadraConfig(ModelConfig):
    vocab: int = 0
    width: int = 0
    layers: tuple = ()
    norm_eps: float = 1e-5
    logit_scale: float = 1.0
    bigram: Optional[BigramSizes] = None
    max_positions: int = DEFAULT_MAX_POSITIONS

    ARCHITECTURE: ClassVar[str] = "Notadra"
    MODEL_TYPE: ClassVar[str] = "notadra"
    REQUIRED: ClassVar[tuple[str, ...]] = ("vocab", "width", "layers", "norm")

    @classmethod
    def from_dict(cls, raw: dict) -> "NotadraConfig":
        cls.require(raw)
        if not isinstance(raw["layers"], list) or not raw["layers"]:
            raise ConfigError("config key 'layers' must be a list of at least one layer")
        layers = []
        for i, entry in enumerate(raw["layers"]):
            where = f"layers[{i}]"
            if not isinstance(entry, dict) or entry.get("type") != "attention":
                kind = entry.get("type") if isinstance(entry, dict) else entry
                raise UnsupportedError(f"{where}: mixer type {kind!r} is not 'attention'")
            mlp = None if entry.get("mlp") is None else RoutedExpertsSizes.read(_section(entry, "mlp", where), where + ".mlp")
            layers.append(NotadraLayer("attention", SharedAttentionSizes.read(_section(entry, "mixer", where), where + ".mixer"), mlp))
        bigram = None
        if raw.get("embedding") is not None and _section(raw, "embedding", "config.json").get("bigram") is not None:
            b = _section(raw["embedding"], "bigram", "embedding")
            bigram = BigramSizes(*(whole(b.get(key), "embedding.bigram." + key, least)
                                   for key, least in (("buckets", 1), ("mul_prev", 0), ("mul_cur", 0))))
        scale = raw.get("logit_scale")
        cfg = cls(vocab=whole(raw["vocab"], "vocab", 1), width=whole(raw["width"], "width", 1), layers=tuple(layers),
                  norm_eps=f32(_section(raw, "norm", "config.json").get("eps"), "norm.eps"),
                  logit_scale=1.0 if scale is None else f32(scale, "logit_scale"), bigram=bigram,
                  max_positions=whole(raw.get("max_positions", DEFAULT_MAX_POSITIONS), "max_positions", 1))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if not self.norm_eps >= 0.0:
            raise ConfigError(f"norm.eps {self.norm_eps} must not be negative")
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if m.kv_from is None:
                continue
            if m.kv_from >= i:
                raise ConfigError(f"layers[{i}].mixer.kv_from {m.kv_from} must name an earlier layer")
            src = self.layers[m.kv_from].mixer
            if src.kv_from is not None:
                raise ConfigError(f"layers[{i}].mixer.kv_from {m.kv_from}: that layer has no keys and values of its own")
            if (src.kv_heads, src.dim, src.vdim) != (m.kv_heads, m.dim, m.vdim):
                raise ConfigError(f"layers[{i}] has {m.kv_heads} kv heads of {m.dim} and {m.vdim}, the layer {m.kv_from} whose keys it "
                                  f"reads {src.kv_heads} of {src.dim} and {src.vdim}")

    def to_dict(self) -> dict:
        out = {"architecture": self.ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "logit_scale": self.logit_scale, "layers": [layer.to_dict() for layer in self.layers]}
        if self.bigram is not None:
            out["embedding"] = {"bigram": self.bigram.to_dict()}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out
