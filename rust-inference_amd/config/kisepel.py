"""Configuration of the Kisepel decoder, from its config.json.

A Kisepel model is a list of layers whose mixer and feed-forward read the rows of one norm and are added to the residual
together.  A layer's mixer is one of three: linear attention with a fixed decay per head (``"lightning"``), a state-space
mixer with a scalar decay per head (``"mamba2"``), or two mixers side by side (``"parallel"``): softmax attention in chunks of the
sequence and the gated delta rule with a decay per key channel.  Its feed-forward is a mixture of experts that a table of token
ids chooses, beside an expert every token uses.  A stretch of the layers may run several times in a row with the same weights,
the embedding's output being added again before each pass but the first.  config.json names the design in ``"architecture"`` and
gives every size and constant:

    vocab, width, norm: {eps}, embedding: {scale} (absent: 1), logit_scale (absent: 1),
    loop: {start, stop, times} (absent: every layer once),
    layers: [{type: "lightning", mixer: {heads, dim, vdim, decay: [one per head]}, mlp},
             {type: "mamba2", mixer: {heads, vdim, state, groups, conv, norm_groups}, mlp},
             {type: "parallel", mixer: {left: {heads, kv_heads, dim, vdim, scale, mask: {size},
                                               rot: {dims, base, scaling: {factor}}},
                                        right: {heads, kv_heads, dim, vdim, conv[, rank]}}, mlp}, ...]
    mlp: {kind: "moe", expert: {ff}, router: {experts, top}, shared: {ff}} or null

``rank`` is the width of the delta rule's two narrow products, which a checkpoint's tensors give; a configuration that is to be
filled with random weights names it.  ``max_positions`` is no key of the design (positions enter through angles and chunks
alone); where it is given it is the default length of a cache that is given none.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import ClassVar, Optional

from ..errors import ConfigError, UnsupportedError
from .base import ModelConfig, f32, whole
from .dagezen import StateSpaceSizes
from .zakelorn import DecayAttentionSizes

DEFAULT_MAX_POSITIONS = 1 << 20


def _section(raw, key: str, where: str) -> dict:
    v = raw.get(key) if isinstance(raw, dict) else None
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: {key!r} must be an object, got {v!r}")
    return v


def _heads(m: dict, where: str, keys: tuple) -> tuple[int, int]:
    missing = [k for k in keys if k not in m]
    if missing:
        raise ConfigError(f"{where} lacks {', '.join(missing)}")
    heads = whole(m["heads"], where + ".heads", 1)
    kv = whole(m.get("kv_heads", heads), where + ".kv_heads", 1)
    if heads % kv:
        raise ConfigError(f"{where}: {heads} heads not divisible by {kv} kv heads")
    return heads, kv


@dataclass(frozen=True)
class ChunkedAttentionSizes:
    heads: int
    kv_heads: int
    dim: int                          # size of a query or key head
    vdim: int                         # size of a value head
    scale: float                      # factor on q . k
    chunk: Optional[int]              # a query sees the keys of its own run of this many positions; None: all before it
    rot_dims: int                     # the first rot_dims elements of a head turn, in halves
    rot_base: float
    rot_factor: float                 # every frequency is divided by it

    @classmethod
    def read(cls, m: dict, where: str) -> "ChunkedAttentionSizes":
        heads, kv = _heads(m, where, ("heads", "dim", "scale"))
        dim = whole(m["dim"], where + ".dim", 1)
        chunk = None
        if m.get("mask") is not None and _section(m, "mask", where).get("size") is not None:
            chunk = whole(m["mask"]["size"], where + ".mask.size", 1)
        dims, base, factor = 0, 10000.0, 1.0
        if m.get("rot") is not None:
            rot = _section(m, "rot", where)
            dims = whole(rot.get("dims", dim), where + ".rot.dims", 0)
            base = f32(rot.get("base", base), where + ".rot.base")
            if rot.get("scaling") is not None:
                factor = f32(_section(rot, "scaling", where + ".rot").get("factor", 1.0), where + ".rot.scaling.factor")
        if dims % 2 or dims > dim:
            raise ConfigError(f"{where}.rot.dims {dims} must be even and at most the head size {dim}")
        if not base > 0 or not factor > 0:
            raise ConfigError(f"{where}.rot: base {base} and factor {factor} must be positive")
        return cls(heads, kv, dim, whole(m.get("vdim", dim), where + ".vdim", 1), f32(m["scale"], where + ".scale"), chunk, dims,
                   base, factor)

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.chunk is not None:
            out["mask"] = {"size": self.chunk}
        if self.rot_dims:
            out["rot"] = {"dims": self.rot_dims, "base": self.rot_base, "scaling": {"factor": self.rot_factor}}
        return out


@dataclass(frozen=True)
class ChannelDeltaSizes:
    heads: int                        # value heads, each with a state of dim x vdim
    kv_heads: int                     # query/key heads, shared by heads / kv_heads value heads each
    dim: int
    vdim: int
    conv: int                         # taps of the short convolutions over q, k and v
    rank: Optional[int] = None        # width of the decay's and the gate's narrow middles; None: the checkpoint gives them

    @classmethod
    def read(cls, m: dict, where: str) -> "ChannelDeltaSizes":
        heads, kv = _heads(m, where, ("heads", "dim", "conv"))
        dim = whole(m["dim"], where + ".dim", 1)
        rank = whole(m["rank"], where + ".rank", 1) if m.get("rank") is not None else None
        return cls(heads, kv, dim, whole(m.get("vdim", dim), where + ".vdim", 1), whole(m["conv"], where + ".conv", 1), rank)

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}
        if self.rank is not None:
            out["rank"] = self.rank
        return out


@dataclass(frozen=True)
class PairSizes:
    left: ChunkedAttentionSizes
    right: ChannelDeltaSizes

    @classmethod
    def read(cls, m: dict, where: str) -> "PairSizes":
        return cls(ChunkedAttentionSizes.read(_section(m, "left", where), where + ".left"),
                   ChannelDeltaSizes.read(_section(m, "right", where), where + ".right"))

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


@dataclass(frozen=True)
class TableExpertsSizes:
    experts: int
    top: int
    ff: int                           # width of one expert
    shared_ff: Optional[int]          # width of the expert every token uses; None: there is none

    @classmethod
    def read(cls, mlp: dict, where: str) -> "TableExpertsSizes":
        if mlp.get("kind") != "moe":
            raise UnsupportedError(f"{where}: feed-forward kind {mlp.get('kind')!r} is not 'moe'")
        expert, router = _section(mlp, "expert", where), _section(mlp, "router", where)
        experts = whole(router.get("experts"), where + ".router.experts", 1)
        top = whole(router.get("top"), where + ".router.top", 1)
        if top > experts:
            raise ConfigError(f"{where}.router: {top} of {experts} experts")
        shared = None
        if mlp.get("shared") is not None:
            shared = whole(_section(mlp, "shared", where).get("ff"), where + ".shared.ff", 1)
        return cls(experts, top, whole(expert.get("ff"), where + ".expert.ff", 1), shared)

    def to_dict(self) -> dict:
        return {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top},
                "shared": None if self.shared_ff is None else {"ff": self.shared_ff}}


MIXER_SIZES = {"lightning": DecayAttentionSizes, "mamba2": StateSpaceSizes, "parallel": PairSizes}


@dataclass(frozen=True)
class KisepelLayer:
    type: str                                     # a key of MIXER_SIZES
    mixer: object
    mlp: Optional[TableExpertsSizes] = None       # None: the layer has no feed-forward

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class KisepelConfig(ModelConfig):
    vocab: int = 0
    width: int = 0
    layers: tuple = ()
    norm_eps: float = 1e-5
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1
    max_positions: int = DEFAULT_MAX_POSITIONS

    ARCHITECTURE: ClassVar[str] = "Kisepel"
    MODEL_TYPE: ClassVar[str] = "kisepel"
    REQUIRED: ClassVar[tuple[str, ...]] = ("vocab", "width", "layers", "norm")

    @classmethod
    def from_dict(cls, raw: dict) -> "KisepelConfig":
        cls.require(raw)
        if not isinstance(raw["layers"], list) or not raw["layers"]:
            raise ConfigError("config key 'layers' must be a list of at least one layer")
        layers = []
        for i, entry in enumerate(raw["layers"]):
            where = f"layers[{i}]"
            kind = entry.get("type") if isinstance(entry, dict) else entry
            if kind not in MIXER_SIZES:
                raise UnsupportedError(f"{where}: mixer type {kind!r} is none of {', '.join(sorted(MIXER_SIZES))}")
            mlp = None
            if entry.get("mlp") is not None:
                mlp = TableExpertsSizes.read(_section(entry, "mlp", where), where + ".mlp")
            layers.append(KisepelLayer(kind, MIXER_SIZES[kind].read(_section(entry, "mixer", where), where + ".mixer"), mlp))
        start = stop = 0
        times = 1
        if raw.get("loop") is not None:
            loop = _section(raw, "loop", "config.json")
            start, stop = whole(loop.get("start"), "loop.start"), whole(loop.get("stop"), "loop.stop")
            times = whole(loop.get("times", 1), "loop.times", 1)
        embedding = _section(raw, "embedding", "config.json") if raw.get("embedding") is not None else {}
        cfg = cls(vocab=whole(raw["vocab"], "vocab", 1), width=whole(raw["width"], "width", 1), layers=tuple(layers),
                  norm_eps=f32(_section(raw, "norm", "config.json").get("eps"), "norm.eps"),
                  embedding_scale=f32(embedding.get("scale", 1.0), "embedding.scale"),
                  logit_scale=f32(raw.get("logit_scale", 1.0), "logit_scale"),
                  loop_start=start, loop_stop=stop, loop_times=times,
                  max_positions=whole(raw.get("max_positions", DEFAULT_MAX_POSITIONS), "max_positions", 1))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if not self.norm_eps >= 0.0:
            raise ConfigError(f"norm.eps {self.norm_eps} must not be negative")
        if not 0 <= self.loop_start <= self.loop_stop <= len(self.layers):
            raise ConfigError(f"loop {self.loop_start}..{self.loop_stop} does not lie inside the {len(self.layers)} layers")

    def order(self) -> list[tuple[int, bool]]:
        """The layers in the order they run, each with whether the embedding's output is added right before it: the looped
        stretch ``times`` times in a row, every pass but the first beginning with that sum."""
        n, a, b = len(self.layers), self.loop_start, self.loop_stop
        looped = [(i, turn > 0 and i == a) for turn in range(self.loop_times) for i in range(a, b)]
        return [(i, False) for i in range(a)] + looped + [(i, False) for i in range(b, n)]

    def to_dict(self) -> dict:
        out = {"architecture": self.ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "embedding": {"scale": self.embedding_scale}, "logit_scale": self.logit_scale,
               "layers": [layer.to_dict() for layer in self.layers]}
        if self.loop_times != 1 or self.loop_stop > self.loop_start:
            out["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out
