"""The configuration of the Lapunex decoder.

config.json names the design with ``"architecture": "Lapunex"`` and lists its layers: every entry of ``layers`` has a
``type`` (which mixer: ``parallel`` or ``lightning``), the mixer's sizes and constants (``mixer``) and its feed-forward (``mlp``:
``{"kind": "dense", "ff": n}``, ``{"kind": "moe", "expert": {...}, "router": {...}}``, or null for none).  ``loop``: the layers ``start
.. stop - 1`` run ``times`` times in a row with the same weights.  Beside them: ``vocab``, ``width``, ``streams`` (residual
streams), ``norm.eps`` and ``embedding.scale``.  Every size and constant is read from here; nothing is assumed equal to
anything else (heads and groups, key and value sizes, rotated dims, decays and experts differ from layer to layer).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple, Union

from .base import ConfigError, KeyReader

MIXERS = ("parallel", "lightning")
FEED_FORWARDS = ("dense", "moe")


@dataclass(frozen=True)
class Yarn:
    """Frequencies blended between the original ones and those of a context ``factor`` times as long."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int
    scaling: Optional[Yarn] = None


@dataclass(frozen=True)
class SoftmaxHalf:
    """The left half of ``parallel``: softmax attention over every earlier token, with a sink and a gate per head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[Rotation] = None


@dataclass(frozen=True)
class MatrixMemory:
    """The right half of ``parallel``: a matrix per head with exponential gates."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass(frozen=True)
class ParallelMixer:
    left: SoftmaxHalf
    right: MatrixMemory
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class Lightning:
    """Linear attention with a fixed decay per head."""
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class Dense:
    ff: int


@dataclass(frozen=True)
class Experts:
    ff: int                       # of one expert
    limit: float
    experts: int
    top: int
    scale: float = 1.0
    groups: int = 1
    keep: int = 1                 # groups that a token's experts may come from


@dataclass(frozen=True)
class Loop:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class LapunexLayer:
    type: str
    mixer: Union[ParallelMixer, Lightning]
    mlp: Union[Dense, Experts, None] = None


def _section(r: KeyReader, key: str) -> KeyReader:
    v = r.data.get(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{r.where}: required key {key!r} is missing or no object")
    return KeyReader(v, f"{r.where}.{key}")


def _rotation(m: KeyReader, dim: int) -> Optional[Rotation]:
    if m.data.get("rot") is None:
        return None
    r = _section(m, "rot")
    dims = r.integer("dims", default=dim, minimum=2)
    if dims % 2 or dims > dim:
        raise ConfigError(f"{r.where}: 'dims' {dims} must be even and at most 'dim' {dim}")
    base = r.number("base")
    scaling = None
    if r.data.get("scaling") is not None:
        s = _section(r, "scaling")
        scaling = Yarn(s.number("factor"), s.number("original"), s.number("fast"), s.number("slow"))
        if base == 1.0:
            raise ConfigError(f"{r.where}: with 'scaling' the 'base' must not be 1")
    return Rotation(base, dims, scaling)


def _softmax(m: KeyReader) -> SoftmaxHalf:
    heads = m.integer("heads")
    kv_heads = m.integer("kv_heads", default=heads)
    if heads % kv_heads:
        raise ConfigError(f"{m.where}: 'heads' {heads} is no multiple of 'kv_heads' {kv_heads}")
    dim = m.integer("dim")
    m.absent_or("mask", (), "this design's attention sees every earlier token")
    return SoftmaxHalf(heads, kv_heads, dim, m.integer("vdim", default=dim), m.number("scale", positive=False), _rotation(m, dim))


def _parallel(m: KeyReader) -> ParallelMixer:
    right = _section(m, "right")
    dim = right.integer("dim")
    memory = MatrixMemory(right.integer("heads"), dim, right.integer("vdim", default=dim), right.number("gate_cap"))
    return ParallelMixer(_softmax(_section(m, "left")), memory, m.number("left_scale", default=1.0, positive=False),
                         m.number("right_scale", default=1.0, positive=False))


def _lightning(m: KeyReader) -> Lightning:
    heads, dim = m.integer("heads"), m.integer("dim")
    decay = m.data.get("decay")
    if not isinstance(decay, list) or len(decay) != heads or any(isinstance(x, bool) or not isinstance(x, (int, float)) or not x >= 0 for x in decay):
        raise ConfigError(f"{m.where}: key 'decay' must list one number, not below 0, for each of the {heads} heads")
    return Lightning(heads, dim, m.integer("vdim", default=dim), tuple(float(x) for x in decay))


def _feed_forward(f: KeyReader) -> Union[Dense, Experts]:
    kind = f.data.get("kind", "dense")
    if kind == "dense":
        return Dense(f.integer("ff"))
    if kind != "moe":
        raise ConfigError(f"{f.where}: 'kind' = {kind!r} is no feed-forward of this design; known: {list(FEED_FORWARDS)}")
    e, r = _section(f, "expert"), _section(f, "router")
    experts, top, groups, keep = r.integer("experts"), r.integer("top"), 1, 1
    if r.data.get("groups") is not None:
        g = _section(r, "groups")
        groups, keep = g.integer("count"), g.integer("keep")
        if experts % groups or keep > groups:
            raise ConfigError(f"{g.where}: {experts} experts are no {groups} equal groups of which {keep} can be kept")
    if top > keep * (experts // groups):
        raise ConfigError(f"{r.where}: 'top' {top} is more than the {keep * (experts // groups)} experts that can be chosen")
    return Experts(e.integer("ff"), e.number("limit"), experts, top, r.number("scale", default=1.0, positive=False), groups, keep)


@dataclass(frozen=True)
class LapunexConfig:
    vocab: int
    width: int
    layers: Tuple[LapunexLayer, ...]
    norm_eps: float
    streams: int = 1
    embedding_scale: float = 1.0
    loop: Optional[Loop] = None
    max_positions: int = 1 << 17            # the design sets no limit: this bounds the rotation tables and a request's block table
    eos_token_ids: Tuple[int, ...] = ()
    architecture: str = "Lapunex"

    @staticmethod
    def from_dict(data: Dict[str, Any], where: str = "config.json") -> "LapunexConfig":
        r = KeyReader(data, where)
        layers = data.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError(f"{where}: required key 'layers' is missing or holds no layer")
        out = []
        for i, entry in enumerate(layers):
            at = f"{where}: layers[{i}]"
            if not isinstance(entry, dict):
                raise ConfigError(f"{at} is no object")
            kind = entry.get("type")
            if kind not in MIXERS:
                raise ConfigError(f"{at}: 'type' = {kind!r} is no mixer of this design; known: {list(MIXERS)}")
            e = KeyReader(entry, at)
            mixer = (_parallel if kind == "parallel" else _lightning)(_section(e, "mixer"))
            out.append(LapunexLayer(kind, mixer, None if entry.get("mlp") is None else _feed_forward(_section(e, "mlp"))))
        loop = None
        if data.get("loop") is not None:
            l = _section(r, "loop")
            loop = Loop(l.integer("start", minimum=0), l.integer("stop"), l.integer("times"))
            if not loop.start < loop.stop <= len(out):
                raise ConfigError(f"{l.where}: 'start' {loop.start} and 'stop' {loop.stop} name no run of the {len(out)} layers")
        scale = _section(r, "embedding").number("scale", default=1.0, positive=False) if data.get("embedding") is not None else 1.0
        return LapunexConfig(vocab=r.integer("vocab"), width=r.integer("width"), layers=tuple(out), norm_eps=_section(r, "norm").number("eps"),
                             streams=r.integer("streams", default=1), embedding_scale=scale, loop=loop,
                             max_positions=r.integer("max_positions", default=1 << 17), eos_token_ids=r.token_ids("eos_token_id"))

    def to_dict(self) -> Dict[str, Any]:
        """The config.json that reads back as this configuration."""
        layers = []
        for layer in self.layers:
            m = layer.mixer
            if layer.type == "parallel":
                a, b = m.left, m.right
                left: Dict[str, Any] = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale}
                if a.rot is not None:
                    left["rot"] = {"base": a.rot.base, "dims": a.rot.dims}
                    if a.rot.scaling is not None:
                        s = a.rot.scaling
                        left["rot"]["scaling"] = {"factor": s.factor, "original": s.original, "fast": s.fast, "slow": s.slow}
                md: Dict[str, Any] = {"left": left, "right": {"heads": b.heads, "dim": b.dim, "vdim": b.vdim, "gate_cap": b.gate_cap},
                                      "left_scale": m.left_scale, "right_scale": m.right_scale}
            else:
                md = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": list(m.decay)}
            f = layer.mlp
            fd: Optional[Dict[str, Any]] = None
            if isinstance(f, Dense):
                fd = {"kind": "dense", "ff": f.ff}
            elif f is not None:
                router: Dict[str, Any] = {"experts": f.experts, "top": f.top, "scale": f.scale}
                if f.groups > 1:
                    router["groups"] = {"count": f.groups, "keep": f.keep}
                fd = {"kind": "moe", "expert": {"ff": f.ff, "limit": f.limit}, "router": router}
            layers.append({"type": layer.type, "mixer": md, "mlp": fd})
        d: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "layers": layers,
                             "streams": self.streams, "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale},
                             "max_positions": self.max_positions}
        if self.loop is not None:
            d["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        if self.eos_token_ids:
            d["eos_token_id"] = list(self.eos_token_ids)
        return d
