"""The configuration of the Gefudra decoder.

config.json names the design with ``"architecture": "Gefudra"`` and lists its layers: every entry of ``layers`` has a
``type`` (which mixer: ``latent_attention``, ``attention`` or ``wkv``), the mixer's sizes and constants (``mixer``) and its
feed-forward (``mlp``: ``{"kind": "dense", "ff": n, "limit": l}``, or null for none).  ``loop``: the layers ``start .. stop - 1`` run
``times`` times in a row with the same weights.  Beside them: ``vocab``, ``width``, ``norm.eps``, ``residual_mult`` and
``logit_scale``.  Every size and constant is read from here (the low rank of a ``wkv`` layer's decay is the shape of its tensor
``w1``); nothing is assumed equal to anything else from layer to layer.
"""
from __future__ import annotations

import dataclasses
from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .base import ConfigError, KeyReader

MIXERS = ("latent_attention", "attention", "wkv")
FEED_FORWARDS = ("dense",)


@dataclass(frozen=True)
class LatentAttention:
    """Attention without positions over one latent vector per token, queries through a latent of their own, with a sink."""
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    window: int = 0               # 0: every earlier token is seen


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int


@dataclass(frozen=True)
class DifferentialAttention:
    """Two attentions per head over the same values, the second taken off the first."""
    heads: int
    kv_heads: int
    dim: int                      # of one map's queries and keys
    vdim: int
    scale: float
    diff: float
    softcap: Optional[float] = None
    rot: Optional[Rotation] = None


@dataclass(frozen=True)
class TimeMixer:
    """The recurrent mixer with a decay per key channel."""
    heads: int
    dim: int
    rank: Optional[int] = None    # of the decay's projection; None: open until the tensors' shapes are known


@dataclass(frozen=True)
class FeedForward:
    ff: int
    limit: float


@dataclass(frozen=True)
class Loop:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class GefudraLayer:
    type: str
    mixer: Any                    # LatentAttention, DifferentialAttention or TimeMixer
    ff: Optional[FeedForward] = None


def _section(data: Dict[str, Any], key: str, where: str) -> Dict[str, Any]:
    v = data.get(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: required key {key!r} is missing or no object")
    return v


def _latent(m: KeyReader) -> LatentAttention:
    window = 0
    if m.data.get("mask") is not None:
        window = KeyReader(_section(m.data, "mask", m.where), m.where + ".mask").integer("size")
    dim = m.integer("dim")
    return LatentAttention(m.integer("heads"), dim, m.integer("vdim", default=dim), m.integer("kv_rank"), m.integer("q_rank"),
                           m.number("scale"), window)


def _differential(m: KeyReader) -> DifferentialAttention:
    heads = m.integer("heads")
    kv_heads = m.integer("kv_heads", default=heads)
    if heads % kv_heads:
        raise ConfigError(f"{m.where}: 'heads' {heads} is no multiple of 'kv_heads' {kv_heads}")
    dim = m.integer("dim")
    m.absent_or("mask", (), "this design's differential attention sees every earlier token")
    rot = None
    if m.data.get("rot") is not None:
        r = KeyReader(_section(m.data, "rot", m.where), m.where + ".rot")
        dims = r.integer("dims", default=dim, minimum=2)
        if dims % 2 or dims > dim:
            raise ConfigError(f"{r.where}: 'dims' {dims} must be even and at most 'dim' {dim}")
        rot = Rotation(r.number("base"), dims)
    return DifferentialAttention(heads, kv_heads, dim, m.integer("vdim", default=dim), m.number("scale"), m.number("diff", positive=False),
                                 m.number("softcap", default=None), rot)


def _time_mixer(m: KeyReader) -> TimeMixer:
    return TimeMixer(m.integer("heads"), m.integer("dim"), m.integer("rank", default=None))


_READERS = {"latent_attention": _latent, "attention": _differential, "wkv": _time_mixer}


@dataclass(frozen=True)
class GefudraConfig:
    vocab: int
    width: int
    layers: Tuple[GefudraLayer, ...]
    norm_eps: float
    residual_mult: float = 1.0
    logit_scale: float = 1.0
    loop: Optional[Loop] = None
    max_positions: int = 1 << 17            # the design sets no limit: this bounds the rotation tables and a request's block table
    eos_token_ids: Tuple[int, ...] = ()
    architecture: str = "Gefudra"

    @staticmethod
    def from_dict(data: Dict[str, Any], where: str = "config.json") -> "GefudraConfig":
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
            mixer = _READERS[kind](KeyReader(_section(entry, "mixer", at), at + ".mixer"))
            ff = None
            if entry.get("mlp") is not None:
                f = KeyReader(_section(entry, "mlp", at), at + ".mlp")
                if f.data.get("kind", "dense") not in FEED_FORWARDS:
                    raise ConfigError(f"{f.where}: 'kind' = {f.data.get('kind')!r} is no feed-forward of this design; known: {list(FEED_FORWARDS)}")
                ff = FeedForward(f.integer("ff"), f.number("limit"))
            out.append(GefudraLayer(kind, mixer, ff))
        loop = None
        if data.get("loop") is not None:
            l = KeyReader(_section(data, "loop", where), where + ": loop")
            loop = Loop(l.integer("start", minimum=0), l.integer("stop"), l.integer("times"))
            if not loop.start < loop.stop <= len(out):
                raise ConfigError(f"{l.where}: 'start' {loop.start} and 'stop' {loop.stop} name no run of the {len(out)} layers")
        norm = KeyReader(_section(data, "norm", where), where + ": norm")
        return GefudraConfig(vocab=r.integer("vocab"), width=r.integer("width"), layers=tuple(out), norm_eps=norm.number("eps"),
                             residual_mult=r.number("residual_mult", default=1.0, positive=False),
                             logit_scale=r.number("logit_scale", default=1.0, positive=False), loop=loop,
                             max_positions=r.integer("max_positions", default=1 << 17), eos_token_ids=r.token_ids("eos_token_id"))

    def to_dict(self) -> Dict[str, Any]:
        """The config.json that reads back as this configuration."""
        layers = []
        for layer in self.layers:
            m = layer.mixer
            if layer.type == "latent_attention":
                md: Dict[str, Any] = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "kv_rank": m.kv_rank, "q_rank": m.q_rank, "scale": m.scale}
                if m.window:
                    md["mask"] = {"size": m.window}
            elif layer.type == "attention":
                md = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale, "diff": m.diff}
                if m.softcap is not None:
                    md["softcap"] = m.softcap
                if m.rot is not None:
                    md["rot"] = {"base": m.rot.base, "dims": m.rot.dims}
            else:
                md = {"heads": m.heads, "dim": m.dim}
                if m.rank is not None:
                    md["rank"] = m.rank
            fd = None if layer.ff is None else {"kind": "dense", "ff": layer.ff.ff, "limit": layer.ff.limit}
            layers.append({"type": layer.type, "mixer": md, "mlp": fd})
        d: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "layers": layers,
                             "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult, "logit_scale": self.logit_scale,
                             "max_positions": self.max_positions}
        if self.loop is not None:
            d["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        if self.eos_token_ids:
            d["eos_token_id"] = list(self.eos_token_ids)
        return d


def complete_config(cfg: GefudraConfig, shapes: Dict[str, Tuple[int, ...]]) -> GefudraConfig:
    """``cfg`` with the sizes that config.json leaves to the tensors: a ``wkv`` layer's rank is the height of ``<layer>.mix.w1``.
    (A tensor that is missing leaves the size open; what the loader then reports names the tensor.)"""
    layers = []
    for i, layer in enumerate(cfg.layers):
        shape = shapes.get(f"l{i}.mix.w1")
        if layer.type == "wkv" and layer.mixer.rank is None and shape is not None and len(shape) == 2:
            layer = dataclasses.replace(layer, mixer=dataclasses.replace(layer.mixer, rank=int(shape[0])))
        layers.append(layer)
    return dataclasses.replace(cfg, layers=tuple(layers))
