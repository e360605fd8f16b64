"""Several residual streams instead of one (``x [n, streams * width]`` float32, a row's streams side by side).

A sublayer reads a weighted sum of the streams and writes through a matrix between them and a weight per stream:

    u = sum_s in[s] x_s,   y = f(norm(u)),   x_t <- sum_s mix[s, t] x_s + out[t] y        (all t at once from the old x)

``StreamsNorm`` makes ``norm(u)`` (without ``in``: of the sum of the streams, behind the last sublayer) and on its way there lets the
last sublayer's output into the streams (a product of few rows may do both in its epilogue: ``StreamsEnd``): ``pending`` between these parts is a ``StreamUpdate``, the output with the matrix and the weights
that it enters by, and the one kernel (``ops.streams_norm``) reads and writes every stream once between two sublayers.  ``StreamsBlock``
is the arrangement of a mixer and a feed-forward in one layer.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional

import torch

from ..kernels import ops
from .base import BuildContext, Part, PartSpec, ScaledRows, StreamUpdate, StreamsEnd, TensorSpec, make_part, register_part
from .block import _SublayersInTurn


class StreamsNorm(Part):
    """RMS norm of a weighted sum of the streams.  ``tensor``, ``one_plus``: as ``rmsnorm``."""
    graph_safe = True
    takes_planes = True
    deferrable = True            # a product may end in it (``StreamsEnd``): a factor per row times a weight per column, of the weighted sum

    def __init__(self, size: int, eps: float, streams: int, tensor: str = "weight", one_plus: bool = False):
        self.size, self.eps, self.streams = int(size), float(eps), int(streams)
        if not 1 <= self.streams <= ops.STREAMS_MAX:
            raise ValueError(f"streams: {streams} residual streams are not supported (1 to {ops.STREAMS_MAX})")
        self.tensor, self.one_plus = str(tensor), bool(one_plus)
        self.weight = None

    def tensors(self) -> Dict[str, TensorSpec]:
        return {self.tensor: TensorSpec((self.size,), init="normal" if self.one_plus else "one_plus_normal")}

    def load(self, tensors, build: BuildContext) -> None:
        w = tensors[self.tensor].float()
        self.weight = (1.0 + w if self.one_plus else w).contiguous()
        self.dtype = build.dtype

    def forward(self, x: torch.Tensor, pending: Optional[StreamUpdate] = None, read: Optional[torch.Tensor] = None, write_back: bool = True):
        """``read``: the weights of the sum (None: ones)."""
        delta, mix, out = (pending.delta, pending.mix, pending.out) if pending is not None else (None, None, None)
        return ops.streams_norm(x, self.streams, self.weight, self.eps, self.dtype, delta=delta, mix=mix, out_weights=out, read=read,
                                write_back=write_back)


@dataclass(frozen=True)
class StreamsRead:
    """A norm with the weights that its sum of the streams is made with: what a block may end in."""
    norm: StreamsNorm
    read: Optional[torch.Tensor]


class StreamsBlock(_SublayersInTurn):
    """A mixer and a feed-forward (which may be missing, with its norm) between several residual streams.  ``connections``: under
    which names the two sublayers' tensors ``in [streams]``, ``out [streams]`` and ``mix [streams, streams]`` (from, to) lie."""

    CHILDREN = ("norm1", "mixer", "norm2", "ffn")
    takes_planes = True          # ``pending``'s output may be float32 planes of partial sums
    ends_in_planes = True        # forward takes ``planes_ok``
    ends_in_next_norm = True     # forward takes ``next_norm`` (a StreamsRead, or a StreamsNorm of the plain sum)

    def __init__(self, streams: int, norm1: PartSpec, mixer: PartSpec, norm2: Optional[PartSpec] = None, ffn: Optional[PartSpec] = None,
                 connections=("connection1", "connection2")):
        if (norm2 is None) != (ffn is None):
            raise ValueError("streams block: the second norm and the feed-forward come together or not at all")
        self.streams = int(streams)
        self.specs = {"norm1": norm1, "mixer": mixer, "norm2": norm2, "ffn": ffn}
        self.norm1 = make_part("norm", norm1)
        self.mixer = make_part("mixer", mixer)
        self.norm2 = make_part("norm", norm2) if norm2 is not None else None
        self.ffn = make_part("ffn", ffn) if ffn is not None else None
        for p in (self.norm1, self.norm2):
            if p is not None and p.streams != self.streams:
                raise ValueError(f"streams block: a norm of {p.streams} streams in a block of {self.streams}")
        self.names = tuple(connections)[:1 if ffn is None else 2]
        self.connections = []
        self.graph_safe = all(p.graph_safe for _, p in self._children())

    def tensors(self) -> Dict[str, TensorSpec]:
        out, s = super().tensors(), self.streams
        for name in self.names:
            # (a random model's streams are read, written and kept with weights around one)
            out.update({f"{name}.in": TensorSpec((s,), init="one_plus_normal"), f"{name}.out": TensorSpec((s,), init="one_plus_normal"),
                        f"{name}.mix": TensorSpec((s, s), init="identity_plus_normal")})
        return out

    def load(self, tensors, build: BuildContext) -> None:
        super().load(tensors, build)
        self.connections = [{k: tensors[f"{name}.{k}"].float().contiguous() for k in ("in", "out", "mix")} for name in self.names]

    @property
    def first_norm(self):
        return StreamsRead(self.norm1, self.connections[0]["in"])

    def takes_scaled_rows(self, n_rows: int) -> bool:
        """Whether ``pending`` may be ScaledRows of so many rows made with ``first_norm``."""
        return self.mixer.takes_scaled_rows(n_rows)

    def forward(self, x: torch.Tensor, pending, step, cache, next_norm=None, planes_ok=False):
        first = self.connections[0]
        h = pending if isinstance(pending, ScaledRows) else self.norm1.forward(x, pending, first["in"])
        n_rows = x.shape[0]
        inner = self.ffn is not None
        ahead = None if next_norm is None else next_norm if isinstance(next_norm, StreamsRead) else StreamsRead(next_norm, None)
        second = self.connections[1] if inner else None
        if inner:                # what the mixer may end in: the second norm, if the feed-forward takes such rows
            target = StreamsRead(self.norm2, second["in"]) if self.ffn.takes_scaled_rows(n_rows) else None
        else:
            target = ahead
        h = self._ended(x, self.mixer, (h, step, cache), target, inner or planes_ok, first)
        if not inner:
            return h
        if not isinstance(h, ScaledRows):
            h = self.norm2.forward(x, h, second["in"])
        return self._ended(x, self.ffn, (h,), ahead, planes_ok, second)

    @staticmethod
    def _ended(x, part, args, target: Optional[StreamsRead], planes_ok: bool, connection):
        """The output of ``part``: on its way into the streams (StreamUpdate), or, where its last product ended in the norm
        ``target``, in them already (ScaledRows)."""
        kw = {"planes_ok": True} if planes_ok and part.ends_in_planes else {}
        if target is not None and part.ends_in_norm:
            kw["into"] = StreamsEnd(x, target.norm, target.read, connection["mix"], connection["out"])
        out = part.forward(*args, **kw)
        return out if isinstance(out, ScaledRows) else StreamUpdate(out, connection["mix"], connection["out"])


register_part("norm", "streams_rmsnorm", StreamsNorm)
register_part("block", "streams", StreamsBlock)
