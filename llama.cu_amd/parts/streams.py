"""Several residual streams instead of one (``x [n, streams * width]`` float32, a row's streams side by side).

A sublayer reads a weighted sum of the streams and writes through a matrix between them and a weight per stream:

    u = sum_s in[s] x_s,   y = f(norm(u)),   x_t <- sum_s mix[s, t] x_s + out[t] y        (all t at once from the old x)

``StreamsNorm`` makes ``norm(u)`` (without ``in``: of the sum of the streams, behind the last sublayer) and on its way there lets the
last sublayer's output into the streams: ``pending`` between these parts is a ``StreamUpdate``, the output with the matrix and the weights
that it enters by, and the one kernel (``ops.streams_norm``) reads and writes every stream once between two sublayers.  ``StreamsBlock``
is the arrangement of a mixer and a feed-forward in one layer.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..kernels import ops
from .base import BuildContext, Part, PartSpec, StreamUpdate, TensorSpec, make_part, register_part
from .block import _SublayersInTurn


class StreamsNorm(Part):
    """RMS norm of a weighted sum of the streams.  ``tensor``, ``one_plus``: as ``rmsnorm``."""
    graph_safe = True
    takes_planes = True

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


class StreamsBlock(_SublayersInTurn):
    """A mixer and a feed-forward (which may be missing, with its norm) between several residual streams.  ``connections``: under
    which names the two sublayers' tensors ``in [streams]``, ``out [streams]`` and ``mix [streams, streams]`` (from, to) lie."""

    CHILDREN = ("norm1", "mixer", "norm2", "ffn")
    takes_planes = True          # ``pending``'s output may be float32 planes of partial sums
    ends_in_planes = True        # forward takes ``planes_ok``

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

    def forward(self, x: torch.Tensor, pending, step, cache, next_norm=None, planes_ok=False):
        first = self.connections[0]
        h = self.norm1.forward(x, pending, first["in"])
        later = {"planes_ok": True} if self.mixer.ends_in_planes and (self.ffn is not None or planes_ok) else {}
        pending = StreamUpdate(self.mixer.forward(h, step, cache, **later), first["mix"], first["out"])
        if self.ffn is None:
            return pending
        second = self.connections[1]
        h = self.norm2.forward(x, pending, second["in"])
        later = {"planes_ok": True} if planes_ok and self.ffn.ends_in_planes else {}
        return StreamUpdate(self.ffn.forward(h, **later), second["mix"], second["out"])


register_part("norm", "streams_rmsnorm", StreamsNorm)
register_part("block", "streams", StreamsBlock)
