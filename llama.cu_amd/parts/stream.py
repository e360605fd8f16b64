"""Changes of the residual stream between two layers, named by entries of the run order (``RunEntry.before``).

``remix``: ``x <- W [x, x0]``, ``x0`` the embedding's output: what a group of layers that runs several times in a row with the
same weights reads before each of its runs.  The product reads both halves in the compute type and leaves a 32-bit
stream; the last branch's output is added to ``x`` in the kernel that writes its half of the operand.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import BuildContext, Part, TensorSpec, register_part
from .linear import Weight, linear


class Remix(Part):
    graph_safe = True
    takes_planes = True

    def __init__(self, hidden_size: int, tensor: str = "weight", delta_scale: float = 1.0):
        """``tensor``: the matrix ``[width, 2 width]`` (the stream's columns first); ``delta_scale``: what a branch's output is
        multiplied by before it is added to the stream."""
        self.hidden_size, self.tensor, self.delta_scale = int(hidden_size), str(tensor), float(delta_scale)
        self.weight = None

    def tensors(self):
        return {self.tensor: TensorSpec((self.hidden_size, 2 * self.hidden_size))}

    def load(self, tensors, build: BuildContext) -> None:
        self.weight = Weight(tensors[self.tensor], build)
        self.dtype = build.dtype

    def begin(self, x: torch.Tensor) -> torch.Tensor:
        """The operand ``[n, 2 width]`` with the embedding's output in its right half."""
        both = torch.empty((x.shape[0], 2 * self.hidden_size), dtype=self.dtype, device=x.device)
        ops.stream_rows(x, both[:, self.hidden_size:])
        return both

    def forward(self, x: torch.Tensor, pending, both: torch.Tensor) -> torch.Tensor:
        """The new stream; ``pending``: the last branch's output, not yet added to ``x`` (rows or planes, or None)."""
        ops.stream_rows(x, both[:, :self.hidden_size], delta=pending, delta_scale=self.delta_scale)
        return linear(both, self.weight, out_dtype=torch.float32)


register_part("stream", "remix", Remix)
