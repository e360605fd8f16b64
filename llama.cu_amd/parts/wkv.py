"""A recurrent mixer whose state per head is a matrix with a decay per key channel that every token sets, a bonus for the
token's own key, and projections that read a mix of the token and the one before it.

With the mixer's input ``h`` (``h'``: the token before's, zeros in front of the first) and per head key channels ``i``:

    x_s = h + (h' - h) * mu_s                                  for each projection s of r, k, v, g, w
    r, k, v = W_r x_r, W_k x_k, W_v x_v                        (heads x dim each);   gate = silu(W_g x_g)
    w = exp(-exp(W_2 tanh(W_1 x_w) + w0))                      per head and key channel
    o = (S + diag(u) k v^T)^T r,     S <- diag(w) S + k v^T    the bonus u for the current token only
    out = W_o (o / rms(o) per head * norm * gate)

The block's norm hands over 32-bit rows, which are mixed in 32-bit and rounded once, as operands of the projections;
everything between those and ``W_o`` is 32-bit (``csrc/kernels/wkv.hip``).  Per request the engine's state slot holds ``S [heads,
dim, dim]`` and, behind it, the last token's ``h``; both count as zero at position 0.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..kernels import ops
from .base import BuildContext, Part, SlotState, TensorSpec, register_part
from .linear import GroupWeight, Weight, finish, linear, linear_groups


class WKV(Part):
    graph_safe = True
    reads_float32 = True         # the block's norm writes 32-bit rows for it
    ends_in_norm = True
    ends_in_planes = True

    # the tensors' names under the part's own; ``names`` replaces any
    NAMES = {"mu": "mu", "r": "r", "k": "k", "v": "v", "g": "g", "w1": "w1", "w2": "w2", "w0": "w0", "u": "u", "norm": "norm", "o": "o"}
    MIXES = ("r", "k", "v", "g", "w")            # the mixed rows, in the order in which they are made
    GROUP = ("r", "k", "v", "g")                 # the projections of one size

    def __init__(self, hidden_size: int, heads: int, head_dim: int, decay_rank: int, norm_eps: float,
                 names: Optional[Dict[str, str]] = None):
        self.hidden_size, self.heads, self.head_dim = int(hidden_size), int(heads), int(head_dim)
        self.decay_rank, self.norm_eps = int(decay_rank), float(norm_eps)
        if not 1 <= self.decay_rank <= 512:
            raise ValueError(f"wkv: the decay's low rank {decay_rank} is not supported (1 to 512)")
        if not 1 <= self.head_dim <= 256:
            raise ValueError(f"wkv: heads of {head_dim} are not supported (at most 256)")
        self.names = dict(self.NAMES, **(names or {}))
        self.inner = self.heads * self.head_dim
        # the state's matrices, filled up so that the last token's rows behind them start at a multiple of 16 bytes
        self.h_offset = (self.heads * self.head_dim * self.head_dim + 3) // 4 * 4

    def tensors(self) -> Dict[str, TensorSpec]:
        d, hd, rank, nm = self.hidden_size, self.inner, self.decay_rank, self.names
        t = {f"{nm['mu']}.{s}": TensorSpec((d,)) for s in self.MIXES}
        t.update({nm[s]: TensorSpec((hd, d)) for s in self.GROUP})
        t.update({nm["w1"]: TensorSpec((rank, d)), nm["w2"]: TensorSpec((hd, rank)), nm["w0"]: TensorSpec((hd,)),
                  nm["u"]: TensorSpec((self.heads, self.head_dim)), nm["norm"]: TensorSpec((hd,), init="one_plus_normal"),
                  nm["o"]: TensorSpec((d, hd))})
        return t

    def cache_need(self):
        return SlotState((self.h_offset + (self.hidden_size + 3) // 4 * 4,), torch.float32)

    def load(self, tensors, build: BuildContext) -> None:
        nm = self.names
        self.w_in = GroupWeight(torch.stack([tensors[nm[s]] for s in self.GROUP]), build)
        self.w1 = Weight(tensors[nm["w1"]], build)
        self.w_o = Weight(tensors[nm["o"]], build)
        f32 = lambda name: tensors[name].float().contiguous()
        # what enters the recurrence is 32-bit whatever the file holds
        self.mu = torch.stack([f32(f"{nm['mu']}.{s}") for s in self.MIXES]).contiguous()
        self.w2_t = f32(nm["w2"]).t().contiguous()                  # [rank, heads * dim]: the kernel's lanes read neighbours
        self.w0, self.u, self.norm = f32(nm["w0"]), f32(nm["u"]).reshape(-1).contiguous(), f32(nm["norm"])
        self.offsets = {s: i * self.inner for i, s in enumerate(self.GROUP)}
        self.dtype = build.dtype

    def forward(self, h, step, cache, into=None, planes_ok=False, out_dtype=None, state: Optional[torch.Tensor] = None):
        state = state if state is not None else cache.state
        if state is None:
            raise ops.KernelError("wkv: the layer was given no state slots")
        if h.dtype != torch.float32:
            h = h.float()
        mixed = ops.token_shift(h, self.mu, state, self.h_offset, step, self.dtype)
        n = h.shape[0]
        rows = torch.empty((n, len(self.GROUP) * self.inner), dtype=self.dtype, device=h.device)
        rows = linear_groups(mixed[:len(self.GROUP)], self.w_in, rows)
        low = linear(mixed[len(self.GROUP)], self.w1, out_dtype=torch.float32)
        y = ops.wkv(rows, self.offsets, low, self.w2_t, self.w0, self.u, self.norm, state, step, self.heads, self.head_dim,
                    self.norm_eps, self.dtype)
        return finish(y, self.w_o, self.dtype, into=into, planes_ok=planes_ok, out_dtype=out_dtype)


register_part("mixer", "wkv", WKV)
