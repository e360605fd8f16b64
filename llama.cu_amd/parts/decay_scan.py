"""Linear attention with one decay per head and token: two mixers over the same kernels (``ops.decay_scan``).

Both keep a 32-bit matrix ``S [head_dim, value_dim]`` per head in the engine's state slots, zero at a request's position 0 and
carried from step to step, and let ``S <- a S + b k v^T``, ``o = S^T q``.

``lightning`` (a fixed decay):    q, k, v = silu(W h);  a = decay[head], b = 1
                                  out = W_o (o / rms(o over all heads) * norm * sigmoid(W_g h))
``matrix_memory`` (exponential    q = head_dim^(-1/2) W_q h;  i = cap tanh((W_i h + b_i) / cap), f = log sigmoid(cap tanh((W_f h + b_f) / cap))
gates, mLSTM):                    m = max(f + m', i);  a = exp(f + m' - m), b = exp(i - m);  n <- a n + b k
                                  y = o / (max(|n . q|, exp(-m)) + 1e-6);  out = W_o (y / rms(y per head) * norm * sigmoid(W_g h))

Everything between the input products and the output product is 32-bit but q, k and v, which are the input product's (and silu's)
output in the compute type.  Both can hand the rows that their output product would multiply to a mixer that multiplies several mixers' rows at once
(``splits_output``).
"""
from __future__ import annotations

import math
from typing import Dict, Optional, Sequence

import torch

from ..kernels import ops
from ..weights.loader import fused_rows
from .base import BuildContext, Part, ScaledRows, SlotState, StreamsEnd, TensorSpec, register_part
from .linear import Weight, end_in_norm, finish, linear_scaled, project, skinny_takes


class _DecayScan(Part):
    graph_safe = True
    splits_output = True
    ends_in_planes = True
    ends_in_norm = True
    GATED = False
    IN = ()                       # the input matrices, in the order of their rows in the one product

    def _sizes(self, what: str, hidden_size: int, heads: int, head_dim: int, value_dim: int, norm_eps: float, names) -> None:
        self.hidden_size, self.heads, self.head_dim, self.value_dim = int(hidden_size), int(heads), int(head_dim), int(value_dim)
        if self.head_dim > 256 or self.value_dim > 512:
            raise ValueError(f"{what}: heads of {head_dim} (values {value_dim}) are not supported by the kernels (at most 256 and 512)")
        self.norm_eps = float(norm_eps)
        self.names = dict(self.NAMES, **(names or {}))
        hk, hv = self.heads * self.head_dim, self.heads * self.value_dim
        self.offsets = {"q": 0, "k": hk, "v": 2 * hk, "g": 2 * hk + hv}
        self.in_rows = 2 * hk + 2 * hv
        self.output_width = hv
        self.w_in = self.w_o = self.output_matrix = None

    def tensors(self) -> Dict[str, TensorSpec]:
        d, hk, hv, nm = self.hidden_size, self.heads * self.head_dim, self.heads * self.value_dim, self.names
        return {nm["q"]: TensorSpec((hk, d)), nm["k"]: TensorSpec((hk, d)), nm["v"]: TensorSpec((hv, d)), nm["g"]: TensorSpec((hv, d)),
                nm["o"]: TensorSpec((d, hv)), nm["norm"]: TensorSpec((hv,), init="one_plus_normal")}

    def fused_groups(self, dtype, device):
        return [(tuple(self.names[k] for k in self.IN), 0)]

    def cache_need(self):
        return SlotState((ops.decay_state_floats(self.heads, self.head_dim, self.value_dim, self.GATED),), torch.float32)

    def load(self, tensors, build: BuildContext) -> None:
        nm = self.names
        self.w_in = Weight(fused_rows([tensors[nm[k]] for k in self.IN]), build)
        self.weight = tensors[nm["norm"]].float().contiguous()
        self.output_matrix = tensors[nm["o"]]
        self.w_o = Weight(self.output_matrix, build) if self.own_output else None
        self.dtype = build.dtype

    def _state(self, cache, state):
        state = state if state is not None else cache.state
        if state is None:
            raise ops.KernelError("decay scan: the layer was given no state slots")
        return state

    def takes_scaled_rows(self, n_rows: int) -> bool:
        return self.dtype == torch.bfloat16 and n_rows <= ops.ADD_NORM_MAX_ROWS and skinny_takes(n_rows, self.w_in, preferred=True)

    def _operand(self, h):
        rows = h.rows if isinstance(h, ScaledRows) else h
        return torch.empty((rows.shape[0], self.output_width), dtype=self.dtype, device=rows.device)

    def forward(self, h, step, cache, out_dtype=None, planes_ok=False, into=None, state: Optional[torch.Tensor] = None):
        out = self._operand(h)
        self.forward_rows(h, step, cache, out, 1.0, state)
        return finish(out, self.w_o, self.dtype, into=into, planes_ok=planes_ok, out_dtype=out_dtype)


class Lightning(_DecayScan):
    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}
    IN = ("q", "k", "v", "g")

    def __init__(self, hidden_size: int, heads: int, head_dim: int, value_dim: int, decay: Sequence[float], norm_eps: float,
                 names: Optional[Dict[str, str]] = None):
        """``decay``: one factor per head."""
        self._sizes("lightning", hidden_size, heads, head_dim, value_dim, norm_eps, names)
        self.decay = [float(x) for x in decay]
        if len(self.decay) != self.heads or any(not x >= 0 for x in self.decay):
            raise ValueError(f"lightning: decays {list(decay)} for {self.heads} heads (one each, none below 0)")

    def load(self, tensors, build: BuildContext) -> None:
        super().load(tensors, build)
        # the logarithm in two 32-bit parts: a chunk's decays are exponentials of its multiples (a decay of 0 leaves nothing after one token)
        logs = [math.log(x) if x > 0 else -1.0e4 for x in self.decay]
        high = torch.tensor(logs, dtype=torch.float64).float()
        low = (torch.tensor(logs, dtype=torch.float64) - high.double()).float()
        self.log_decay = torch.stack([high, low], dim=1).contiguous().to(build.device)
        self.decay_vec = torch.tensor(self.decay, dtype=torch.float32, device=build.device)

    def _scan(self, h, step, cache, out, factor, state, scaled_rows=False):
        rows = project(h, self.w_in, self.dtype)
        return ops.decay_scan(rows, self.offsets, self._state(cache, state), step, self.heads, self.head_dim, self.value_dim, self.weight,
                              self.norm_eps, out, silu=True, factor=factor, decay=self.decay_vec, log_decay=self.log_decay, scaled_rows=scaled_rows)

    def forward_rows(self, h, step, cache, out, factor: float = 1.0, state: Optional[torch.Tensor] = None) -> None:
        self._scan(h, step, cache, out, factor, state)

    def forward(self, h, step, cache, out_dtype=None, planes_ok=False, into=None, state: Optional[torch.Tensor] = None):
        n = step.n
        if step.decode_only and self.dtype == torch.bfloat16 and out_dtype in (None, self.dtype) and n <= ops.ADD_NORM_MAX_ROWS \
                and skinny_takes(n, self.w_o, preferred=True):
            # few single tokens: the norm over the heads is a factor per row, which the output product applies
            out = self._operand(h)
            sumsq = self._scan(h, step, cache, out, 1.0, state, scaled_rows=True)
            scaled = ScaledRows(out, sumsq, self.output_width, self.norm_eps)
            fused = end_in_norm(scaled, self.w_o, into) if isinstance(into, StreamsEnd) else None
            return fused if fused is not None else linear_scaled(scaled, self.w_o, out_dtype=self.dtype)
        return super().forward(h, step, cache, out_dtype=out_dtype, planes_ok=planes_ok, into=into, state=state)


class MatrixMemory(_DecayScan):
    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm", "i": "i", "i_bias": "i.b", "f": "f", "f_bias": "f.b"}
    GATED = True
    IN = ("q", "k", "v", "g", "i", "f")

    def __init__(self, hidden_size: int, heads: int, head_dim: int, value_dim: int, gate_cap: float, norm_eps: float,
                 query_scale: Optional[float] = None, names: Optional[Dict[str, str]] = None):
        """``query_scale``: what the queries are multiplied by (default ``head_dim ** -0.5``)."""
        self._sizes("matrix memory", hidden_size, heads, head_dim, value_dim, norm_eps, names)
        self.gate_cap = float(gate_cap)
        if not self.gate_cap > 0:
            raise ValueError(f"matrix memory: the gates' cap {gate_cap} must be positive")
        self.query_scale = float(query_scale) if query_scale is not None else float(head_dim) ** -0.5

    def tensors(self) -> Dict[str, TensorSpec]:
        t, nm, nh = super().tensors(), self.names, self.heads
        t.update({nm["i"]: TensorSpec((nh, self.hidden_size)), nm["f"]: TensorSpec((nh, self.hidden_size)), nm["i_bias"]: TensorSpec((nh,)),
                  nm["f_bias"]: TensorSpec((nh,), init="one_plus_normal")})
        return t

    def load(self, tensors, build: BuildContext) -> None:
        super().load(tensors, build)
        nm = self.names
        self.gate_bias = (tensors[nm["i_bias"]].float().contiguous(), tensors[nm["f_bias"]].float().contiguous())
        # the product of many rows leaves q, k, v and g in the compute type and the gates' projections in 32-bit: two products of parts
        # of the one matrix
        self.w_rows, self.w_gates = self.w_in.plain[:self.in_rows], self.w_in.plain[self.in_rows:]

    def forward_rows(self, h, step, cache, out, factor: float = 1.0, state: Optional[torch.Tensor] = None) -> None:
        if step.decode_only or self.dtype == torch.float32:
            both = project(h, self.w_in, torch.float32)
            rows, gates = both[:, :self.in_rows], both[:, self.in_rows:]
        else:
            rows, gates = project(h, self.w_rows, self.dtype), project(h, self.w_gates, torch.float32)
        ops.decay_scan(rows, self.offsets, self._state(cache, state), step, self.heads, self.head_dim, self.value_dim, self.weight, self.norm_eps,
                       out, scale=self.query_scale, factor=factor, gates=gates, gate_bias=self.gate_bias, cap=self.gate_cap)


register_part("mixer", "lightning", Lightning)
register_part("mixer", "matrix_memory", MatrixMemory)
