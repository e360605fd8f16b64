"""Differential attention: every head attends twice, with queries and keys of its own each time, over one set of values, and
the second result is taken off the first.

    q = W_q h, k = W_k h                    per head two maps of ``head_dim`` dims side by side;   v = W_v h
    a_m = causal softmax(score of map m) v, score = scale * rot(q_m) . rot(k_m), then softcap * tanh(score / softcap)
    lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff             one number for the layer, made at load in 32-bit
    o = a_1 - lambda a_2,   o <- o / rms(o) * (1 - diff)        per head, no weight
    out = W_o (heads * sigmoid(W_g h))

The paged attention kernels run it as plain attention, one head per (head, map) (``ops.qkv_prepare``).  Where both keys of a
head fit a head size of the matrix-core kernels side by side (``joint``), the cache holds them as one key beside the head's
values, and the query of a map has zeros at the other map's dims: a page holds every key and value once.  Else, where
one map's key and the values fit, every map is a stored head of its own with a copy of the values; what fits neither
way, and float32, goes to the generic kernel, joint.  Positions, angles, scores, softmax, the difference and its norm
are 32-bit.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..kernels import ops
from ..weights.loader import fused_rows
from .base import BuildContext, PagedKV, Part, PartSpec, TensorSpec, make_part, register_part
from .linear import Weight, finish, project, skinny_takes

MAPS = 2


class DifferentialAttention(Part):
    ends_in_norm = True
    ends_in_planes = True

    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "lq1": "lq1", "lk1": "lk1", "lq2": "lq2", "lk2": "lk2"}

    def __init__(self, hidden_size: int, heads: int, kv_heads: int, head_dim: int, value_dim: int, scale: float, diff: float,
                 norm_eps: float, softcap: float = 0.0, window: int = 0, position: Optional[PartSpec] = None, gate: bool = True,
                 page_size: int = 0, names: Optional[Dict[str, str]] = None):
        """``head_dim``: one map's query/key dims; ``diff``: the constant in lambda, and ``1 - diff`` behind the norm; ``gate``: an
        output gate of its own for every element (tensor ``g``)."""
        if heads % kv_heads:
            raise ValueError(f"differential attention: {heads} heads are no multiple of {kv_heads} key/value heads")
        self.hidden_size, self.heads, self.kv_heads = int(hidden_size), int(heads), int(kv_heads)
        self.head_dim, self.value_dim, self.scale = int(head_dim), int(value_dim), float(scale)
        self.diff, self.norm_eps, self.softcap, self.window = float(diff), float(norm_eps), float(softcap or 0.0), int(window or 0)
        if self.softcap < 0:
            raise ValueError(f"differential attention: the cap on the scores {softcap} must be positive (or 0 for none)")
        self.gate = bool(gate)
        self.own_page_size = int(page_size or 0)
        self.names = dict(self.NAMES, **(names or {}))
        self.position = make_part("position", position or PartSpec("none"))
        if self.position.score_slopes() is not None or type(self.position).apply is not Part.apply:
            raise ValueError("differential attention takes a rotation or no position encoding")
        self.graph_safe = self.position.graph_safe
        self.joint = True
        self.stored_dim, self.stored_value_dim = (MAPS * self.head_dim + 7) // 8 * 8, self.value_dim
        if max(self.stored_dim, self.value_dim) > ops.GENERIC_MAX_HEAD_DIM:
            raise ValueError(f"differential attention: two maps of {head_dim} or values of {value_dim} are more than the kernels take ({ops.GENERIC_MAX_HEAD_DIM})")
        self.page_size, self.dtype = 0, None

    def tensors(self) -> Dict[str, TensorSpec]:
        d, nm, hv = self.hidden_size, self.names, self.heads * self.value_dim
        t = {nm["q"]: TensorSpec((self.heads * MAPS * self.head_dim, d)), nm["k"]: TensorSpec((self.kv_heads * MAPS * self.head_dim, d)),
             nm["v"]: TensorSpec((self.kv_heads * self.value_dim, d)), nm["o"]: TensorSpec((d, hv))}
        if self.gate:
            t[nm["g"]] = TensorSpec((hv, d))
        t.update({nm[x]: TensorSpec((self.head_dim,)) for x in ("lq1", "lk1", "lq2", "lk2")})
        return t

    def _in_keys(self):
        return ("q", "k", "v") + (("g",) if self.gate else ())

    def fused_groups(self, dtype, device):
        return [(tuple(self.names[k] for k in self._in_keys()), 0)]

    # what the attention kernels see: a plain head per (head, map)
    @property
    def map_heads(self) -> int:
        return MAPS * self.heads

    @property
    def stored_heads(self) -> int:
        return self.kv_heads if self.joint else MAPS * self.kv_heads

    def cache_need(self):
        return PagedKV(self.stored_heads, self.stored_dim, self.window, self.own_page_size,
                       self.stored_value_dim if self.stored_value_dim != self.stored_dim else 0)

    def decode_splits(self, batch: int, max_ctx_len: int) -> int:
        return ops.decode_splits(batch, self.map_heads, self.stored_heads, max_ctx_len)

    def load(self, tensors, build: BuildContext) -> None:
        nm, nh, nkv, dh, dv = self.names, self.heads, self.kv_heads, self.head_dim, self.value_dim
        self.w_in = Weight(fused_rows([tensors[nm[k]] for k in self._in_keys()]), build)
        self.offsets = (0, nh * MAPS * dh, (nh + nkv) * MAPS * dh)
        self.g_off = (nh + nkv) * MAPS * dh + nkv * dv
        self.w_o = Weight(tensors[nm["o"]], build)
        l = {x: tensors[nm[x]].float() for x in ("lq1", "lk1", "lq2", "lk2")}
        self.lam = float(torch.exp((l["lq1"] * l["lk1"]).sum()) - torch.exp((l["lq2"] * l["lk2"]).sum()) + self.diff)
        self.page_size, self.dtype = build.page_size, build.dtype
        self.position.load({}, build)
        if build.dtype == torch.bfloat16:
            page = self.own_page_size or build.page_size
            for joint in (True, False):
                need = max(MAPS * dh if joint else dh, dv)
                for size in (32, 64, 96, 128):
                    if size >= need and ops.mfma_attention_refusal(build.dtype, MAPS * nh, nkv if joint else MAPS * nkv, size, page) is None:
                        self.joint, self.stored_dim, self.stored_value_dim = joint, size, size
                        return
            ops.say_once(f"differential attention with {nh} heads of two maps of {dh} (values {dv}) in {nkv} groups runs on the generic "
                         "kernel, not on the matrix cores")

    def _matrix_cores(self, page_size: int) -> bool:
        return (self.dtype == torch.bfloat16 and self.stored_value_dim == self.stored_dim
                and ops.mfma_attention_refusal(self.dtype, self.map_heads, self.stored_heads, self.stored_dim, page_size) is None)

    def prepare(self, step) -> None:
        if self._matrix_cores(self.own_page_size or self.page_size):
            ops.plan_attention(step, self.map_heads, self.stored_heads, self.window, capped=bool(self.softcap))

    def takes_scaled_rows(self, n_rows: int) -> bool:
        return self.dtype == torch.bfloat16 and n_rows <= ops.ADD_NORM_MAX_ROWS and skinny_takes(n_rows, self.w_in, preferred=True)

    def forward(self, h, step, cache, into=None, planes_ok=False, out_dtype=None):
        if not cache.writes:
            raise ops.KernelError("differential attention needs a cache of its own")
        nh, nkv = self.heads, self.kv_heads
        page_size = cache.page_size or self.page_size
        rot = self.position.rotary_tables()
        cos, sin, rot_dim, pairing = rot if rot is not None else (None, None, 0, 0)
        rows = project(h, self.w_in, self.dtype)
        q = ops.qkv_prepare(rows, self.offsets, MAPS * nh, MAPS * nkv, self.head_dim, self.value_dim, self.stored_dim, self.stored_value_dim,
                            self.dtype, positions=step.positions, cos=cos, sin=sin, rot_dim=rot_dim, pairing=pairing, cache=cache.pages,
                            slots=step.slots(cache.group), page_size=page_size, maps=MAPS, joint=self.joint)
        both = torch.empty((rows.shape[0], MAPS * nh * self.stored_value_dim), dtype=self.dtype, device=rows.device)
        ops.paged_attention(q, both, cache.pages, step, cache.group, self.map_heads, self.stored_heads, self.stored_dim, page_size,
                            self.scale, self.window, value_dim=self.stored_value_dim, force_generic=not self._matrix_cores(page_size),
                            softcap=self.softcap)
        gate = rows[:, self.g_off:self.g_off + nh * self.value_dim] if self.gate else None
        out = ops.two_maps(both, nh, self.value_dim, self.lam, self.norm_eps, 1.0 - self.diff, gate=gate,
                           head_stride=self.stored_value_dim, map_group=1 if self.joint else nh // nkv)
        return finish(out, self.w_o, self.dtype, into=into, planes_ok=planes_ok, out_dtype=out_dtype)


register_part("mixer", "differential_attention", DifferentialAttention)
