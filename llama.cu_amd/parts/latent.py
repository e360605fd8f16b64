"""Latent attention: every token's keys and values of all heads are functions of one small latent vector and one
rotated key part, and only those two are cached.

    q_h = [q_plain, q_turned] = rows of W_q x               (per head: ``head_dim`` plain dims, then ``rot_dim`` turned ones)
    [c_raw, r_raw] = W_dkv x;  c = c_raw / rms(c_raw) * w;   r = rotate(r_raw, position)     (the cache holds [c, r])
    k_h = [W_uk_h c, r],  v_h = W_uv_h c;   softmax over the causal scores  scale * q_h . k_h;   out = W_o concat_h(...)

Each of the following is optional: the queries come through a latent of their own, ``q = W_uq (norm of W_dq x)`` (``q_rank``);
there are no turned parts, so attention knows no positions (``rot_dim`` 0); a window; a sink, ``exp(sink_h)`` in every
denominator of head ``h``; an output gate for every element, ``concat_h(...) * sigmoid(W_g x)``.

Computed in the folded form: ``q_plain . (W_uk_h c) = (W_uk_h^T q_plain) . c``, so all heads attend over ONE cached key
head ``[c, r]`` with the value ``c`` (the paged attention kernels, one key/value head, every query head in its group),
and ``W_uv_h`` is applied to the attention's output.  The two small products per head are ``linear_groups``: one
weight-streaming launch for few bfloat16 rows (the output gate in its epilogue), the library's batched product for
many, the engine's own 32-bit kernel, head by head, in float32.  Where queries come through a latent and nothing is
turned, ``W_uk_h^T W_uq_h`` is one matrix, and it is multiplied out at load (in 64-bit, rounded once) if a product with it is no
more work than the two: the queries' product then leaves folded queries.  A layer with ``shares_kv`` has no
``W_dkv``: it reads the cache of the layer named in the run order, with matrices, queries and scale of its own.
Positions, angles, the rotation, the latents' norms, scores and softmax are 32-bit.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..kernels import ops
from ..weights.loader import fused_rows
from .base import BuildContext, PagedKV, Part, PartSpec, TensorSpec, make_part, register_part
from .linear import GroupWeight, Weight, finish, linear, linear_groups, project, skinny_takes


class LatentAttention(Part):
    graph_safe = True
    ends_in_norm = True
    ends_in_planes = True

    NAMES = {"q": "q", "dq": "dq", "dq_norm": "dq.norm", "uq": "uq", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk", "uv": "uv",
             "sink": "sink", "g": "g", "o": "o"}

    def __init__(self, hidden_size: int, heads: int, head_dim: int, rot_dim: int, value_dim: int, kv_rank: int, scale: float,
                 theta: float = 0.0, max_positions: int = 0, norm_eps: float = 0.0, shares_kv: bool = False, page_size: int = 0,
                 names: Optional[Dict[str, str]] = None, q_rank: int = 0, window: int = 0, sink: bool = False, gate: bool = False):
        """``head_dim``: a head's query/key dims that are not rotated; ``rot_dim``: its rotated dims (dim ``i`` pairs with
        ``i + rot_dim / 2``, angle ``position * theta^(-2i / rot_dim)``; 0: none); ``kv_rank``: the latent's size; ``q_rank``: the
        queries' latent's (0: queries are a projection of the input); ``window``: a query sees so many keys up to its own
        (0: all); ``sink``, ``gate``: as above (tensors ``sink`` ``[heads]``, ``g`` ``[heads * value_dim, hidden]``)."""
        self.hidden_size, self.heads, self.head_dim = int(hidden_size), int(heads), int(head_dim)
        self.rot_dim, self.value_dim, self.kv_rank = int(rot_dim or 0), int(value_dim), int(kv_rank)
        if self.rot_dim < 0 or self.rot_dim % 2:
            raise ValueError(f"latent attention: rot_dim {rot_dim} must be even (or 0 for no turned part)")
        self.q_rank, self.window, self.sink, self.gate = int(q_rank or 0), int(window or 0), bool(sink), bool(gate)
        if self.q_rank and self.rot_dim:
            raise ValueError("latent attention: queries through a latent of their own go without a turned part")
        self.scale, self.norm_eps = float(scale), float(norm_eps)
        self.shares_kv = bool(shares_kv)
        self.own_page_size = int(page_size or 0)
        self.names = dict(self.NAMES, **(names or {}))
        self.position = None
        if self.rot_dim:
            self.position = make_part("position", PartSpec("rotary", {"head_dim": self.rot_dim, "theta": float(theta),
                                                                      "max_positions": int(max_positions)}))
        # what the one cached head takes: [c, r] filled up to a multiple of 8 dims; the value is c
        self.stored_dim = (self.kv_rank + self.rot_dim + 7) // 8 * 8
        self.stored_value_dim = self.kv_rank
        if self.stored_dim > ops.GENERIC_MAX_HEAD_DIM:
            raise ValueError(f"latent attention: kv_rank + rot_dim = {self.kv_rank + self.rot_dim} is more than the kernels take ({ops.GENERIC_MAX_HEAD_DIM})")
        self.page_size = 0
        self.dtype = None

    @property
    def q_width(self) -> int:
        """Columns of all heads' queries, before they are folded."""
        return self.heads * (self.head_dim + self.rot_dim)

    def tensors(self) -> Dict[str, TensorSpec]:
        d, nh, dn, dr, dv, rank, nm = self.hidden_size, self.heads, self.head_dim, self.rot_dim, self.value_dim, self.kv_rank, self.names
        t = {nm["uk"]: TensorSpec((nh * dn, rank)), nm["uv"]: TensorSpec((nh * dv, rank)), nm["o"]: TensorSpec((d, nh * dv))}
        if self.q_rank:
            t[nm["dq"]] = TensorSpec((self.q_rank, d))
            t[nm["dq_norm"]] = TensorSpec((self.q_rank,), init="one_plus_normal")
            t[nm["uq"]] = TensorSpec((self.q_width, self.q_rank))
        else:
            t[nm["q"]] = TensorSpec((self.q_width, d))
        if not self.shares_kv:
            t[nm["dkv"]] = TensorSpec((rank + dr, d))
            t[nm["dkv_norm"]] = TensorSpec((rank,), init="one_plus_normal")
        if self.sink:
            t[nm["sink"]] = TensorSpec((nh,))
        if self.gate:
            t[nm["g"]] = TensorSpec((nh * dv, d))
        return t

    def _in_keys(self):
        """The input's projections, in the order of their rows in the one product."""
        return ("dq" if self.q_rank else "q",) + (() if self.shares_kv else ("dkv",)) + (("g",) if self.gate else ())

    def fused_groups(self, dtype, device):
        keys = self._in_keys()
        return [(tuple(self.names[k] for k in keys), 0)] if len(keys) > 1 else []

    def cache_need(self):
        return PagedKV(1, self.stored_dim, self.window, self.own_page_size, self.stored_value_dim if self.stored_value_dim != self.stored_dim else 0)

    def decode_splits(self, batch: int, max_ctx_len: int) -> int:
        return ops.decode_splits(batch, self.heads, 1, max_ctx_len)

    def load(self, tensors, build: BuildContext) -> None:
        nm, nh, dn, dr, dv, rank = self.names, self.heads, self.head_dim, self.rot_dim, self.value_dim, self.kv_rank
        self.dtype, self.page_size = build.dtype, build.page_size
        f32 = lambda name: tensors[nm[name]].float().contiguous()
        if build.dtype == torch.bfloat16:
            # where a head size of the matrix-core kernels holds [c, r], key and value are both stored at that size (whatever
            # the layer's heads: a layer that reads this cache may have other heads, and must find the same sizes)
            for size in (32, 64, 96, 128):
                if size >= rank + dr and ops.mfma_attention_refusal(build.dtype, 1, 1, size, self.own_page_size or build.page_size) is None:
                    self.stored_dim = self.stored_value_dim = size
                    break
            if not self._matrix_cores(self.own_page_size or build.page_size):
                ops.say_once(f"latent attention with {nh} heads over a latent of {rank} + {dr} runs on the generic kernel, not on the matrix cores")
        keys = self._in_keys()
        mats = [tensors[nm[k]] for k in keys]
        self.w_in = Weight(fused_rows(mats) if len(mats) > 1 else mats[0], build)
        at = [0]
        for m in mats:
            at.append(at[-1] + m.shape[0])
        self.kv_off = at[1]                                                      # (not used by a layer that shares)
        self.g_off = at[len(keys) - 1]
        self.c_norm = None if self.shares_kv else f32("dkv_norm")
        self.sinks = f32("sink") if self.sink else None
        # per head the matrix that folds a query, [what a stored key takes, plain dims], and the values', [value dims, what a
        # stored value takes]: zeros at the dims of zeros (and at a turned part's place, which is written afterwards)
        fold = tensors[nm["uk"]].view(nh, dn, rank).transpose(1, 2)
        fold = torch.cat([fold, fold.new_zeros((nh, self.stored_dim - rank, dn))], dim=1) if self.stored_dim > rank else fold
        uv = tensors[nm["uv"]].view(nh, dv, rank)
        uv = torch.cat([uv, uv.new_zeros((nh, dv, self.stored_value_dim - rank))], dim=2) if self.stored_value_dim > rank else uv
        self.w_uv = GroupWeight(uv, build)
        self.w_uq = self.w_fold = self.w_folded_q = self.cq_norm = None
        if self.q_rank:
            self.cq_norm = f32("dq_norm")
            uq = tensors[nm["uq"]]
            if self.stored_dim * self.q_rank <= dn * (self.q_rank + self.stored_dim):
                folded = torch.bmm(fold.double().contiguous(), uq.view(nh, dn, self.q_rank).double().contiguous())
                self.w_folded_q = Weight(folded.to(uq.dtype).view(nh * self.stored_dim, self.q_rank), build)
            else:
                self.w_uq = Weight(uq, build)
        if self.w_folded_q is None:
            self.w_fold = GroupWeight(fold, build)
        self.w_o = Weight(tensors[nm["o"]], build)
        if self.position is not None:
            self.position.load({}, build)

    def _matrix_cores(self, page_size: int) -> bool:
        return (self.dtype == torch.bfloat16 and self.stored_value_dim == self.stored_dim and (not self.sink or self.scale > 0)
                and ops.mfma_attention_refusal(self.dtype, self.heads, 1, self.stored_dim, page_size) is None)

    def prepare(self, step) -> None:
        if self._matrix_cores(self.own_page_size or self.page_size):
            ops.plan_attention(step, self.heads, 1, self.window, biased=self.sink)

    def takes_scaled_rows(self, n_rows: int) -> bool:
        return self.dtype == torch.bfloat16 and n_rows <= ops.ADD_NORM_MAX_ROWS and skinny_takes(n_rows, self.w_in, preferred=True)

    def forward(self, h, step, cache, into=None, planes_ok=False, out_dtype=None):
        nh, dn, dr, dv, rank, dk, dvs = self.heads, self.head_dim, self.rot_dim, self.value_dim, self.kv_rank, self.stored_dim, self.stored_value_dim
        if self.shares_kv == cache.writes:
            raise ops.KernelError("latent attention: a layer that shares another's latent must be given that layer's cache in "
                                  "the run order (and only such a layer)")
        page_size = cache.page_size or self.page_size
        rows = project(h, self.w_in, self.dtype)
        n = rows.shape[0]
        store = not self.shares_kv
        into_cache = dict(c_norm=self.c_norm, eps=self.norm_eps, cache=cache.pages if store else None,
                          slots=step.slots(cache.group) if store else None, page_size=page_size)
        unturned = (nh, 0, 0, self.kv_off, rank, 0, dk, dvs, None, None, None)
        new = lambda width: torch.empty((n, width), dtype=self.dtype, device=rows.device)
        queries = rows                                                    # a row's first q_width columns are its queries
        if self.q_rank:                                                   # ... or its first q_rank columns their latent
            cq = new(self.q_rank)
            ops.latent_prepare(rows, None, *unturned, cq_off=0, cq_norm=self.cq_norm, cq_out=cq, **into_cache)
            queries = linear(cq, self.w_folded_q if self.w_folded_q is not None else self.w_uq, out_dtype=self.dtype)
        if self.w_folded_q is not None:
            q = queries
        else:
            q = linear_groups(queries[:, :self.q_width].view(n, nh, dn + dr)[:, :, :dn].permute(1, 0, 2), self.w_fold, new(nh * dk))
        if dr:
            cos, sin, _, _ = self.position.rotary_tables()
            ops.latent_prepare(rows, q, nh, dn + dr, dn, self.kv_off, rank, dr, dk, dvs, step.positions, cos, sin, **into_cache)
        elif not self.q_rank and store:
            ops.latent_prepare(rows, None, *unturned, **into_cache)
        mixed = new(nh * dvs)
        ops.paged_attention(q, mixed, cache.pages, step, cache.group, nh, 1, dk, page_size, self.scale, self.window,
                            value_dim=dvs, force_generic=not self._matrix_cores(page_size), sinks=self.sinks)
        gate = rows[:, self.g_off:self.g_off + nh * dv] if self.gate else None
        heads_out = linear_groups(mixed.view(n, nh, dvs).permute(1, 0, 2), self.w_uv, new(nh * dv), gate=gate)
        return finish(heads_out, self.w_o, self.dtype, into=into, planes_ok=planes_ok, out_dtype=out_dtype)


register_part("mixer", "latent_attention", LatentAttention)
