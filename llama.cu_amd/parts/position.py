"""Position encodings of the attention mixer.

A position encoding tells the attention mixer how queries and keys depend on a
token's place.  The interface:

  ``load(build)``                       make tables on the device
  ``rotary_tables() -> (cos, sin, rot_dim, pairing) or None``
        if not None, the mixer applies the rotation in the same kernel that writes
        keys and values to the cache;
  ``apply(qkv, positions, heads, kv_heads, head_dim)``
        any other change of queries and keys, in place, before the cache write
        (the default does nothing);
  ``score_slopes() -> float32 [heads] or None``
        a bias inside the scores that grows with the distance between key and query
        (the default: none).
"""
from __future__ import annotations

import weakref

import numpy as np
import torch

from .base import BuildContext, Part, register_part


class NoPosition(Part):
    graph_safe = True

    """Queries and keys are used as they are."""

    def load(self, tensors, build: BuildContext) -> None:
        pass

    def score_slopes(self):
        """None, or float32 [heads] on the device: the encoding is (also) a bias inside the scores,
        ``slope[h] * (key position - query position)`` added to the scaled score.  The mixer hands it to
        the attention kernel (the generic one: the matrix-core kernels take no bias)."""
        return None


class _Tables:
    """The cosine and sine tables of one (theta, rotated dims, positions) on one device."""

    def __init__(self, cos: torch.Tensor, sin: torch.Tensor):
        self.cos, self.sin = cos, sin


# The tables depend on (theta, rotated dims, positions, device, scaling) alone, so the layers of a model that agree in
# these share one pair: 32 layers at 131,072 positions would else build and hold 32 x 67 MB.  The table lives as
# long as a part holds it.
_tables: "weakref.WeakValueDictionary" = weakref.WeakValueDictionary()


class Rotary(NoPosition):
    """Rotation of pairs of dims by ``pos * theta^(-2i/rot_dim)``.

    The tables follow llama.cu/src/model/mod.rs:200-209: the frequency
    ``theta^(-2i/dh)`` and the angle ``pos * freq`` are 32-bit values; the table holds
    the sine and cosine of that 32-bit angle (taken in 64-bit, rounded once).  The
    pairing is a parameter: ``interleaved`` pairs neighbours ``(2i, 2i+1)`` as
    llama.cu/src/op/rope.cuh:21-34 does; otherwise ``(i, i + rot_dim/2)``, the order in
    which files with config.json's tensor names hold the rows of q and k.
    """

    def __init__(self, head_dim: int, theta: float, max_positions: int, interleaved: bool = False,
                 rot_dim: int = 0, scaling_factor: float = 1.0, yarn=None):
        """``scaling_factor``: linear scaling, every frequency is divided by it (in 32-bit).  ``yarn`` (``{"factor", "original", "fast",
        "slow"}``): frequencies blended between themselves and themselves divided by ``factor``.  The pair whose angle makes ``t`` turns
        in ``original`` positions is ``pair(t) = rot_dim ln(original / (2 pi t)) / (2 ln theta)``; pairs up to ``floor(pair(fast))`` keep their
        frequency, pairs from ``ceil(pair(slow))`` on have it divided, in between the share is linear; cosine and sine are multiplied by ``0.1
        ln(factor) + 1``."""
        self.yarn = None if yarn is None else tuple(float(yarn[k]) for k in ("factor", "original", "fast", "slow"))
        if self.yarn is not None and (min(self.yarn) <= 0 or float(theta) in (0.0, 1.0) or float(scaling_factor) != 1.0):
            raise ValueError(f"rotary: blended frequencies {yarn} need positive numbers, a base that is not 1 and no other scaling")
        self.head_dim = int(head_dim)
        self.scaling_factor = float(scaling_factor)
        if not self.scaling_factor > 0:
            raise ValueError(f"rotary: the scaling factor {scaling_factor} must be positive")
        self.rot_dim = int(rot_dim) if rot_dim else int(head_dim)
        if self.rot_dim % 2 or self.rot_dim > self.head_dim:
            raise ValueError(f"rotary: rot_dim {self.rot_dim} must be even and at most head_dim {self.head_dim}")
        self.theta = float(theta)
        self.max_positions = int(max_positions)
        self.interleaved = bool(interleaved)
        self.cos = self.sin = None

    def yarn_frequencies(self):
        """(frequencies [rot_dim / 2] in 64-bit, the factor on cosine and sine)"""
        factor, original, fast, slow = self.yarn

        def pair(turns):
            return self.rot_dim * np.log(original / (2.0 * np.pi * turns)) / (2.0 * np.log(self.theta))

        i = np.arange(self.rot_dim // 2, dtype=np.float64)
        freq = np.power(self.theta, -2.0 * i / self.rot_dim)
        low, high = max(np.floor(pair(fast)), 0.0), min(np.ceil(pair(slow)), self.rot_dim - 1.0)
        share = np.clip((i - low) / max(high - low, 0.001), 0.0, 1.0)
        return freq / factor * share + freq * (1.0 - share), 0.1 * np.log(factor) + 1.0

    def host_tables(self):
        half = self.rot_dim // 2
        if self.yarn is not None:               # in 64-bit, rounded once
            freq, size = self.yarn_frequencies()
            ang = np.arange(self.max_positions, dtype=np.float64)[:, None] * freq[None, :]
            return (size * np.cos(ang)).astype(np.float32), (size * np.sin(ang)).astype(np.float32)
        # 32-bit throughout, as the reference: theta.powf(-((2 * i) as f32 / dh as f32))
        expo = -(np.float32(2.0) * np.arange(half, dtype=np.float32) / np.float32(self.rot_dim))
        freq = np.power(np.float32(self.theta), expo.astype(np.float32)).astype(np.float32)
        if self.scaling_factor != 1.0:
            freq = (freq / np.float32(self.scaling_factor)).astype(np.float32)
        pos = np.arange(self.max_positions, dtype=np.float32)
        ang = (pos[:, None] * freq[None, :]).astype(np.float32).astype(np.float64)   # the 32-bit product
        return np.cos(ang).astype(np.float32), np.sin(ang).astype(np.float32)

    def load(self, tensors, build: BuildContext) -> None:
        key = (self.theta, self.rot_dim, self.max_positions, str(torch.device(build.device)), self.scaling_factor, self.yarn)
        tables = _tables.get(key)
        if tables is None:
            cos, sin = self.host_tables()
            tables = _tables[key] = _Tables(torch.from_numpy(cos).to(build.device).contiguous(),
                                            torch.from_numpy(sin).to(build.device).contiguous())
        self._tables = tables                  # keeps the shared pair alive
        self.cos, self.sin = tables.cos, tables.sin

    def rotary_tables(self):
        return self.cos, self.sin, self.rot_dim, 1 if self.interleaved else 0

    def rotated_dims(self) -> int:
        return self.rot_dim


class DistanceBias(NoPosition):
    """No change of queries and keys: the scaled score of key ``j`` for the query at ``i`` of head ``h`` is lowered
    by ``slope[h] * (i - j)`` with ``slope[h] = 2^(-exponent * (h + 1) / heads)``, ``h = 0 .. heads - 1``."""

    def __init__(self, heads: int, exponent: float = 8.0):
        self.heads, self.exponent = int(heads), float(exponent)
        self.slopes = None

    def host_slopes(self):
        return np.array([2.0 ** (-self.exponent * (h + 1) / self.heads) for h in range(self.heads)], dtype=np.float32)

    def load(self, tensors, build: BuildContext) -> None:
        self.slopes = torch.from_numpy(self.host_slopes()).to(build.device).contiguous()

    def score_slopes(self):
        return self.slopes


register_part("position", "none", NoPosition)
register_part("position", "distance_bias", DistanceBias)
register_part("position", "rotary", Rotary)
