"""Rotary position encoding, half-split ("neox") pairing.

Frequencies f_i = theta^(-2i/d) for i < d/2, computed in float32 with the
exponent -2.0f*i/d in float32; angle = float32(position) * f_i in float32
(kernels/src/rope_kernel_cpu.cpp:127-141).  The pair (x_i, x_{i+d/2}) becomes
(x_i cos - x_{i+d/2} sin, x_i sin + x_{i+d/2} cos)
(kernels/src/rope_kernel_cpu.cpp:156-179).  ``rotary_dim`` = d may be smaller
than the head size; the rest of the head is left as it is.  The table holds
sin and cos of the float32 angle, evaluated in float64 and rounded once.

"rope_interleaved" is the same table for an encoding whose pair i is the neighbours
(2i, 2i + 1); the mixer that applies it is told so by ``RotaryTables.pairing``.

``scaling_factor`` c (linear scaling): every f_i is divided by c.  ``angles`` "float64": frequencies
and angles in float64 too, so that the table's entries are the exact ones rounded once; the default
"float32" is the reference's.
"""
from __future__ import annotations

import numpy as np
import torch

from .base import BuildEnv, PositionEncoding, RotaryTables, register_part


class NeoxRope(PositionEncoding):
    def __init__(self, spec):
        super().__init__(spec)
        p = spec.params
        self.head_dim = int(p["head_dim"])
        self.rotary_dim = int(p.get("rotary_dim", self.head_dim))
        self.theta = float(p["theta"])
        self.max_positions = int(p["max_positions"])
        self.scaling_factor = float(p.get("scaling_factor") or 1.0)
        self.exact = {"float32": False, "float64": True}[p.get("angles", "float32")]
        if self.scaling_factor <= 0.0:
            raise ValueError("a rotation's scaling factor must be positive")
        if self.rotary_dim % 2 or self.rotary_dim > self.head_dim or self.rotary_dim <= 0:
            raise ValueError(f"rotary_dim {self.rotary_dim} must be even and at most head_dim {self.head_dim}")
        self.cos = None
        self.sin = None

    def load(self, weights, env: BuildEnv) -> None:
        super().load(weights, env)
        n = min(self.max_positions, env.max_model_len)
        self.num_positions = n
        key = ("rope_neox", self.theta, self.rotary_dim, n, str(env.device), self.scaling_factor, self.exact)
        if key in env.shared:                 # layers with the same angles share one table
            self.cos, self.sin = env.shared[key]
            return
        half = self.rotary_dim // 2
        real = np.float64 if self.exact else np.float32
        i = np.arange(half, dtype=real)
        exponent = (real(-2.0) * i) / real(self.rotary_dim)
        freq = np.power(real(self.theta), exponent, dtype=real)
        if self.scaling_factor != 1.0:
            freq = freq / real(self.scaling_factor)
        pos = np.arange(n, dtype=real)
        angle = (pos[:, None] * freq[None, :]).astype(real)
        a64 = angle.astype(np.float64)
        self.cos = torch.from_numpy(np.cos(a64).astype(np.float32)).to(env.device).contiguous()
        self.sin = torch.from_numpy(np.sin(a64).astype(np.float32)).to(env.device).contiguous()
        env.shared[key] = (self.cos, self.sin)

    def rotary(self) -> RotaryTables:
        return RotaryTables(self.cos, self.sin, self.rotary_dim, "half")


class InterleavedRope(NeoxRope):
    def rotary(self) -> RotaryTables:
        return RotaryTables(self.cos, self.sin, self.rotary_dim, "interleaved")


register_part("position", "rope_neox", NeoxRope)
register_part("position", "rope_interleaved", InterleavedRope)
