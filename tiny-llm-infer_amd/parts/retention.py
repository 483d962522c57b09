"""Retention: linear attention with a fixed decay a head, rotated queries and keys and no softmax.

For the rows h_t of one sequence (H heads, key size dk, value size dv, one decay c_a a head from the
configuration):

    q = Wq h,  k = Wk h   [H dk],    v = Wv h   [H dv]                            (no biases)
    q, k turned by the position (``position``),  k <- k / sqrt(dk)
    per head:  S_t = c_a S_(t-1) + k_t v_t^T,    o_t = S_t^T q_t
    y = o / sqrt(mean(o^2) + eps) * silu(Wg h)       head by head, no weight
    out = Wo y

S [dk, dv] starts at zero and is per-request state in float32; rotation, recurrence, norm and gate
are float32.  Nothing is kept in the paged cache."""
from __future__ import annotations

import math
from typing import Dict, List, Tuple

import torch

from ..cache.manager import StateNeed
from ..weights.loader import TensorDecl
from .base import BuildEnv, RotaryTables, StepView, build_part, register_part
from .joined import SplitMixer


class Retention(SplitMixer):
    def __init__(self, spec):
        super().__init__(spec)
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.heads = int(p["num_heads"])
        self.dk = int(p["key_dim"])
        self.dv = int(p["value_dim"])
        self.eps = float(p["norm_eps"])
        self.decay_values = [float(c) for c in p["decay"]]
        if len(self.decay_values) != self.heads:
            raise ValueError(f"{len(self.decay_values)} decays for {self.heads} heads")
        self.position = build_part("position", spec.parts["position"]) if "position" in spec.parts else None

    def inputs(self) -> List[Tuple[str, int]]:
        return [("q", self.heads * self.dk), ("k", self.heads * self.dk), ("v", self.heads * self.dv), ("gate", self.heads * self.dv)]

    @property
    def rows_width(self) -> int:
        return self.heads * self.dv

    def tensors(self) -> List[TensorDecl]:
        n = self.spec.names
        return [TensorDecl(n[r], (size, self.hidden)) for r, size in self.inputs()] + \
            [TensorDecl(n["o"], (self.hidden, self.rows_width))] + (self.position.tensors() if self.position is not None else [])

    def load_between(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load_between(weights, env)
        env.ops.check_lightning_sizes(self.heads, self.dk, self.dv)
        self.rotary = None
        if self.position is not None:
            self.position.load(weights, env)
            tables = self.position.rotary()
            self.rotary = None if tables is None else RotaryTables(*tables)
            if self.rotary is not None and self.rotary.rotary_dim > self.dk:
                raise ValueError(f"{self.rotary.rotary_dim} turned elements do not fit a head of {self.dk}")
        self.decay = torch.tensor(self.decay_values, dtype=torch.float32, device=env.device)

    def state_need(self) -> StateNeed:
        return StateNeed(tuple(self.env.ops.lightning_state_shape(self.heads, self.dk, self.dv)), torch.float32)

    def workspace_elems(self, rows: int) -> int:
        # the projections, then q, k, v (padded at worst to twice their size) and o in float32, or the states before chunks of rows
        qk, v = self.heads * self.dk, self.heads * self.dv
        return rows * (2 * qk + 2 * v + max(2 * (4 * qk + 2 * v) + 2 * v + v, qk * self.dv // 32))

    def between(self, x, proj, at, step: StepView, out, out_at, scale) -> None:
        self.env.ops.retention(proj, at, self.decay, step.state, step, self.heads, self.dk, self.dv, self.rotary,
                               1.0 / math.sqrt(self.dk), self.eps, scale, out, out_at)


register_part("mixer", "retention", Retention)
