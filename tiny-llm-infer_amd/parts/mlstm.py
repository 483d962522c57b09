"""The matrix memory of the xLSTM (mLSTM): a recurrent mixer with exponential gates.

For the rows h_t of one sequence (H heads, key size dk, value size dv):

    q = Wq h / sqrt(dk),  k = Wk h   [H dk],    v = Wv h   [H dv]
    i = cap tanh((Wi h + bi) / cap),   f = logsigmoid(cap tanh((Wf h + bf) / cap))     one a head
    m_t = max(f + m_(t-1), i)                                                          m = 0 at first
    S_t = exp(f + m_(t-1) - m_t) S_(t-1) + exp(i - m_t) k v^T,   n_t likewise with k alone
    o_t = S_t^T q / (max(|n_t . q|, exp(-m_t)) + 1e-6)
    y = o / sqrt(mean(o^2) + eps) * w * sigmoid(Wg h)        the mean head by head, w over all heads' elements
    out = Wo y

S, n and m start at zero and are per-request state in float32; the gates (from their products'
float32 sums on), the recurrence, the norm and the output gate are float32.  Nothing is kept in the
paged cache."""
from __future__ import annotations

import math
from typing import Dict, List, Tuple

import torch

from ..cache.manager import StateNeed
from ..weights.loader import TensorDecl
from .base import BuildEnv, StepView, register_part
from .joined import SplitMixer


class MatrixLSTM(SplitMixer):
    def __init__(self, spec):
        super().__init__(spec)
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.heads = int(p["num_heads"])
        self.dk = int(p["key_dim"])
        self.dv = int(p["value_dim"])
        self.eps = float(p["norm_eps"])
        self.cap = float(p["gate_cap"])
        if self.cap <= 0.0:
            raise ValueError("the gates' cap must be positive")

    def inputs(self) -> List[Tuple[str, int]]:
        return [("q", self.heads * self.dk), ("k", self.heads * self.dk), ("v", self.heads * self.dv), ("gate", self.heads * self.dv)]

    @property
    def rows_width(self) -> int:
        return self.heads * self.dv

    def tensors(self) -> List[TensorDecl]:
        n = self.spec.names
        gates = [TensorDecl(n[r], (self.heads, self.hidden)) for r in ("i", "f")] + \
            [TensorDecl(n["i_bias"], (self.heads,), "normal(0.0,0.5)"), TensorDecl(n["f_bias"], (self.heads,), "normal(3.0,1.0)")]
        return [TensorDecl(n[r], (size, self.hidden)) for r, size in self.inputs()] + gates + \
            [TensorDecl(n["norm"], (self.rows_width,), "ones_normal"), TensorDecl(n["o"], (self.hidden, self.rows_width))]

    def load_between(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load_between(weights, env)
        n = self.spec.names
        env.ops.check_lightning_sizes(self.heads, self.dk, self.dv)
        self.w_gates = torch.cat([weights[n[r]].to(env.dtype) for r in ("i", "f")]).contiguous()      # few rows: kept row-major
        self.gate_bias = torch.cat([weights[n[r]].to(torch.float32) for r in ("i_bias", "f_bias")]).contiguous()
        self.norm = weights[n["norm"]].to(torch.float32).contiguous()

    def state_need(self):
        return {"S": StateNeed(tuple(self.env.ops.mlstm_state_shape(self.heads, self.dk, self.dv)), torch.float32),
                "m": StateNeed((self.heads,), torch.float32)}

    def workspace_elems(self, rows: int) -> int:
        qk, v = self.heads * self.dk, self.heads * self.dv
        return rows * (2 * qk + 2 * v + max(2 * (4 * qk + 2 * v) + 2 * v + v, qk * (self.dv + 1) // 32) + 8 * self.heads)

    def between(self, x, proj, at, step: StepView, out, out_at, scale) -> None:
        self.env.ops.mlstm(proj, at, x, self.w_gates, self.gate_bias, self.cap, step.state["S"], step.state["m"], step,
                           self.heads, self.dk, self.dv, 1.0 / math.sqrt(self.dk), self.norm, self.eps, scale, out, out_at)


register_part("mixer", "mlstm", MatrixLSTM)
