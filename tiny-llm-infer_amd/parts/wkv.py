"""The RWKV's time mixing: a recurrent mixer that keeps a matrix of state a head, which decays by a
number a channel and token, and the last row it read.

For the rows h_t of one sequence (H heads, key size dk, value size dv; h_(-1) = 0):

    x_s = h_t + (h_(t-1) - h_t) * mu_s        for s in r, k, v, g, w
    r = W_r x_r,  k = W_k x_k   [H dk],   v = W_v x_v,  g = W_g x_g   [H dv]          (no biases)
    d = exp(-exp(W_2 tanh(W_1 x_w) + w_0))   [H dk]
    per head:  o_t = (S_(t-1) + diag(u) k v^T)^T r,    S_t = diag(d) S_(t-1) + k v^T
    y = o / sqrt(mean(o^2) + eps) * w * silu(g)     the mean head by head, w over all heads' elements
    out = W_o y

S [dk, dv] starts at zero and is per-request state in float32; the last h is kept in the run's type, in
which the mixer reads it, so that a prompt cut into portions mixes the same numbers as one that is not.
The mixes are made in float32 and rounded once; W_1's product leaves its sums in float32, and the decay,
the recurrence, the norm and the gate are float32.  The decay's inner size is the checkpoint's to say.
Nothing is kept in the paged cache."""
from __future__ import annotations

from typing import Dict, List

import torch

from ..cache.manager import StateNeed
from ..weights.loader import AnySize, TensorDecl
from .base import BuildEnv, Mixer, StepView, register_part
from .linear import GroupedMatrix, as_matrix


class TimeMix(Mixer):
    replayable = True
    SHIFTS = ("r", "k", "v", "g", "w")

    def __init__(self, spec):
        super().__init__(spec)
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.heads = int(p["num_heads"])
        self.dk = int(p["key_dim"])
        self.dv = int(p.get("value_dim") or self.dk)
        self.rank = int(p["decay_rank"])
        self.eps = float(p["norm_eps"])

    def tensors(self) -> List[TensorDecl]:
        n, H, D = self.spec.names, self.heads, self.hidden
        qk, v, rank = H * self.dk, H * self.dv, AnySize(self.rank)
        return [TensorDecl(n["mu_" + s], (D,), "normal(0.5,0.2)") for s in self.SHIFTS] + \
            [TensorDecl(n["r"], (qk, D)), TensorDecl(n["k"], (qk, D)), TensorDecl(n["v"], (v, D)), TensorDecl(n["g"], (v, D)),
             TensorDecl(n["w1"], (rank, D)), TensorDecl(n["w2"], (qk, rank)), TensorDecl(n["w0"], (qk,), "normal(-3.0,1.0)"),
             TensorDecl(n["u"], (H, self.dk), "normal(0.5,0.3)"), TensorDecl(n["norm"], (v,), "ones_normal"),
             TensorDecl(n["o"], (D, v))]

    def load(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load(weights, env)
        n = self.spec.names

        def f32(role):
            return weights[n[role]].to(torch.float32).contiguous()
        self.rank = int(weights[n["w1"]].shape[0])
        if weights[n["w2"]].shape[1] != self.rank:
            raise ValueError(f"the decay's matrices meet in {self.rank} and {weights[n['w2']].shape[1]} elements")
        env.ops.check_wkv_sizes(self.heads, self.dk, self.dv, self.rank)
        self.mu = torch.stack([f32("mu_" + s) for s in self.SHIFTS]).contiguous()
        self.w_in = GroupedMatrix([weights[n[s]] for s in ("r", "k", "v", "g")], env, few=weights[n["w1"]])
        self.w2 = weights[n["w2"]].to(env.dtype).contiguous()
        self.w0, self.u, self.norm = f32("w0"), f32("u"), f32("norm")
        self.w_o = as_matrix(weights[n["o"]], env)

    def state_need(self):
        return {"S": StateNeed(tuple(self.env.ops.wkv_state_shape(self.heads, self.dk, self.dv)), torch.float32),
                "last": StateNeed((self.hidden,), None)}

    def workspace_elems(self, rows: int) -> int:
        # the mixes and projections, then in float32 decays, heads' outputs and the states before chunks of rows
        qk, v = self.heads * self.dk, self.heads * self.dv
        return rows * (5 * self.hidden + 2 * (2 * qk + 2 * v) + 2 * (qk + v + self.rank) + 2 * qk * self.dv // 32 + v)

    def mixes_of_normed_rows(self, step: StepView):
        """What the block's norm needs to make the mixes itself: (mu [mixes, size], the kept rows)."""
        return self.mu, step.state["last"]

    def forward(self, x: torch.Tensor, step: StepView):
        """x: normed rows [T, hidden], or their mixes [5, T, hidden] where the norm before has made them."""
        ops = self.env.ops
        mixes = x if x.dim() == 3 else ops.token_mixes(x, self.mu, step.state["last"], step)
        proj, z, z_strides = ops.linear_groups(mixes, self.w_in, step)
        y = ops.wkv(proj, z, z_strides, self.w2, self.w0, self.u, step.state["S"], step, self.heads, self.dk, self.dv, self.norm,
                    self.eps, self.env.dtype)
        return ops.linear(y, self.w_o, deferred=True)


register_part("mixer", "wkv", TimeMix)
