"""Residual block that norms what a sublayer reads and what it gives:

    x <- x + s1 * n1b(mixer(n1(x))),     x <- x + s2 * n2b(ff(n2(x)))

with RMS norms n (a weight each) and, where the spec names them, vectors s1, s2 that scale a sublayer's
normed output element by element (they are multiplied into that norm's float32 weight once, when it is
loaded).  Behind the sublayers may stand a token's own vector (``side``, see ``TokenSide``):
x <- x + n3(side(x)).  Without a feed-forward the second line is left out.

One pass over a row norms a sublayer's output, adds it to the float32 residual and norms the sum for
whoever reads it next.  The block's last sum is left to the next block, which knows its own first norm, or
to the final norm (``NormedDelta``).

``TokenSide``: y = P (act(G x) * e), e the part of this layer of the token's row in a table [vocab, layers
dim] that all layers share; x is the residual itself."""
from __future__ import annotations

from typing import Dict, List

import torch

from ..weights.loader import TensorDecl
from .base import Block, BuildEnv, Part, StepView, build_part, register_part
from .linear import as_matrix


class NormedDelta:
    """What a block still owes the residual: weight * y / sqrt(mean(y^2) + eps)."""

    def __init__(self, y, weight: torch.Tensor, eps: float):
        self.y, self.weight, self.eps = y, weight, eps


class TokenSide(Part):
    replayable = True

    def __init__(self, spec):
        super().__init__(spec)
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.vocab = int(p["vocab_size"])
        self.dim = int(p["dim"])
        self.layers = int(p["layers"])
        self.at = int(p["layer"]) * self.dim
        self.activation = str(p["activation"])
        self.norm = build_part("norm", spec.parts["norm"])

    def tensors(self) -> List[TensorDecl]:
        n = self.spec.names
        return [TensorDecl(n["table"], (self.vocab, self.layers * self.dim)), TensorDecl(n["gate"], (self.dim, self.hidden)),
                TensorDecl(n["proj"], (self.hidden, self.dim))] + self.norm.tensors()

    def load(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load(weights, env)
        n = self.spec.names
        env.ops.check_activation(self.activation)
        self.norm.load(weights, env)
        key = ("token_side", n["table"])
        if key not in env.shared:                 # rows are gathered: row-major, one copy for all layers
            env.shared[key] = weights[n["table"]].to(env.dtype).contiguous()
        self.table = env.shared[key]
        self.w_gate = as_matrix(weights[n["gate"]], env)
        self.w_proj = as_matrix(weights[n["proj"]], env)

    def forward(self, x: torch.Tensor, step: StepView):
        """x: the residual's rows in the run's type; returns y, not normed."""
        ops = self.env.ops
        z = ops.linear_act(x, self.w_gate, self.activation, token=(self.table, self.at, step.token_ids))
        return ops.linear(z, self.w_proj, deferred=True)


class SandwichBlock(Block):
    def __init__(self, spec, mixer, ffn, norms):
        super().__init__(spec)
        self.mixer = mixer
        self.ffn = ffn
        self.norms = dict(norms)
        self.roles = ["mixer"] + (["ffn"] if ffn is not None else [])
        for role in self.roles:
            for r in (role, role + "_out"):
                if r not in self.norms:
                    raise ValueError(f"a block of this arrangement needs the norm '{r}'")
        self.side = build_part("side", spec.parts["side"]) if "side" in spec.parts else None
        self.size = int(norms["mixer"].size)
        self.replayable = all(p.replayable for p in self._parts())

    def _parts(self):
        out = []
        for role, part in (("mixer", self.mixer), ("ffn", self.ffn)):
            if part is not None:
                out += [self.norms[role], part, self.norms[role + "_out"]]
        return out + ([self.side] if self.side is not None else [])

    def _scales(self):
        return [role for role in self.roles if role + "_scale" in self.spec.names]

    def tensors(self) -> List[TensorDecl]:
        own = [TensorDecl(self.spec.names[role + "_scale"], (self.size,), "normal(1.0,0.1)") for role in self._scales()]
        return own + [d for p in self._parts() for d in p.tensors()]

    def load(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load(weights, env)
        for part in self._parts():
            part.load(weights, env)

        def rms(norm):
            r = norm.as_rms()
            if r is None:
                raise ValueError(f"this arrangement norms with the RMS norm that its kernel has built in, not with '{norm.spec.kind}'")
            return r
        self.first = {role: rms(self.norms[role]) for role in self.roles}
        self.last = {}
        for role in self.roles:
            weight, eps = rms(self.norms[role + "_out"])
            if role in self._scales():
                weight = (weight * weights[self.spec.names[role + "_scale"]].to(torch.float32)).contiguous()
            self.last[role] = (weight, eps)
        self.side_rms = rms(self.side.norm) if self.side is not None else None

    def _read(self, resid, owed, role: str, step: StepView, reader):
        """The rows that the sublayer ``role`` reads, after what is owed to the residual has been added to it."""
        ops = self.env.ops
        weight, eps = self.first[role]
        y, w_out, eps_out = (owed.y, owed.weight, owed.eps) if owed is not None else (None, None, 0.0)
        mixes = getattr(reader, "mixes_of_normed_rows", None)
        if mixes is not None:                     # a reader of mixes of every row with the row before it: made in the same pass
            mixed = ops.norm_add_norm_mixes(resid, y, w_out, eps_out, weight, eps, self.env.dtype, mixes(step), step)
            if mixed is not None:
                return mixed
        return ops.norm_add_norm(resid, y, w_out, eps_out, weight, eps, self.env.dtype)

    def forward(self, resid: torch.Tensor, pending, step: StepView):
        if pending is not None and not isinstance(pending, NormedDelta):
            raise TypeError("the block before this one leaves a sum of another kind to the residual; blocks of this "
                            "arrangement follow their own kind only")
        owed = pending
        for role, part in (("mixer", self.mixer), ("ffn", self.ffn)):
            if part is None:
                continue
            y = part.forward(self._read(resid, owed, role, step, part), step)
            owed = NormedDelta(y, *self.last[role])
        if self.side is None:
            return owed
        rows = self.env.ops.norm_add(resid, owed.y, owed.weight, owed.eps, self.env.dtype)
        return NormedDelta(self.side.forward(rows, step), *self.side_rms)

    def close(self, resid, pending, final_norm, rows=None, num_rows=None):
        rms = final_norm.as_rms()
        if rms is None:
            raise ValueError("the norm after blocks of this arrangement must be an RMS norm")
        return self.env.ops.norm_add_norm(resid, pending.y, pending.weight, pending.eps, rms[0], rms[1], self.env.dtype,
                                          rows=rows, num_rows=num_rows)


register_part("side", "token_side", TokenSide)
register_part("block", "sandwich", SandwichBlock)
