"""Parts that are a product, something in between, and a product again, and how several of them that
read the same rows become one.

A ``SplitMixer`` or ``GatedDense`` makes *rows* (what its last matrix multiplies) from *projections*
(what its first matrices give).  Whoever holds such parts side by side may stack the first matrices
of all of them into one product, let every part leave its rows, times a factor, in its own columns
of one buffer, and multiply that with the last matrices side by side:

    sum_p c_p W_p rows_p  =  [W_1 | W_2 | ..] [c_1 rows_1 ; c_2 rows_2 ; ..]

so that the sum of the parts is taken in float32 inside one product, and the factors before the
rows are rounded to the run's type.  ``SideBySide`` does that for two mixers, the block
"parallel_one_norm" for a mixer and a feed-forward that read one norm,
x <- x + m (mixer(h) + ff(h)), h = norm(x)."""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from ..weights.loader import TensorDecl
from .base import Block, BuildEnv, FeedForward, Mixer, StepView, build_part, register_part, run_norm
from .linear import GatedMatrix, as_matrix, fuse_rows


def _aligned(n: int) -> int:
    return (n + 7) // 8 * 8          # columns of a buffer start at multiples of 8 elements


class JoinedRows:
    """The last matrices of several parts side by side, and the buffer of rows that they multiply.  A
    part's columns start at a multiple of 8; the columns between (none for sizes in eights) are zero
    in both."""

    def __init__(self, widths: List[int], matrices: List[torch.Tensor], env: BuildEnv):
        self.at, end = [], 0
        for w in widths:
            self.at.append(end)
            end = _aligned(end + w)
        self.width, self.gaps = end, end != sum(widths)
        self.env = env
        if len(matrices) == 1 and not self.gaps:
            joined = matrices[0]
        else:
            joined = torch.zeros((matrices[0].shape[0], end), dtype=env.dtype, device=matrices[0].device)
            for at, w, m in zip(self.at, widths, matrices):
                joined[:, at:at + w] = m
        self.matrix = as_matrix(joined, env)

    def buffer(self, rows: int) -> torch.Tensor:
        make = torch.zeros if self.gaps else torch.empty
        return make((rows, self.width), dtype=self.env.dtype, device=self.env.device)

    def product(self, buffer: torch.Tensor):
        return self.env.ops.linear(buffer, self.matrix, deferred=True)


class SplitMixer(Mixer):
    """A mixer in three steps.  A subclass gives ``inputs()`` (the roles of the matrices that read x, in
    the order of their projections, with the rows of each), ``output`` (the role of the last matrix),
    ``rows_width``, ``load_between`` and ``between``."""
    replayable = True
    between_reads_x = False          # ``between`` needs x as a tensor of normed rows (not as rows that owe their factor)

    def inputs(self) -> List[Tuple[str, int]]:
        raise NotImplementedError

    @property
    def rows_width(self) -> int:
        raise NotImplementedError

    @property
    def inputs_width(self) -> int:
        return sum(n for _, n in self.inputs())

    def input_matrices(self, weights: Dict[str, torch.Tensor]) -> List[torch.Tensor]:
        return [weights[self.spec.names[r]] for r, _ in self.inputs()]

    def output_matrix(self, weights: Dict[str, torch.Tensor]) -> torch.Tensor:
        return weights[self.spec.names["o"]]

    def load_between(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        self.env = env

    def between(self, x, proj: torch.Tensor, at: int, step: StepView, out: torch.Tensor, out_at: int, scale: float) -> None:
        """From the projections ``proj[:, at : at + inputs_width]`` to the rows, times ``scale``, in
        ``out[:, out_at : out_at + rows_width]``."""
        raise NotImplementedError

    # ---- as one of several parts whose rows are joined
    def load_rows(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        self.load_between(weights, env)
        self.w_in = fuse_rows(self.input_matrices(weights), env)

    @property
    def takes_normed_rows(self) -> bool:
        return not self.between_reads_x and getattr(self, "w_in", None) is not None and self.w_in.tiled is not None

    def rows(self, x, step: StepView, out: torch.Tensor, out_at: int, scale: float) -> None:
        self.between(x, self.env.ops.linear(x, self.w_in), 0, step, out, out_at, scale)

    # ---- alone
    def load(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        self.load_rows(weights, env)
        self.joined = JoinedRows([self.rows_width], [self.output_matrix(weights)], env)

    def forward(self, x, step: StepView):
        out = self.joined.buffer(step.num_rows)
        self.rows(x, step, out, 0, 1.0)
        return self.joined.product(out)


class SideBySide(SplitMixer):
    """Two mixers that read the same rows:  left_scale * left(x) + right_scale * right(x).  One product for
    the projections of both, one for both outputs.  State and cache are the mixers' own: a step hands
    each the state it asked for; at most one of them may keep something in the paged cache."""

    def __init__(self, spec):
        super().__init__(spec)
        self.sides = {side: build_part("mixer", spec.parts[side]) for side in ("left", "right")}
        self.scales = {side: float(spec.params[side + "_scale"]) for side in self.sides}
        for side, m in self.sides.items():
            if not isinstance(m, SplitMixer):
                raise ValueError(f"the {side} mixer ('{m.spec.kind}') is not one whose projections and rows can be joined")
        self.cached = [s for s, m in self.sides.items() if m.cache_need() is not None]
        if len(self.cached) > 1:
            raise ValueError("two mixers side by side of which both keep keys in the cache are not supported")
        self.replayable = all(m.replayable for m in self.sides.values())
        self.between_reads_x = any(m.between_reads_x for m in self.sides.values())

    def tensors(self) -> List[TensorDecl]:
        return [d for m in self.sides.values() for d in m.tensors()]

    def cache_need(self):
        return self.sides[self.cached[0]].cache_need() if self.cached else None

    def state_need(self):
        needs = {}
        for side, m in self.sides.items():
            need = m.state_need()
            if isinstance(need, dict):
                needs.update({f"{side}.{k}": n for k, n in need.items()})
            elif need is not None:
                needs[side] = need
        return needs or None

    def inputs(self) -> List[Tuple[str, int]]:
        return [(f"{side}.{r}", n) for side, m in self.sides.items() for r, n in m.inputs()]

    def input_matrices(self, weights) -> List[torch.Tensor]:
        return [w for m in self.sides.values() for w in m.input_matrices(weights)]

    @property
    def rows_width(self) -> int:
        left, right = self.sides["left"], self.sides["right"]
        return _aligned(left.rows_width) + right.rows_width

    def output_matrix(self, weights) -> torch.Tensor:
        left, right = self.sides["left"], self.sides["right"]
        a, b = left.output_matrix(weights), right.output_matrix(weights)
        gap = _aligned(left.rows_width) - left.rows_width
        return torch.cat([a, torch.zeros((a.shape[0], gap), dtype=a.dtype, device=a.device), b], dim=1)

    def load_between(self, weights, env: BuildEnv) -> None:
        super().load_between(weights, env)
        for m in self.sides.values():
            m.load_between(weights, env)

    def workspace_elems(self, rows: int) -> int:
        return sum(m.workspace_elems(rows) for m in self.sides.values())

    def between(self, x, proj, at, step: StepView, out, out_at, scale) -> None:
        states, width = step.state or {}, 0
        left = self.sides["left"]
        gap = _aligned(left.rows_width) - left.rows_width
        if gap:
            out[:, out_at + left.rows_width:out_at + left.rows_width + gap] = 0
        for side, m in self.sides.items():
            own = {k[len(side) + 1:]: t for k, t in states.items() if k.startswith(side + ".")}
            step.state = own or states.get(side)
            m.between(x, proj, at, step, out, out_at + width, scale * self.scales[side])
            at += m.inputs_width
            width = _aligned(width + m.rows_width)
        step.state = states or None


class GatedDense(FeedForward):
    """Dense gated feed-forward for a named gate activation:  down( act(gate(x)) * up(x) ), one of the
    kernel library's ``GATE_ACTIVATIONS``."""
    replayable = True

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec.params["hidden_size"])
        self.inter = int(spec.params["intermediate_size"])
        self.activation = str(spec.params["activation"])

    def tensors(self) -> List[TensorDecl]:
        n = self.spec.names
        return [TensorDecl(n["gate"], (self.inter, self.hidden)), TensorDecl(n["up"], (self.inter, self.hidden)),
                TensorDecl(n["down"], (self.hidden, self.inter))]

    @property
    def rows_width(self) -> int:
        return self.inter

    def output_matrix(self, weights) -> torch.Tensor:
        return weights[self.spec.names["down"]]

    def load_rows(self, weights, env: BuildEnv) -> None:
        self.env = env
        env.ops.check_gate_activation(self.activation)
        n = self.spec.names
        self.w_gate_up = GatedMatrix(weights[n["gate"]], weights[n["up"]], env)

    @property
    def takes_normed_rows(self) -> bool:
        return getattr(getattr(self, "w_gate_up", None), "gated", None) is not None

    def workspace_elems(self, rows: int) -> int:
        return rows * 3 * self.inter

    def rows(self, x, step: StepView, out, out_at, scale) -> None:
        self.env.ops.linear_swiglu(x, self.w_gate_up, activation=self.activation, scale=scale, into=(out, out_at))

    def load(self, weights, env: BuildEnv) -> None:
        self.load_rows(weights, env)
        self.joined = JoinedRows([self.inter], [self.output_matrix(weights)], env)

    def forward(self, x, step: StepView):
        out = self.joined.buffer(step.num_rows)
        self.rows(x, step, out, 0, 1.0)
        return self.joined.product(out)


class OneNormParallelBlock(Block):
    """x <- x + m (mixer(h) + ff(h)), h = norm(x), m the constant ``residual_mult``: the rows of the mixer and of
    the feed-forward are multiplied with both last matrices in one product.  Without a feed-forward
    x <- x + m mixer(h).  The sum is left to whoever normalises next, as in the other arrangements."""

    def __init__(self, spec, mixer, ffn, norms):
        super().__init__(spec)
        self.mixer, self.ffn, self.norm = mixer, ffn, norms["mixer"]
        self.mult = float(spec.params.get("residual_mult", 1.0))
        for part in self._sublayers():
            if not (hasattr(part, "load_rows") and hasattr(part, "rows")):
                raise ValueError(f"'{part.spec.kind}' is not a part whose rows can be joined with another's")
        self.replayable = all(p.replayable for p in [self.norm] + self._sublayers())

    def _sublayers(self):
        return [p for p in (self.mixer, self.ffn) if p is not None]

    def tensors(self) -> List[TensorDecl]:
        return self.norm.tensors() + [d for p in self._sublayers() for d in p.tensors()]

    def load(self, weights, env: BuildEnv) -> None:
        super().load(weights, env)
        self.norm.load(weights, env)
        parts = self._sublayers()
        for part in parts:
            part.load_rows(weights, env)
        self.joined = JoinedRows([p.rows_width for p in parts], [p.output_matrix(weights) for p in parts], env)
        self.takes_normed_rows = all(p.takes_normed_rows for p in parts)

    def forward(self, resid: torch.Tensor, pending: Optional[torch.Tensor], step: StepView):
        h = run_norm(self.norm, resid, pending, consumer=self)
        out = self.joined.buffer(step.num_rows)
        for part, at in zip(self._sublayers(), self.joined.at):
            part.rows(h, step, out, at, self.mult)
        return self.joined.product(out)


register_part("mixer", "side_by_side", SideBySide)
register_part("ffn", "gated_dense", GatedDense)
register_part("block", "parallel_one_norm", OneNormParallelBlock)
