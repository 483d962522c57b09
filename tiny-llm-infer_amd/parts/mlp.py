"""Dense gated feed-forward: down( silu(gate(x)) * up(x) ) with
silu(g) = g / (1 + exp(-g)) (model/src/qwen3_paged_batch.cpp:281-295,
kernels/src/swiglu_kernel_cpu.cpp:20-24).  gate and up are stacked into one
matrix so that one product reads x once.  And the dense feed-forward without a gate,
down( act(up(x)) ), for a named activation."""
from __future__ import annotations

from typing import Dict, List

import torch

from ..weights.loader import TensorDecl
from .base import BuildEnv, FeedForward, StepView, register_part
from .linear import GatedMatrix, as_matrix


class SwiGLU(FeedForward):
    replayable = True

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec.params["hidden_size"])
        self.inter = int(spec.params["intermediate_size"])

    def tensors(self) -> List[TensorDecl]:
        n = self.spec.names
        return [TensorDecl(n["gate"], (self.inter, self.hidden)),
                TensorDecl(n["up"], (self.inter, self.hidden)),
                TensorDecl(n["down"], (self.hidden, self.inter))]

    def load(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load(weights, env)
        n = self.spec.names
        self.w_gate_up = GatedMatrix(weights[n["gate"]], weights[n["up"]], env)
        self.w_down = as_matrix(weights[n["down"]], env)

    def workspace_elems(self, rows: int) -> int:
        return rows * 3 * self.inter            # gate and up rows side by side, then the activation

    @property
    def takes_normed_rows(self) -> bool:       # x goes to the gate/up product only
        return getattr(self.w_gate_up, "gated", None) is not None

    def forward(self, x: torch.Tensor, step: StepView) -> torch.Tensor:
        ops = self.env.ops
        return ops.linear(ops.linear_swiglu(x, self.w_gate_up), self.w_down, deferred=True)   # a delta for the next norm


class DenseFF(FeedForward):
    """Dense feed-forward without a gate: down( act(up(x)) ).  ``activation`` names the
    function, one of the kernel library's ``ACTIVATIONS`` ("relu2" is relu(z)^2).  ``on_sums``: it is taken
    of the product's float32 sums, where the product's kernel can, and not of their rounding."""
    replayable = True

    def __init__(self, spec):
        super().__init__(spec)
        self.hidden = int(spec.params["hidden_size"])
        self.inter = int(spec.params["intermediate_size"])
        self.activation = str(spec.params["activation"])
        self.on_sums = bool(spec.params.get("on_sums", False))

    def tensors(self) -> List[TensorDecl]:
        n = self.spec.names
        return [TensorDecl(n["up"], (self.inter, self.hidden)),
                TensorDecl(n["down"], (self.hidden, self.inter))]

    def load(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load(weights, env)
        n = self.spec.names
        env.ops.check_activation(self.activation)
        self.w_up = as_matrix(weights[n["up"]], env)
        self.w_down = as_matrix(weights[n["down"]], env)

    def workspace_elems(self, rows: int) -> int:
        return rows * 2 * self.inter

    def forward(self, x: torch.Tensor, step: StepView) -> torch.Tensor:
        ops = self.env.ops
        if self.on_sums:
            hidden = ops.linear_act(x, self.w_up, self.activation)
        else:
            hidden = ops.activation(ops.linear(x, self.w_up), self.activation)
        return ops.linear(hidden, self.w_down, deferred=True)


register_part("ffn", "swiglu", SwiGLU)
register_part("ffn", "dense_act", DenseFF)
