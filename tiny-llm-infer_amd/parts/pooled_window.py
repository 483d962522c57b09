"""Attention over a window of tokens and, before it, one pooled key and value for every block of tokens.

For the rows h_p of one sequence (H query heads of size d, G key/value heads, values of size e, query
head a reads key head a // (H / G)):

    q_p = norm(Wq h_p + bq),  k_p = norm(Wk h_p + bk),  v_p = Wv h_p + bv
        norm: RMS over ALL heads' elements together, with a weight an element (``q_norm``, ``k_norm``)
    q, k: the first ``rotary_dim`` elements of every head turned by the position (``position``)
    row i sees token j if 0 <= i - j < window, and block b, the positions b P .. b P + P - 1, if
        b P + P - 1 <= i - window; the key of a block is the mean of its tokens' keys as the cache
        holds them, its value the mean of their values; a token whose block is not seen yet and that
        has left the window is not seen
    s = (q_i . key) * scale, one softmax over tokens and blocks whose denominator also holds exp(sink_a)
    out_i = Wo [sum w value]_a

Names of weights that the spec leaves out do not exist: biases, norms, ``sink``.

Two needs of the paged cache: the tokens' keys and values, whose pages go back as the window passes
(a block is pooled when its last token is written, so the tokens of the block that is not whole yet
are kept as well: the need's window is max(window, P)), and the blocks', with one slot for every P
positions, which stay."""
from __future__ import annotations

from typing import Dict, List, Tuple

import torch

from ..cache.manager import PAGE, CacheNeed, CacheRecord
from ..weights.loader import TensorDecl
from .base import BuildEnv, RotaryTables, StepView, build_part, register_part
from .joined import SplitMixer


class PooledWindowAttention(SplitMixer):
    def __init__(self, spec):
        super().__init__(spec)
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.heads = int(p["num_heads"])
        self.kv_heads = int(p["num_kv_heads"])
        self.dim = int(p["head_dim"])
        self.vdim = int(p.get("value_dim") or self.dim)
        self.scale = float(p["scale"])
        self.window = int(p["window"])
        self.pool = int(p["pool"])
        if self.heads % self.kv_heads:
            raise ValueError("num_heads must be a multiple of num_kv_heads")
        if self.window <= 0 or self.pool <= 0:
            raise ValueError("window and pool must be positive")
        self.sizes = {"q": self.heads * self.dim, "k": self.kv_heads * self.dim, "v": self.kv_heads * self.vdim}
        self.position = build_part("position", spec.parts["position"]) if "position" in spec.parts else None
        self.norms = {r: build_part("norm", spec.parts[r + "_norm"]) for r in ("q", "k") if r + "_norm" in spec.parts}

    def inputs(self) -> List[Tuple[str, int]]:
        return list(self.sizes.items())

    @property
    def rows_width(self) -> int:
        return self.heads * self.vdim

    def tensors(self) -> List[TensorDecl]:
        n = self.spec.names
        out = []
        for r, size in self.sizes.items():
            out.append(TensorDecl(n[r], (size, self.hidden)))
            if r + "_bias" in n:
                out.append(TensorDecl(n[r + "_bias"], (size,)))
        for norm in self.norms.values():
            out += norm.tensors()
        if "sink" in n:
            out.append(TensorDecl(n["sink"], (self.heads,), "normal(0.0,1.0)"))
        out.append(TensorDecl(n["o"], (self.hidden, self.rows_width)))
        return out + (self.position.tensors() if self.position is not None else [])

    def load_between(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load_between(weights, env)
        n = self.spec.names
        env.ops.check_sized_attention(self.heads, self.kv_heads, self.dim, self.vdim)
        self.rotary = None
        if self.position is not None:
            self.position.load(weights, env)
            tables = self.position.rotary()
            if tables is not None:
                self.rotary = RotaryTables(*tables)
                if self.rotary.rotary_dim > self.dim:
                    raise ValueError(f"{self.rotary.rotary_dim} turned elements do not fit a head of {self.dim}")
        self.norm_weights, self.eps = {}, 0.0
        for r, norm in self.norms.items():
            norm.load(weights, env)
            rms = norm.as_rms()
            if rms is None or tuple(rms[0].shape) != (self.sizes[r],):
                raise ValueError(f"the {r} norm of this attention must be an RMS norm over all {self.sizes[r]} elements of the projection")
            if self.norm_weights and float(rms[1]) != self.eps:
                raise ValueError("the norms of q and k of this attention have one eps")
            self.norm_weights[r], self.eps = rms[0], float(rms[1])
        self.bias = None
        if any(r + "_bias" in n for r in self.sizes):
            self.bias = torch.cat([weights[n[r + "_bias"]].to(torch.float32) if r + "_bias" in n
                                   else torch.zeros(size, dtype=torch.float32, device=env.device)
                                   for r, size in self.sizes.items()]).contiguous()
        self.sinks = weights[n["sink"]].to(torch.float32).contiguous() if "sink" in n else None

    def cache_need(self) -> Tuple[CacheNeed, CacheNeed]:
        records = (CacheRecord("k", (self.kv_heads, PAGE, self.dim)), CacheRecord("v", (self.kv_heads, self.vdim, PAGE)))
        return CacheNeed(records, max(self.window, self.pool)), CacheNeed(records, stride=self.pool)

    def workspace_elems(self, rows: int) -> int:
        return rows * (2 * sum(self.sizes.values()) + 2 * self.rows_width)

    def between(self, x, proj, at, step: StepView, out, out_at, scale) -> None:
        self.env.ops.pooled_window_attention(
            proj, at, step, step.cache, self.heads, self.kv_heads, self.dim, self.vdim, self.bias,
            self.norm_weights.get("q"), self.norm_weights.get("k"), self.eps, self.rotary, self.scale, self.sinks,
            self.window, self.pool, out, out_at, scale)


register_part("mixer", "pooled_window_attention", PooledWindowAttention)
