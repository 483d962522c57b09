"""Attention whose keys and values are made from one latent vector a position ("latent attention").

With H heads, ``head_dim`` d elements of a query/key head that are not turned and ``rotary_dim``
r that are, value heads of e and a latent vector of ``kv_rank`` n:

    q = W_q x                       [H, d + r] a position, head by head as [plain, turned part]
    W_down x                        [n + r]: the first n, RMS-normed with a weight, are the latent
                                    vector c; the last r, not normed, are one key part for all heads
    k_h = [W_uk,h c | key part],  v_h = W_uv,h c
    s_ij = (q_plain . k_plain + q_turned . k_turned) * scale,   j <= i,   softmax, sum of values

With ``q_rank`` m the queries go through a latent vector of their own, q = W_q norm(W_down_q x), normed with a
weight (``query_norm``).  With a ``gate`` the heads' outputs are multiplied by sigmoid(W_g x), one number a head.
With a ``window`` w position i sees j with 0 <= i - j < w.  A mixer that names no ``down`` matrix has no
latent vectors of its own: it reads those that another call of the step wrote to its cache layer
(``LayerCall.writes_cache`` false).  Layers that share a cache layer state one need: ``cache_window`` is the
largest of their windows.

The position encoding (``position``) turns the r-part of every query head and the shared key
part (pairs (i, i + dims/2), or neighbours for an encoding that says so).  With a ``sink`` (one
learned logit a head) the softmax's denominator also holds exp(sink).  The cache keeps, for a position, c and the turned key part and nothing else (record
"latent", ``[slot, n + r]``): q_plain . (W_uk,h c) = (W_uk,h^T q_plain) . c, so every head's
query is taken into the latent space by a small product of its own and all heads then read the
same cached vectors, and the weighted sum of the c of the seen positions goes through W_uv,h
afterwards (sum_j p_j W_uv,h c_j = W_uv,h sum_j p_j c_j).
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..cache.manager import PAGE, CacheNeed, CacheRecord
from ..weights.loader import TensorDecl
from .base import ROTARY_PAIRINGS, BuildEnv, Mixer, RotaryTables, StepView, build_part, register_part
from .linear import as_matrix, fuse_rows


class LatentAttention(Mixer):
    replayable = True

    def __init__(self, spec):
        super().__init__(spec)
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.heads = int(p["num_heads"])
        self.dim = int(p["head_dim"])
        self.rot = int(p["rotary_dim"])
        self.vdim = int(p.get("value_dim") or self.dim)
        self.rank = int(p["kv_rank"])
        self.scale = float(p["scale"])
        self.q_rank = None if p.get("q_rank") is None else int(p["q_rank"])
        self.window = None if p.get("window") is None else int(p["window"])
        self.cache_window = p.get("cache_window", self.window)
        if self.cache_window is not None and (self.window is None or self.window > self.cache_window):
            raise ValueError(f"a window of {self.window} does not fit a cache that keeps {self.cache_window}")
        self.gated, self.own = "gate" in spec.names, "down" in spec.names
        self.position = build_part("position", spec.parts["position"])
        self.latent_norm = build_part("norm", spec.parts["latent_norm"]) if self.own else None
        self.query_norm = build_part("norm", spec.parts["query_norm"]) if self.q_rank is not None else None

    def tensors(self) -> List[TensorDecl]:
        n = self.spec.names
        return ([TensorDecl(n["down_q"], (self.q_rank, self.hidden))] if self.q_rank is not None else []) + \
            [TensorDecl(n["q"], (self.heads * (self.dim + self.rot), self.q_rank or self.hidden))] + \
            ([TensorDecl(n["down"], (self.rank + self.rot, self.hidden))] if self.own else []) + \
            [TensorDecl(n["up_k"], (self.heads * self.dim, self.rank)),
             TensorDecl(n["up_v"], (self.heads * self.vdim, self.rank)),
             TensorDecl(n["o"], (self.hidden, self.heads * self.vdim))] + \
            ([TensorDecl(n["gate"], (self.heads, self.hidden))] if self.gated else []) + \
            ([TensorDecl(n["sink"], (self.heads,), "normal(0.0,1.0)")] if "sink" in n else []) + \
            [d for part in (self.latent_norm, self.query_norm, self.position) if part is not None for d in part.tensors()]

    def load(self, weights: Dict[str, torch.Tensor], env: BuildEnv) -> None:
        super().load(weights, env)
        n = self.spec.names
        env.ops.check_sized_attention(self.heads, 1, self.rank + self.rot, self.rank)
        self.position.load(weights, env)
        for norm in (self.latent_norm, self.query_norm):
            if norm is not None:
                norm.load(weights, env)
        tables = self.position.rotary()
        if tables is None:
            raise ValueError("the position encoding of this attention must be a rotation")
        tables = RotaryTables(*tables)
        if tables.pairing not in ROTARY_PAIRINGS:
            raise ValueError(f"rotary pairing '{tables.pairing}' is not known; known: {', '.join(ROTARY_PAIRINGS)}")
        if tables.rotary_dim > self.rot:
            raise ValueError(f"{tables.rotary_dim} turned elements do not fit a part of {self.rot}")
        self.rotary = (tables.cos, tables.sin, int(tables.rotary_dim))
        # The kernels turn the pairs (i, i + dims / 2).  An encoding that pairs neighbours (2i, 2i + 1) is served
        # by them all the same: a score does not change when the turned parts of q and of the key are permuted
        # alike, so the rows that make those parts are put in the order 0, 2, 4, .., 1, 3, 5, .. once, here.
        w_q, w_down = weights[n["q"]], weights[n["down"]] if self.own else None
        if tables.pairing == "interleaved":
            rd = int(tables.rotary_dim)
            order = torch.cat([torch.arange(0, rd, 2), torch.arange(1, rd, 2), torch.arange(rd, self.rot)]).to(w_q.device)
            per = self.dim + self.rot
            q_rows = torch.cat([torch.arange(self.dim, device=w_q.device), self.dim + order])
            w_q = w_q.view(self.heads, per, -1)[:, q_rows].reshape(self.heads * per, -1)
            if self.own:
                w_down = torch.cat([w_down[:self.rank], w_down[self.rank:][order]], dim=0)

        def rms_of(norm, size, what):
            rms = norm.as_rms()
            if rms is None or tuple(rms[0].shape) != (size,):
                raise ValueError(f"the norm of the {what} must be an RMS norm over its elements")
            return rms[0], float(rms[1])
        self.norm_weight, self.norm_eps = rms_of(self.latent_norm, self.rank, "latent vector") if self.own else (None, 0.0)
        # one product for everything that reads x: the queries or what they are made from, the latent vector and the
        # key part, the gates' logits
        inputs = [("q", w_q) if self.q_rank is None else ("down_q", weights[n["down_q"]])]
        if self.own:
            inputs.append(("down", w_down))
        if self.gated:
            inputs.append(("gate", weights[n["gate"]]))
        self.at, width = {}, 0
        for role, m in inputs:
            self.at[role], width = width, width + m.shape[0]
        self.w_in = fuse_rows([m for _, m in inputs], env)
        if self.q_rank is not None:
            self.q_weight, self.q_eps = rms_of(self.query_norm, self.q_rank, "queries' latent vector")
            self.w_uq = as_matrix(w_q, env)
        # a sink: one learned logit a head in the softmax's denominator, with no key and no value
        self.sinks = weights[n["sink"]].to(torch.float32).contiguous() if "sink" in n else None
        # a matrix a head, row-major: into the latent space [H, n, d] (W_uk of the head, transposed) and out of it [H, e, n]
        self.w_qk = weights[n["up_k"]].to(env.dtype).view(self.heads, self.dim, self.rank).transpose(1, 2).contiguous()
        self.w_v = weights[n["up_v"]].to(env.dtype).view(self.heads, self.vdim, self.rank).contiguous()
        self.w_o = as_matrix(weights[n["o"]], env)

    def cache_need(self) -> Optional[CacheNeed]:
        return CacheNeed((CacheRecord("latent", (PAGE, self.rank + self.rot)),), self.cache_window)

    def workspace_elems(self, rows: int) -> int:
        key = self.rank + self.rot
        return rows * (2 * (self.heads * (self.dim + self.rot) + key + 2 * (self.q_rank or 0) + self.heads) +
                       self.heads * (key + self.rank + self.vdim))

    def forward(self, x: torch.Tensor, step: StepView) -> torch.Tensor:
        ops = self.env.ops
        proj = ops.linear(x, self.w_in)
        query, q_at = proj, self.at.get("q")
        if self.q_rank is not None:
            rows = ops.norm_rows(proj, self.at["down_q"], self.q_rank, self.q_weight, self.q_eps)
            query, q_at = ops.linear(rows, self.w_uq), 0
        own = (proj, self.at["down"], self.norm_weight, self.norm_eps) if self.own else None
        o = ops.latent_attention(query, q_at, own, step, step.cache, self.heads, self.dim, self.rot, self.rank, self.vdim,
                                 self.rotary, self.scale, self.w_qk, self.w_v, window=self.window, sinks=self.sinks,
                                 gate=(proj, self.at["gate"]) if self.gated else None)
        return ops.linear(o, self.w_o, deferred=True)


register_part("mixer", "latent_attention", LatentAttention)
