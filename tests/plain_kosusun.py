"""The Kosusun decoder written out plainly: one function a mechanism, float64, whole sequences,
no cache, no batching, loops where a loop says it best.  What the engine is compared with; it
shares no code with the engine.

Notation: T positions, width D.  A layer is x <- x + m (mixer(h) + ff(h)) with one norm h = norm(x)
that both read.

``cfg`` is the parsed config.json (a dict), ``w`` maps tensor names to float64 tensors.
"""
from __future__ import annotations

import json
import math
import os
import struct
from typing import Dict, List, Optional

import torch

F = torch.float64


def read_safetensors(path: str) -> Dict[str, torch.Tensor]:
    kinds = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "I32": torch.int32}
    with open(path, "rb") as fh:
        raw = fh.read()
    (hlen,) = struct.unpack("<Q", raw[:8])
    header = json.loads(raw[8:8 + hlen])
    out = {}
    for name, info in header.items():
        if name == "__metadata__":
            continue
        b, e = info["data_offsets"]
        t = torch.frombuffer(bytearray(raw[8 + hlen + b:8 + hlen + e]), dtype=kinds[info["dtype"]]).reshape(info["shape"])
        out[name] = t.to(F) if t.dtype.is_floating_point else t.clone()
    return out


def read_model(folder: str):
    with open(os.path.join(folder, "config.json")) as fh:
        cfg = json.load(fh)
    return cfg, read_safetensors(os.path.join(folder, "model.safetensors"))


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def weighted_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * weight


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def turn(x: torch.Tensor, positions: torch.Tensor, rot: Dict, neighbours: bool) -> torch.Tensor:
    """The first rot.dims elements of the last axis turned by the position; pair i is (i, i + dims/2),
    or (2i, 2i + 1) with ``neighbours``; angle = position * base^(-2i/dims) / factor.  x is [T, ..., n]."""
    dims, base = rot["dims"], float(rot["base"])
    factor = float((rot.get("scaling") or {}).get("factor", 1.0))
    out = x.clone()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        angle = positions.to(F) * (base ** (-2.0 * i / dims) / factor)
        angle = angle.view(-1, *([1] * (x.dim() - 2)))
        c, s = torch.cos(angle), torch.sin(angle)
        out[..., a] = x[..., a] * c - x[..., b] * s
        out[..., b] = x[..., b] * c + x[..., a] * s
    return out


def pooled_blocks(x: torch.Tensor, pool: int) -> torch.Tensor:
    """Means of the whole blocks of ``pool`` consecutive rows of [T, ...]."""
    n = x.shape[0] // pool
    return torch.stack([x[b * pool:(b + 1) * pool].mean(dim=0) for b in range(n)]) if n else x[:0]


def seen_tokens(i: int, size: int) -> List[int]:
    return [j for j in range(i + 1) if i - j < size]


def seen_blocks(i: int, size: int, pool: int) -> List[int]:
    out, b = [], 0
    while b * pool + pool - 1 <= i - size:
        out.append(b)
        b += 1
    return out


def softmax_with_sink(scores: torch.Tensor, sink: Optional[float]) -> torch.Tensor:
    """Weights of one row's scores when the denominator also holds exp(sink)."""
    top = float(scores.max())
    if sink is not None:
        top = max(top, sink)
    e = torch.exp(scores - top)
    return e / (e.sum() + (0.0 if sink is None else math.exp(sink - top)))


def windowed_attention(q, k, v, scale: float, size: int, pool: int, sinks) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]: the window's tokens and the pooled blocks
    before it in one softmax."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    bk, bv = pooled_blocks(k, pool), pooled_blocks(v, pool)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        t, b = seen_tokens(i, size), seen_blocks(i, size, pool)
        for h in range(H):
            g = h // (H // G)
            keys = torch.cat([k[t, g], bk[b, g]]) if b else k[t, g]
            values = torch.cat([v[t, g], bv[b, g]]) if b else v[t, g]
            out[i, h] = softmax_with_sink((keys @ q[i, h]) * scale, None if sinks is None else float(sinks[h])) @ values
    return out


def pooled_window_attention(h: torch.Tensor, m: Dict, w: Dict[str, torch.Tensor], p: str, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    G = m["kv_heads"]
    pos = torch.arange(T)
    q = weighted_norm(h @ w[p + "q"].T + w[p + "q.b"], w[p + "q.norm"], eps).view(T, H, d)
    k = weighted_norm(h @ w[p + "k"].T + w[p + "k.b"], w[p + "k.norm"], eps).view(T, G, d)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, e)
    q, k = turn(q, pos, m["rot"], True), turn(k, pos, m["rot"], True)
    o = windowed_attention(q, k, v, float(m["scale"]), m["mask"]["size"], m["mask"]["pool"], w[p + "sink"])
    return o.reshape(T, H * e) @ w[p + "o"].T


def decaying_memory(q, k, v, decay) -> torch.Tensor:
    """S <- decay S + k v^T, o = S^T q, head by head; q, k [T, H, d], v [T, H, e]."""
    T, H, d = q.shape
    e = v.shape[2]
    out = torch.zeros(T, H, e, dtype=q.dtype)
    for h in range(H):
        S = torch.zeros(d, e, dtype=q.dtype)
        for t in range(T):
            S = float(decay[h]) * S + torch.outer(k[t, h], v[t, h])
            out[t, h] = S.T @ q[t, h]
    return out


def retention(h: torch.Tensor, m: Dict, w: Dict[str, torch.Tensor], p: str, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q = turn((h @ w[p + "q"].T).view(T, H, d), pos, m["rot"], False)
    k = turn((h @ w[p + "k"].T).view(T, H, d), pos, m["rot"], False) * d ** -0.5
    v = (h @ w[p + "v"].T).view(T, H, e)
    o = unit_rms(decaying_memory(q, k, v, m["decay"]), eps).reshape(T, H * e)
    return (o * torch.nn.functional.silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def matrix_memory(q, k, v, i, f) -> torch.Tensor:
    """The mLSTM's memory with log gates i, f [T, H] and a running maximum that starts at 0."""
    T, H, d = q.shape
    e = v.shape[2]
    out = torch.zeros(T, H, e, dtype=q.dtype)
    for h in range(H):
        S, n, m = torch.zeros(d, e, dtype=q.dtype), torch.zeros(d, dtype=q.dtype), 0.0
        for t in range(T):
            ft, it = float(f[t, h]), float(i[t, h])
            new = max(ft + m, it)
            keep, take = math.exp(ft + m - new), math.exp(it - new)
            S = keep * S + take * torch.outer(k[t, h], v[t, h])
            n = keep * n + take * k[t, h]
            m = new
            out[t, h] = (S.T @ q[t, h]) / (max(abs(float(n @ q[t, h])), math.exp(-m)) + 1e-6)
    return out


def mlstm_gates(h: torch.Tensor, m: Dict, w: Dict[str, torch.Tensor], p: str):
    cap = float(m["gate_cap"])
    i = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    return i, f


def mlstm(h: torch.Tensor, m: Dict, w: Dict[str, torch.Tensor], p: str, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, e)
    i, f = mlstm_gates(h, m, w, p)
    o = unit_rms(matrix_memory(q, k, v, i, f), eps).reshape(T, H * e) * w[p + "norm"]
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def side_by_side(h: torch.Tensor, m: Dict, w: Dict[str, torch.Tensor], p: str, eps: float) -> torch.Tensor:
    return (float(m["left_scale"]) * pooled_window_attention(h, m["left"], w, p + "left.", eps)
            + float(m["right_scale"]) * retention(h, m["right"], w, p + "right.", eps))


def dense(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


MIXERS = {"parallel": side_by_side, "mlstm": mlstm}


def layer(x: torch.Tensor, i: int, cfg: Dict, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    spec, p, eps = cfg["layers"][i], f"l{i}.", float(cfg["norm"]["eps"])
    h = weighted_norm(x, w[p + "norm1"], eps)
    y = MIXERS[spec["type"]](h, spec["mixer"], w, p + "mix.", eps)
    if spec.get("mlp") is not None:
        y = y + dense(h, w, p + "mlp.")
    return x + float(cfg["residual_mult"]) * y


def forward(cfg: Dict, w: Dict[str, torch.Tensor], tokens: List[int], layers: Optional[List] = None) -> torch.Tensor:
    """Logits [T, vocab]; the residual after every layer is appended to ``layers`` if given."""
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, w)
        if layers is not None:
            layers.append(x)
    return (weighted_norm(x, w["final.norm"], float(cfg["norm"]["eps"])) @ w["head"].T) * float(cfg["logit_scale"])
