"""The Kunitar decoder written out plainly: one function a mechanism, float64, whole sequences, no
cache, no batching, loops where a loop says it best.  What the engine is compared with; it shares no
code with the engine.

Notation: T positions, width D.  A layer is
    x <- x + s1 * n1b(mixer(n1(x)));   x <- x + s2 * n2b(ff(n2(x)));   x <- x + n3(P (gelu(G x) * e))
with RMS norms n, vectors s1, s2 and the token's own vector e of that layer.

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


def gelu_erf(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def squared_relu(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) ** 2


def turn(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """Neighbours (2i, 2i + 1) of the first ``dims`` elements of the last axis turned by position * base^(-2i/dims);
    x is [T, ..., n]."""
    out = x.clone()
    for i in range(dims // 2):
        angle = (positions.to(F) * base ** (-2.0 * i / dims)).view(-1, *([1] * (x.dim() - 2)))
        c, s = torch.cos(angle), torch.sin(angle)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def seen(i: int, size: int) -> List[int]:
    return [j for j in range(i + 1) if i - j < size]


def latent_rows(h: torch.Tensor, m: Dict, w: Dict[str, torch.Tensor], p: str, eps: float):
    """What a layer keeps of every position: the normed latent vector and the turned key part."""
    both = h @ w[p + "dkv"].T
    c = weighted_norm(both[:, :m["kv_rank"]], w[p + "dkv.norm"], eps)
    return c, turn(both[:, m["kv_rank"]:], torch.arange(h.shape[0]), m["rot"]["dims"], float(m["rot"]["base"]))


def windowed(q, k, v, scale: float, size: int) -> torch.Tensor:
    """q, k [T, H, d], v [T, H, e] -> [T, H, e]: softmax over the window's keys."""
    out = torch.zeros(q.shape[0], q.shape[1], v.shape[2], dtype=q.dtype)
    for i in range(q.shape[0]):
        js = slice(max(0, i - size + 1), i + 1)
        out[i] = torch.einsum("hj,jhe->he", torch.softmax(torch.einsum("hd,jhd->hj", q[i], k[js]) * scale, dim=1), v[js])
    return out


def latent_attention(h, m: Dict, w, p: str, eps: float, kept) -> torch.Tensor:
    """``kept``: (latent vectors [T, n], turned key parts [T, r]) of this layer or of the one it reads."""
    T, H, d, r, e = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, part = kept
    cq = weighted_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).view(T, H, d + r)
    q = torch.cat([q[..., :d], turn(q[..., d:], torch.arange(T), m["rot"]["dims"], float(m["rot"]["base"]))], dim=-1)
    k = torch.cat([(c @ w[p + "uk"].T).view(T, H, d), part[:, None, :].expand(T, H, r)], dim=-1)
    v = (c @ w[p + "uv"].T).view(T, H, e)
    o = windowed(q, k, v, float(m["scale"]), m["mask"]["size"])
    o = o * torch.sigmoid(h @ w[p + "g"].T)[..., None]
    return o.reshape(T, H * e) @ w[p + "o"].T


def shifted(h: torch.Tensor) -> torch.Tensor:
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def decayed_memory(r, k, v, decay, u) -> torch.Tensor:
    """o_t = (S + diag(u) k v^T)^T r, then S <- diag(decay_t) S + k v^T; r, k, decay [T, H, d], v [T, H, e], u [H, d]."""
    T, H, d = r.shape
    out = torch.zeros(T, H, v.shape[2], dtype=r.dtype)
    S = torch.zeros(H, d, v.shape[2], dtype=r.dtype)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = ((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(dim=1)
        S = decay[t][:, :, None] * S + kv
    return out


def decays(mix: torch.Tensor, w, p: str) -> torch.Tensor:
    return torch.exp(-torch.exp(torch.tanh(mix @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]))


def wkv(h: torch.Tensor, m: Dict, w, p: str, eps: float) -> torch.Tensor:
    T, H, d = h.shape[0], m["heads"], m["dim"]
    before = shifted(h)
    mix = {s: h + (before - h) * w[p + "mu." + s] for s in "rkvgw"}
    r, k, v = ((mix[s] @ w[p + s].T).view(T, H, d) for s in "rkv")
    o = decayed_memory(r, k, v, decays(mix["w"], w, p).view(T, H, d), w[p + "u"])
    o = unit_rms(o, eps).reshape(T, H * d) * w[p + "norm"]
    return (o * torch.nn.functional.silu(mix["g"] @ w[p + "g"].T)) @ w[p + "o"].T


def dense(h, f: Dict, w, p: str) -> torch.Tensor:
    return gelu_erf(h @ w[p + "up"].T) @ w[p + "down"].T


def expert(x, w, p: str) -> torch.Tensor:
    return squared_relu(x @ w[p + "up"].T) @ w[p + "down"].T


def experts(h, f: Dict, w, p: str) -> torch.Tensor:
    s = torch.sigmoid(h @ w[p + "router"].T)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in torch.sort(s[t], descending=True, stable=True).indices[:f["router"]["top"]].tolist():
            out[t] += expert(s[t, e] * h[t], w, p + f"e{e}.")
    if f.get("shared") is not None:
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * expert(h, w, p + "shared.")
    return out


FEED_FORWARDS = {"dense": dense, "moe": experts}


def token_side(x, own, w, p: str, eps: float) -> torch.Tensor:
    """What a token's own vector of this layer (``own`` [T, dim]) adds."""
    y = (gelu_tanh(x @ w[p + "side.gate"].T) * own) @ w[p + "side.proj"].T
    return weighted_norm(y, w[p + "side.norm"], eps)


def layer(x, i: int, cfg: Dict, w, tokens: torch.Tensor, kept: Dict) -> torch.Tensor:
    spec, p, eps = cfg["layers"][i], f"l{i}.", float(cfg["norm"]["eps"])
    m = spec["mixer"]
    h = weighted_norm(x, w[p + "norm1"], eps)
    if spec["type"] == "wkv":
        y = wkv(h, m, w, p + "mix.", eps)
    else:
        source = m.get("kv_from")
        if source is None:
            kept[i] = latent_rows(h, m, w, p + "mix.", eps)
            source = i
        y = latent_attention(h, m, w, p + "mix.", eps, kept[source])
    x = x + weighted_norm(y, w[p + "norm1b"], eps) * w[p + "ls1"]
    f = spec.get("mlp")
    if f is not None:
        y = FEED_FORWARDS[f["kind"]](weighted_norm(x, w[p + "norm2"], eps), f, w, p + "mlp.")
        x = x + weighted_norm(y, w[p + "norm2b"], eps) * w[p + "ls2"]
    dim = cfg["token_side"]["dim"]
    return x + token_side(x, w["side.embed"][tokens][:, i * dim:(i + 1) * dim], w, p, eps)


def forward(cfg: Dict, w: Dict[str, torch.Tensor], tokens: List[int], layers: Optional[List] = None) -> torch.Tensor:
    """Logits [T, vocab]; the residual after every layer is appended to ``layers`` if given."""
    ids = torch.tensor(tokens, dtype=torch.long)
    x = w["embed"][ids] * float(cfg["embedding"]["scale"])
    kept: Dict = {}
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, w, ids, kept)
        if layers is not None:
            layers.append(x)
    return weighted_norm(x, w["final.norm"], float(cfg["norm"]["eps"])) @ w["embed"].T
