"""Shared by the Kunitar tests: small configurations that differ in every size and option, weights
drawn so that every mechanism matters, and model folders of them."""
from __future__ import annotations

import json
import os
from typing import Dict, List

import numpy as np
import torch


def _latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, size, base=10000.0, scale=None, kv_from=None):
    out = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
           "scale": float((dim + rot_dim) ** -0.5 if scale is None else scale), "rot": {"dims": rot_dim, "base": base},
           "mask": {"size": size}}
    if kv_from is not None:
        out["kv_from"] = kv_from
    return out


def _wkv(heads, dim):
    return {"heads": heads, "dim": dim}


def _moe(experts, top, ff, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def _config(vocab, width, side, layers, embed=1.0, eps=1e-5):
    return {"architecture": "Kunitar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed},
            "token_side": {"dim": side}, "layers": layers}


L, W = "latent_attention", "wkv"

# name -> (config.json, rank of the decays, page size of the engine in its tests, seed)
SMALL = {
    # two layers read the vectors of the first, with a smaller and a larger window than its own; two experts a token
    "A": (_config(160, 64, 12, [_layer(L, _latent(4, 16, 8, 24, 32, 48, 20), _dense(96)),
                                _layer(W, _wkv(3, 16), _moe(6, 2, 40, 56)),
                                _layer(L, _latent(2, 24, 8, 16, 32, 16, 9, kv_from=0), _moe(4, 1, 32)),
                                _layer(L, _latent(3, 8, 8, 8, 32, 24, 37, scale=0.4, kv_from=0), _dense(50))], embed=2.5), 8, 16, 3),
    # sizes out of eights: a width of 100, heads of 20 and 7, ranks of 5 and 18; a layer without feed-forward; one head; the
    # first layer is recurrent, another reads none but its own vectors
    "B": (_config(211, 100, 7, [_layer(W, _wkv(3, 20), _moe(5, 3, 37, 21)),
                                _layer(W, _wkv(1, 7), None),
                                _layer(L, _latent(3, 12, 6, 10, 18, 20, 7, base=500.0), _moe(3, 3, 24, 11)),
                                _layer(L, _latent(1, 20, 2, 7, 30, 9, 24, base=300.0), None)], eps=3e-6, embed=0.7), 5, 8, 5),
    # a window of one; experts without a shared one
    "C": (_config(257, 72, 16, [_layer(W, _wkv(2, 40), _dense(56)),
                                _layer(L, _latent(2, 8, 4, 16, 24, 40, 1), _moe(8, 1, 16))], embed=0.9), 24, 16, 11),
    # sizes in sixteens (the matrix-core kernels), pages of 32, products that are one launch
    "R": (_config(320, 128, 32, [_layer(W, _wkv(4, 64), _moe(8, 2, 64, 96)),
                                 _layer(L, _latent(6, 32, 16, 48, 64, 96, 40), _dense(256)),
                                 _layer(W, _wkv(2, 128), _moe(4, 1, 96, 64)),
                                 _layer(W, _wkv(8, 32), None),
                                 _layer(L, _latent(4, 64, 16, 64, 64, 64, 65, kv_from=1), _dense(128))], embed=1.5), 32, 32, 7),
    # heads of 48 and 80: sixteens that no kernel is made for alone
    "S": (_config(192, 96, 8, [_layer(W, _wkv(5, 48), _dense(64)), _layer(W, _wkv(1, 80), _moe(3, 1, 32, 32)),
                               _layer(L, _latent(5, 48, 32, 32, 80, 32, 33, base=2000.0), None)], embed=1.2), 16, 16, 13),
}


def make_weights(cfg: dict, rank: int, seed: int, clear: bool = False) -> Dict[str, torch.Tensor]:
    """bfloat16 weights of a size that makes every mechanism show in the logits.  ``clear`` (for comparisons in
    bfloat16): routers without a close call (they read one wide direction that rounding does not move far), scores of a
    size that a softmax does not multiply rounding with, and recurrences whose keys resemble their queries (a head's
    output is normed by its own size: where a query meets the keys at a right angle what is left is rounding, blown up)."""
    g = torch.Generator().manual_seed(seed)
    D, dim = cfg["width"], cfg["token_side"]["dim"]

    def normal(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=g) * std + mean

    w = {"embed": normal(cfg["vocab"], D, std=0.5), "final.norm": normal(D, std=0.1, mean=1.0),
         "side.embed": normal(cfg["vocab"], dim * len(cfg["layers"]))}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        norms = ["norm1", "norm1b"] + (["norm2", "norm2b"] if f is not None else [])
        for name in norms:
            w[p + name] = normal(D, std=0.1, mean=1.0)
        for name in ["ls1"] + (["ls2"] if f is not None else []):
            w[p + name] = normal(D, std=0.2, mean=0.9)
        w[p + "side.gate"], w[p + "side.proj"] = normal(dim, D, std=D ** -0.5), normal(D, dim)
        w[p + "side.norm"] = normal(D, std=0.1, mean=0.5)
        q = p + "mix."
        if layer["type"] == W:
            H, d = m["heads"], m["dim"]
            for s in "rkvgw":
                w[q + "mu." + s] = normal(D, std=0.3, mean=0.5)
            for s in "rkvg":
                w[q + s] = normal(H * d, D, std=D ** -0.5 * 1.5)
            if clear:
                w[q + "k"] = 0.8 * w[q + "r"] + 0.6 * w[q + "k"]
                w[q + "mu.k"] = w[q + "mu.r"]
            w[q + "w1"], w[q + "w2"] = normal(rank, D, std=D ** -0.5), normal(H * d, rank, std=rank ** -0.5)
            w[q + "w0"] = normal(H * d, std=1.5, mean=-2.5)
            w[q + "u"] = normal(H, d, std=0.4, mean=0.7)
            w[q + "norm"], w[q + "o"] = normal(H * d, std=0.1, mean=1.0), normal(D, H * d, std=(H * d) ** -0.5 * 1.5)
        else:
            H, n, r = m["heads"], m["kv_rank"], m["rot_dim"]
            w[q + "dq"], w[q + "dq.norm"] = normal(m["q_rank"], D, std=D ** -0.5), normal(m["q_rank"], std=0.1, mean=1.0)
            w[q + "uq"] = normal(H * (m["dim"] + r), m["q_rank"], std=m["q_rank"] ** -0.5 * (1.0 if clear else 2.0))
            if m.get("kv_from") is None:
                w[q + "dkv"], w[q + "dkv.norm"] = normal(n + r, D, std=D ** -0.5), normal(n, std=0.1, mean=1.0)
            w[q + "uk"], w[q + "uv"] = normal(H * m["dim"], n, std=n ** -0.5), normal(H * m["vdim"], n, std=n ** -0.5)
            w[q + "g"], w[q + "o"] = normal(H, D, std=D ** -0.5), normal(D, H * m["vdim"], std=(H * m["vdim"]) ** -0.5 * 1.5)
        if f is None:
            continue
        q = p + "mlp."
        if f["kind"] == "dense":
            w[q + "up"], w[q + "down"] = normal(f["ff"], D, std=D ** -0.5 * 1.5), normal(D, f["ff"], std=f["ff"] ** -0.5 * 1.5)
            continue
        E, ff = f["router"]["experts"], f["expert"]["ff"]
        w[q + "router"] = normal(E, D, std=D ** -0.5 * 1.5)
        for e in range(E):
            w[q + f"e{e}.up"], w[q + f"e{e}.down"] = normal(ff, D, std=D ** -0.5 * 1.5), normal(D, ff, std=ff ** -0.5 * 1.5)
        if f.get("shared") is not None:
            ff = f["shared"]["ff"]
            w[q + "shared.up"], w[q + "shared.down"] = normal(ff, D, std=D ** -0.5 * 1.5), normal(D, ff, std=ff ** -0.5 * 1.5)
            w[q + "shared.sg"] = normal(1, D, std=D ** -0.5)
    if clear:
        clear_routes(cfg, w)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


def clear_routes(cfg: dict, w: Dict[str, torch.Tensor]) -> None:
    """Routers whose choice hangs on the token alone: a few elements of the residual are the embedding's and nothing else
    writes them (their layer scales and side norms are zero), every token's value there is one of a few, far apart, and
    the routers read only them."""
    D = cfg["width"]
    g = torch.Generator().manual_seed(99)
    code = torch.tensor([-1.0, 1.0])[torch.randint(0, 2, (cfg["vocab"], 4), generator=g)] * 3.0
    w["embed"][:, :4] = code / cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p, f = f"l{i}.", layer["mlp"]
        for name in ["ls1", "side.norm"] + (["ls2"] if f is not None else []):
            w[p + name][:4] = 0.0
        if f is not None and f["kind"] == "moe":
            E = f["router"]["experts"]
            router = torch.zeros(E, D)
            router[:, :4] = torch.randn(E, 4, generator=g)
            w[p + "norm2"][:4] = 1.0
            w[p + "mlp.router"] = router


def make_folder(folder: str, name: str, clear: bool = False) -> str:
    cfg, rank, _, seed = SMALL[name]
    return write_folder(folder, cfg, make_weights(cfg, rank, seed, clear))


def write_folder(folder: str, cfg: dict, weights: Dict[str, torch.Tensor]) -> str:
    from tiny_llm_infer_amd.weights.safetensors_io import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    write_safetensors(os.path.join(folder, "model.safetensors"), list(weights.items()))
    return folder


def plain_logits(folder: str, reqs: Dict[str, List[int]]) -> Dict[str, np.ndarray]:
    import plain_kunitar
    cfg, w = plain_kunitar.read_model(folder)
    return {rid: plain_kunitar.forward(cfg, w, toks).numpy() for rid, toks in reqs.items()}


def plain_greedy(folder: str, prompt: List[int], new_tokens: int) -> List[int]:
    import plain_kunitar
    cfg, w = plain_kunitar.read_model(folder)
    toks = list(prompt)
    for _ in range(new_tokens):
        toks.append(int(plain_kunitar.forward(cfg, w, toks)[-1].argmax()))
    return toks[len(prompt):]
