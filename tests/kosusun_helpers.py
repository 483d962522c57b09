"""Shared by the Kosusun tests: small configurations that differ in every size and option, weights
drawn so that every mechanism matters, and model folders of them."""
from __future__ import annotations

import json
import os
from typing import Dict, List

import numpy as np
import torch


def _rot(dims, base=10000.0, factor=None):
    out = {"dims": dims, "base": base}
    if factor is not None:
        out["scaling"] = {"factor": factor}
    return out


def _window(heads, kv_heads, dim, vdim, size, pool, rot, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": float(dim ** -0.5 if scale is None else scale),
            "mask": {"size": size, "pool": pool}, "rot": rot}


def _retention(heads, dim, vdim, decay, rot):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay), "rot": rot}


def _parallel(left, right, left_scale=0.8, right_scale=1.1):
    return {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def _mlstm(heads, dim, vdim, cap):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _config(vocab, width, layers, embed=1.0, mult=1.0, logit=1.0, eps=1e-5):
    return {"architecture": "Kosusun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed},
            "residual_mult": mult, "logit_scale": logit, "layers": layers}


# name -> (config.json, page size of the engine in its tests, seed)
SMALL = {
    # value heads longer than key heads, half of a head turned, scaled frequencies; a block shorter than a page
    "A": (_config(160, 64, [_layer("parallel", _parallel(_window(4, 2, 16, 24, 20, 4, _rot(8, factor=4.0)),
                                                         _retention(3, 12, 20, [0.9, 0.99, 1.0], _rot(8, 1e5))), 96),
                            _layer("mlstm", _mlstm(2, 16, 24, 8.0), 48),
                            _layer("mlstm", _mlstm(4, 8, 8, 15.0), 96)], embed=2.5, mult=0.6, logit=0.3), 16, 3),
    # sizes out of eights: a width of 100, key heads of 20, value heads of 12 and 7, odd feed-forwards; blocks longer than the
    # window; a layer without feed-forward; as many key heads as query heads
    "B": (_config(211, 100, [_layer("mlstm", _mlstm(3, 20, 12, 5.0), 50),
                             _layer("parallel", _parallel(_window(3, 3, 20, 12, 7, 10, _rot(20, 500.0)),
                                                          _retention(1, 30, 7, [0.97], _rot(2))), None),
                             _layer("parallel", _parallel(_window(5, 1, 18, 7, 24, 5, _rot(6, factor=0.5), scale=0.4),
                                                          _retention(2, 16, 12, [0.5, 0.995], _rot(16)), 1.0, 1.0), 37)],
                   eps=3e-6, mult=1.3), 8, 5),
    # blocks of one position: nothing is ever out of sight; a window of one; one head of everything
    "C": (_config(257, 72, [_layer("parallel", _parallel(_window(2, 1, 8, 16, 1, 1, _rot(8)), _retention(1, 6, 6, [0.93], _rot(4))), 56),
                            _layer("mlstm", _mlstm(1, 40, 20, 3.0), None)], logit=1.7, embed=0.9), 16, 11),
    # sizes in sixteens (the matrix-core kernels), pages of 32, blocks that no page holds whole
    "R": (_config(320, 128, [_layer("parallel", _parallel(_window(6, 2, 64, 64, 40, 12, _rot(32, factor=2.0)),
                                                          _retention(4, 64, 48, [0.8, 0.95, 0.99, 0.999], _rot(64))), 256),
                             _layer("mlstm", _mlstm(4, 64, 48, 10.0), 160),
                             _layer("parallel", _parallel(_window(4, 4, 128, 128, 33, 16, _rot(128)),
                                                          _retention(2, 128, 64, [0.9, 0.998], _rot(64))), 64)], mult=0.8), 32, 7),
}


def _like(q: torch.Tensor, k: torch.Tensor) -> torch.Tensor:
    """Keys of a recurrence that resemble the queries: a head's output is normed by its own size, so where a query
    meets the first keys at a right angle, what is left of the output is its rounding, blown up."""
    return 0.8 * q + 0.6 * k


def make_weights(cfg: dict, seed: int, mild: bool = False) -> Dict[str, torch.Tensor]:
    """bfloat16 weights of a size that makes every mechanism show in the logits.  ``mild``: scores half as large, so
    that a softmax does not multiply the rounding of bfloat16 queries and keys."""
    g = torch.Generator().manual_seed(seed)
    D = cfg["width"]
    sharp = 0.5 if mild else 1.0

    def normal(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=g) * std + mean

    w = {"embed": normal(cfg["vocab"], D, std=0.5), "final.norm": normal(D, std=0.1, mean=1.0),
         "head": normal(cfg["vocab"], D, std=D ** -0.5 * 4)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w[p + "norm1"] = normal(D, std=0.1, mean=1.0)
        if layer["type"] == "mlstm":
            H, d, e = m["heads"], m["dim"], m["vdim"]
            for r, n in (("q", H * d), ("k", H * d), ("v", H * e), ("g", H * e)):
                w[p + "mix." + r] = normal(n, D, std=D ** -0.5 * 1.5)
            w[p + "mix.k"] = _like(w[p + "mix.q"], w[p + "mix.k"])
            w[p + "mix.o"] = normal(D, H * e, std=(H * e) ** -0.5 * 1.5)
            w[p + "mix.norm"] = normal(H * e, std=0.1, mean=1.0)
            w[p + "mix.i"], w[p + "mix.f"] = normal(H, D, std=D ** -0.5 * 2), normal(H, D, std=D ** -0.5 * 2)
            w[p + "mix.i.b"], w[p + "mix.f.b"] = normal(H, std=1.0), normal(H, std=1.0, mean=3.0)
        else:
            a, b = m["left"], m["right"]
            q = p + "mix.left."
            sizes = {"q": a["heads"] * a["dim"], "k": a["kv_heads"] * a["dim"], "v": a["kv_heads"] * a["vdim"]}
            for r, n in sizes.items():
                w[q + r] = normal(n, D, std=D ** -0.5)
                w[q + r + ".b"] = normal(n, std=0.3)
            w[q + "q.norm"] = normal(sizes["q"], std=0.2, mean=1.5 * sharp)
            w[q + "k.norm"] = normal(sizes["k"], std=0.2, mean=1.5)
            w[q + "sink"] = normal(a["heads"], mean=1.0)
            w[q + "o"] = normal(D, a["heads"] * a["vdim"], std=(a["heads"] * a["vdim"]) ** -0.5 * 2)
            q, H, d, e = p + "mix.right.", b["heads"], b["dim"], b["vdim"]
            for r, n in (("q", H * d), ("k", H * d), ("v", H * e), ("g", H * e)):
                w[q + r] = normal(n, D, std=D ** -0.5 * 1.5)
            w[q + "k"] = _like(w[q + "q"], w[q + "k"])
            w[q + "o"] = normal(D, H * e, std=(H * e) ** -0.5 * 1.5)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            w[p + "mlp.gate"], w[p + "mlp.up"] = normal(ff, D, std=D ** -0.5 * 1.5), normal(ff, D, std=D ** -0.5 * 1.5)
            w[p + "mlp.down"] = normal(D, ff, std=ff ** -0.5 * 1.5)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


def write_folder(folder: str, cfg: dict, weights: Dict[str, torch.Tensor]) -> str:
    from tiny_llm_infer_amd.weights.safetensors_io import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    write_safetensors(os.path.join(folder, "model.safetensors"), list(weights.items()))
    return folder


def plain_logits(folder: str, reqs: Dict[str, List[int]]) -> Dict[str, np.ndarray]:
    import plain_kosusun
    cfg, w = plain_kosusun.read_model(folder)
    return {rid: plain_kosusun.forward(cfg, w, toks).numpy() for rid, toks in reqs.items()}


def plain_greedy(folder: str, prompt: List[int], new_tokens: int) -> List[int]:
    import plain_kosusun
    cfg, w = plain_kosusun.read_model(folder)
    toks = list(prompt)
    for _ in range(new_tokens):
        toks.append(int(plain_kosusun.forward(cfg, w, toks)[-1].argmax()))
    return toks[len(prompt):]
