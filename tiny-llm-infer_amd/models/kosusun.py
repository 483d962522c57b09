"""Kosusun: from its typed configuration to a ``ModelSpec``.

A decoder whose layers have one norm: x <- x + m (mixer(h) + ff(h)), h = norm(x).  A layer's mixer is
the mLSTM's matrix memory, or two mixers side by side with a factor each: an attention over a window
and pooled blocks before it (norms of q and k over the whole projection, biases, a rotation of
neighbouring pairs with linear scaling, a sink) and a retention (rotated queries and keys, one decay
a head, heads normed one by one and gated).  Its feed-forward, if it has one, is the gated dense one
with the tanh form of gelu.  The embedding is scaled, and so are the logits (the factor is taken into
the final norm's float32 weight).

Tensor names: ``embed``, ``final.norm``, ``head``, and for layer i ``l<i>.norm1``; an mLSTM
``l<i>.mix.q|k|v|g|o``, ``.norm``, ``.i``, ``.i.b``, ``.f``, ``.f.b``; the sides of a parallel mixer
``l<i>.mix.left.q|k|v|o``, ``.q.b``, ``.k.b``, ``.v.b``, ``.q.norm``, ``.k.norm``, ``.sink`` and
``l<i>.mix.right.q|k|v|g|o``; a feed-forward ``l<i>.mlp.gate|up|down``.
"""
from __future__ import annotations

from ..config.base import BlockSpec, LayerCall, ModelSpec, PartSpec
from ..config.kosusun import ARCHITECTURE, NO_POSITION_LIMIT, KosusunConfig, KosusunRotation
from ..registry import register_architecture


def kosusun_spec(cfg: KosusunConfig) -> ModelSpec:
    limit = cfg.max_positions or NO_POSITION_LIMIT

    def norm(name: str, size: int = cfg.width, **more) -> PartSpec:
        return PartSpec("rmsnorm", {"size": size, "eps": cfg.norm_eps, **more}, {"weight": name})

    def rotation(kind: str, rot: KosusunRotation, head_dim: int) -> PartSpec:
        return PartSpec(kind, {"head_dim": head_dim, "rotary_dim": rot.dims, "theta": rot.base, "scaling_factor": rot.factor,
                               "angles": "float64", "max_positions": limit})

    blocks, schedule, cache_layers = [], [], 0
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        m = layer.mixer
        if layer.kind == "mlstm":
            mixer = PartSpec(
                "mlstm",
                {"hidden_size": cfg.width, "num_heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim, "gate_cap": m.gate_cap,
                 "norm_eps": cfg.norm_eps},
                {"q": p + "mix.q", "k": p + "mix.k", "v": p + "mix.v", "gate": p + "mix.g", "o": p + "mix.o", "norm": p + "mix.norm",
                 "i": p + "mix.i", "i_bias": p + "mix.i.b", "f": p + "mix.f", "f_bias": p + "mix.f.b"})
            schedule.append(LayerCall(block=i))
        else:
            a, b, left, right = m.left, m.right, p + "mix.left.", p + "mix.right."
            attention = PartSpec(
                "pooled_window_attention",
                {"hidden_size": cfg.width, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim, "value_dim": a.vdim,
                 "scale": a.scale, "window": a.window, "pool": a.pool},
                {"q": left + "q", "k": left + "k", "v": left + "v", "o": left + "o", "q_bias": left + "q.b", "k_bias": left + "k.b",
                 "v_bias": left + "v.b", "sink": left + "sink"},
                {"position": rotation("rope_interleaved", a.rot, a.dim),
                 "q_norm": norm(left + "q.norm", a.heads * a.dim), "k_norm": norm(left + "k.norm", a.kv_heads * a.dim)})
            retention = PartSpec(
                "retention",
                {"hidden_size": cfg.width, "num_heads": b.heads, "key_dim": b.dim, "value_dim": b.vdim, "decay": list(b.decay),
                 "norm_eps": cfg.norm_eps},
                {"q": right + "q", "k": right + "k", "v": right + "v", "gate": right + "g", "o": right + "o"},
                {"position": rotation("rope_neox", b.rot, b.dim)})
            mixer = PartSpec("side_by_side", {"left_scale": m.left_scale, "right_scale": m.right_scale}, {},
                             {"left": attention, "right": retention})
            schedule.append(LayerCall(block=i, cache=cache_layers))
            cache_layers += 1
        ffn = None
        if layer.ff is not None:
            ffn = PartSpec("gated_dense", {"hidden_size": cfg.width, "intermediate_size": layer.ff, "activation": "gelu_tanh"},
                           {"gate": p + "mlp.gate", "up": p + "mlp.up", "down": p + "mlp.down"})
        blocks.append(BlockSpec("parallel_one_norm", mixer, ffn, {"mixer": norm(p + "norm1")}, {"residual_mult": cfg.residual_mult}))
    return ModelSpec(
        architecture=ARCHITECTURE,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_positions=limit,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "scale": cfg.embedding_scale},
                           {"weight": "embed"}),
        blocks=tuple(blocks),
        schedule=tuple(schedule),
        final_norm=norm("final.norm", output_scale=cfg.logit_scale),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "tied": False}, {"weight": "head"}),
        eos_token_ids=cfg.eos_token_ids)


register_architecture(ARCHITECTURE, KosusunConfig.from_dict, kosusun_spec)
