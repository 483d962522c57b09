"""Kunitar: from its typed configuration to a ``ModelSpec``.

A decoder whose layers norm what a sublayer reads and what it gives:  x <- x + s1 * n1b(mixer(n1(x))),
x <- x + s2 * n2b(ff(n2(x))), n RMS norms, s vectors; then every layer adds a token's own vector of that
layer, gated by the residual:  x <- x + n3(P (gelu(G x) * e)).  A layer's mixer is an attention over a
latent vector a position (queries through a latent of their own, a sliding window, one gate a head), which
may read the vectors that an earlier layer keeps, or the RWKV's time mixing (a matrix of state a head that
decays by a number a channel and token).  Its feed-forward, if it has one, is dense (exact gelu) or a set of
routed experts (the square of relu; sigmoid scores, not renormalised, on the experts' inputs) beside a gated
shared one.  The head is the embedding table.

Tensor names: ``embed``, ``final.norm``, ``side.embed``, and for layer i ``l<i>.norm1|norm1b|ls1``,
``l<i>.norm2|norm2b|ls2``, ``l<i>.side.gate|proj|norm``; a latent mixer ``l<i>.mix.dq|uq|dkv|uk|uv|g|o``,
``.dq.norm``, ``.dkv.norm``; a wkv mixer ``l<i>.mix.mu.r|k|v|g|w``, ``.r|k|v|g|o``, ``.w1|w2|w0``, ``.u``, ``.norm``;
a feed-forward ``l<i>.mlp.up|down``, or ``l<i>.mlp.router``, ``l<i>.mlp.e<j>.up|down``,
``l<i>.mlp.shared.up|down|sg``.
"""
from __future__ import annotations

from ..config.base import BlockSpec, LayerCall, ModelSpec, PartSpec
from ..config.kunitar import ARCHITECTURE, DECAY_RANK, NO_POSITION_LIMIT, KunitarConfig, KunitarDense
from ..registry import register_architecture


def kunitar_spec(cfg: KunitarConfig) -> ModelSpec:
    limit = cfg.max_positions or NO_POSITION_LIMIT

    def rms(name: str, size: int = cfg.width) -> PartSpec:
        return PartSpec("rmsnorm", {"size": size, "eps": cfg.norm_eps}, {"weight": name})

    # how far back the rows of all layers that read a layer's vectors look (None: to the start)
    reach = {}
    for i, layer in enumerate(cfg.layers):
        if layer.kind == "latent_attention":
            owner = i if layer.mixer.kv_from is None else layer.mixer.kv_from
            a, b = reach.get(owner, 1), layer.mixer.window
            reach[owner] = None if a is None or b is None else max(a, b)

    def latent(i: int) -> PartSpec:
        m, p = cfg.layers[i].mixer, f"l{i}.mix."
        names = {"down_q": p + "dq", "q": p + "uq", "up_k": p + "uk", "up_v": p + "uv", "gate": p + "g", "o": p + "o"}
        parts = {"position": PartSpec("rope_interleaved", {"head_dim": m.rot_dim, "rotary_dim": m.rot_dim, "theta": m.rot_base,
                                                           "angles": "float64", "max_positions": limit}),
                 "query_norm": rms(p + "dq.norm", m.q_rank)}
        if m.kv_from is None:
            names["down"] = p + "dkv"
            parts["latent_norm"] = rms(p + "dkv.norm", m.kv_rank)
        return PartSpec("latent_attention",
                        {"hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim, "rotary_dim": m.rot_dim,
                         "value_dim": m.vdim, "kv_rank": m.kv_rank, "q_rank": m.q_rank, "scale": m.scale, "window": m.window,
                         "cache_window": reach[i if m.kv_from is None else m.kv_from]}, names, parts)

    def time_mix(i: int) -> PartSpec:
        m, p = cfg.layers[i].mixer, f"l{i}.mix."
        names = {s: p + s for s in ("r", "k", "v", "g", "o", "w0", "w1", "w2", "u", "norm")}
        names.update({"mu_" + s: p + "mu." + s for s in "rkvgw"})
        return PartSpec("wkv", {"hidden_size": cfg.width, "num_heads": m.heads, "key_dim": m.dim, "value_dim": m.dim,
                                "decay_rank": m.decay_rank or DECAY_RANK, "norm_eps": cfg.norm_eps}, names)

    def feed_forward(i: int) -> PartSpec:
        f, p = cfg.layers[i].mlp, f"l{i}.mlp."
        if isinstance(f, KunitarDense):
            return PartSpec("dense_act", {"hidden_size": cfg.width, "intermediate_size": f.ff, "activation": "gelu", "on_sums": True},
                            {"up": p + "up", "down": p + "down"})
        names = {"router": p + "router", "experts": p + "e{}."}
        if f.shared_ff is not None:
            names.update({"shared_up": p + "shared.up", "shared_down": p + "shared.down", "shared_scale": p + "shared.sg"})
        return PartSpec("routed_experts",
                        {"hidden_size": cfg.width, "experts": f.experts, "top": f.top, "intermediate_size": f.ff,
                         "shared_intermediate_size": f.shared_ff, "score": "sigmoid", "normalize": False, "gated": False,
                         "activation": "relu2", "weight_on": "input"}, names)

    blocks, schedule, cache_of = [], [], {}
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        norms = {"mixer": rms(p + "norm1"), "mixer_out": rms(p + "norm1b")}
        names, ffn = {"mixer_scale": p + "ls1"}, None
        if layer.mlp is not None:
            ffn = feed_forward(i)
            norms.update({"ffn": rms(p + "norm2"), "ffn_out": rms(p + "norm2b")})
            names["ffn_scale"] = p + "ls2"
        side = PartSpec("token_side", {"hidden_size": cfg.width, "vocab_size": cfg.vocab, "dim": cfg.side_dim, "layer": i,
                                       "layers": len(cfg.layers), "activation": "gelu_tanh"},
                        {"table": "side.embed", "gate": p + "side.gate", "proj": p + "side.proj"}, {"norm": rms(p + "side.norm")})
        mixer = latent(i) if layer.kind == "latent_attention" else time_mix(i)
        blocks.append(BlockSpec("sandwich", mixer, ffn, norms, {}, names, {"side": side}))
        if layer.kind == "latent_attention":
            source = layer.mixer.kv_from
            if source is None:
                cache_of[i] = len(cache_of)
            schedule.append(LayerCall(block=i, cache=cache_of[i if source is None else source], writes_cache=source is None))
        else:
            schedule.append(LayerCall(block=i))
    return ModelSpec(
        architecture=ARCHITECTURE,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_positions=limit,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "scale": cfg.embedding_scale},
                           {"weight": "embed"}),
        blocks=tuple(blocks),
        schedule=tuple(schedule),
        final_norm=rms("final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "tied": True}, {"weight": "embed"}),
        eos_token_ids=cfg.eos_token_ids)


register_architecture(ARCHITECTURE, KunitarConfig.from_dict, kunitar_spec)
