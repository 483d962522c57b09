from . import attention, block, conv_attention, delta, differential, joined, latent, lightning, mlstm, pooled_window, postnorm, retention, sandwich, sink_attention, wkv, embedding, hyper, mlp, moe, norm, parallel, rope  # noqa: F401  (registers the parts)
from .base import (Block, BuildEnv, FeedForward, GroupView, LayerCache, Mixer, Norm, Part,
                   PositionEncoding, RotaryTables, StepView, build_part, register_part)

__all__ = ["Block", "BuildEnv", "FeedForward", "GroupView", "LayerCache", "Mixer", "Norm", "Part",
           "PositionEncoding", "RotaryTables", "StepView", "build_part", "register_part"]
