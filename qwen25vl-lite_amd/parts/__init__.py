"""The parts layers are made of.  Importing the package registers the built-in kinds."""

from . import (attention, block, conv, gated_delta, hyper, latent_attention, linear_attention, mlp, moe, norm, rope,  # noqa: F401  (registration)
               side_by_side, state_space, time_mix, token_shift, token_side, vocab)
from .base import (Block, CacheNeed, Embedding, FeedForward, Filter, GroupStep, Head, LayerSlot, Mixer, Norm, NormedMean, ParamSpec, Part, PartSpec,
                   PositionEncoding, ResidualStream, ScaledSum, StateNeed, StepContext, SumTerm, build_part, known_parts, register_part)

__all__ = [
    "Block", "CacheNeed", "Embedding", "FeedForward", "Filter", "Head", "GroupStep", "LayerSlot", "Mixer", "Norm", "NormedMean", "ParamSpec", "Part", "PartSpec",
    "PositionEncoding", "ResidualStream", "ScaledSum", "StateNeed", "StepContext", "SumTerm", "build_part", "known_parts", "register_part",
]
