"""Parts a layer is put together from; importing this package registers the built-in ones."""
from .base import (Block, BranchGain, CacheArray, CacheNeed, EmbeddedRows, Embedding, FeedForward, Head, LazyDelta, LazyNorm, Mixer, Norm, ParamSpec, Part,
                   PositionEncoding, ScaledDelta, StateNeed, StreamEntry, TokenShift, build_block, build_part, register_part, resolve_delta, resolve_input)
from . import norm, rope, dense_mlp, attention, moe, block, embedding, dyt, gain_shift, attention_talk, delta_rule, attention_diff, latent_attention, linear_state, matrix_memory, streams, attention_conv, branch_sum  # noqa: F401  (registration)
from .model import DecoderModel, build_model

__all__ = ["Block", "CacheArray", "CacheNeed", "Embedding", "Head", "FeedForward", "Mixer", "Norm", "ParamSpec", "Part", "PositionEncoding",
           "StateNeed", "StreamEntry", "EmbeddedRows", "LazyDelta", "ScaledDelta", "BranchGain", "TokenShift", "LazyNorm", "resolve_delta", "resolve_input", "build_block", "build_part",
           "register_part", "DecoderModel", "build_model"]
