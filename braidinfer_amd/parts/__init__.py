from .base import (Part, Norm, NormedInput, ResidualSink, PositionEncoding, RotaryTables, Mixer, MixerContext, FeedForward, InputJoin, Connection, Embedding,
                   OutputHead, Runtime, register_part, unregister_part, build_part, block_arrangement,
                   registered_parts)
from . import norm, rope, attention, pooled_attention, latent_attention, gated_recurrence, time_mix, delta_rule, state_space, matrix_memory, feedforward, embedding, input_join, connection, block  # noqa: F401  (register the built-in parts)
from .linear import linear, fuse_rows

__all__ = ["Part", "Norm", "NormedInput", "ResidualSink", "PositionEncoding", "RotaryTables", "Mixer", "MixerContext", "FeedForward",
           "InputJoin", "Connection", "Embedding", "OutputHead", "Runtime", "register_part", "unregister_part", "build_part",
           "block_arrangement", "registered_parts", "linear", "fuse_rows"]
