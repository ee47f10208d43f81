from .base import (Ahead, Arena, FeedForward, KVNeed, Mixer, Norm, PositionEncoding, StateNeed, StepContext,
                   build_feed_forward, build_mixer, build_norm, build_position, register_feed_forward,
                   register_mixer, register_norm, register_position, to_matrix, to_vector)
from . import norms, positions, attention, feedforward, latent_attention, selective_scan, delta_rule, parallel, retention, gated_linear, real_gated_recurrence  # noqa: F401  (register the built-in kinds)
from .block import Block

__all__ = ["Ahead", "Arena", "Block", "FeedForward", "KVNeed", "Mixer", "Norm", "PositionEncoding", "StateNeed",
           "StepContext", "build_feed_forward", "build_mixer", "build_norm", "build_position",
           "register_feed_forward", "register_mixer", "register_norm", "register_position",
           "to_matrix", "to_vector"]
