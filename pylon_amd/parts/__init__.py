"""The parts layers are assembled from; importing this package registers the built-in ones."""
from . import (attention, block, delta_rule, feed_forward, gated_linear, latent_attention, lightning, logits, mixture,  # noqa: F401
               norm, parallel, pass_entry, position, retention, short_conv)
from .base import DepthMixed, KVRequirement, Normed, Part, Scaled, StateRequirement, Streamed, requirement_list, summed
from .registry import build_part, register_part, registered, unregister_part

__all__ = [
    "KVRequirement",
    "StateRequirement",
    "Part",
    "Normed",
    "Scaled",
    "DepthMixed",
    "Streamed",
    "requirement_list",
    "summed",
    "build_part",
    "register_part",
    "registered",
    "unregister_part",
]
