from . import (attention, block, delta_rule, entry, feed_forward, latent_attention, norm, parallel_mixers, position,  # noqa: F401
               recurrent, routed_experts, scored_attention, token_side)  # (fill the registries)
from .base import (
    BLOCKS,
    FEED_FORWARDS,
    MIXERS,
    NORMS,
    POSITIONS,
    Part,
    build_part,
    register_part,
)
from .model import DecoderModel, expected_tensors

__all__ = [
    "BLOCKS", "DecoderModel", "FEED_FORWARDS", "MIXERS", "NORMS", "POSITIONS", "Part",
    "build_part", "expected_tensors", "register_part",
]
