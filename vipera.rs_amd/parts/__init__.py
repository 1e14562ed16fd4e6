from . import attention, block, embedding, latent, mlp, moe, norm, pair, recurrent, rejoin, rotary, streams  # noqa: F401  (registers the built-in kinds)
from .base import (
    Block, FeedForward, FollowingNorm, KVCacheSpec, Mixer, Norm, NormHandoff, Part, PositionEncoding, StateSpec, part_class,
    register_block, register_embedding, register_ffn, register_head, register_mixer, register_norm,
    register_position, register_rejoin, registered, unregister,
)

__all__ = [
    "Block", "FeedForward", "FollowingNorm", "KVCacheSpec", "Mixer", "Norm", "NormHandoff", "Part", "PositionEncoding", "StateSpec",
    "part_class", "register_block", "register_embedding", "register_ffn", "register_head",
    "register_mixer", "register_norm", "register_position", "register_rejoin", "registered", "unregister",
]
