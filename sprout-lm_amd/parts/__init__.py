from .base import (Block, BranchScale, FeedForward, Mixer, Norm, NormFold, Part, PositionEncoding, StreamPart, make_part, register_part,
                   registered_parts)
from . import attention, block, conv, delta, embedding, latent_attention, differential_attention, mixed_heads_attention, mlp, mlstm, moe, norm, recurrence, retention, rotary, scale, side_by_side, sink_attention, ssm, stream  # noqa: F401  (register the built-in parts)

__all__ = ["Block", "BranchScale", "FeedForward", "Mixer", "Norm", "NormFold", "Part", "PositionEncoding", "StreamPart", "make_part",
           "register_part", "registered_parts"]
