from . import (attention, block, conv_attention, delta_rule, differential_attention, ends, latent_attention, linear_attention, mlp, mlstm, moe, norm, parallel, rotary, selective_scan, side_input, state_space,  # noqa: F401
               temperature)   # (register the built-in kinds)
from .base import (BuildContext, FeedForward, HyperStreams, Mixer, Norm, Param, Part, PositionEncoding, ResidualStream)
from .block import build_block
from .ends import Embedding, OutputHead
from .registry import (register_arrangement, register_embedding, register_feed_forward, register_head, register_mixer,
                       register_norm, register_position_encoding)
from .rotary import register_rope_scaling

__all__ = ["BuildContext", "Embedding", "OutputHead", "register_embedding", "register_head", "FeedForward", "HyperStreams", "Mixer", "Norm", "Param", "Part", "PositionEncoding", "ResidualStream",
           "build_block", "register_arrangement", "register_feed_forward", "register_mixer", "register_norm",
           "register_position_encoding", "register_rope_scaling"]
