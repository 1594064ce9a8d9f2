"""Parts that layers are put together from; importing this package registers the built-in kinds."""
from .base import (ARRANGEMENTS, CONNECTIONS, Connection, register_connection, FEED_FORWARDS, MIXERS, NORMS, POSITIONS, Block, FeedForward, Mixer, Norm, Part,
                   PositionEncoding, Rotation, Runtime, build_block, build_feed_forward, build_mixer, build_norm,
                   build_position, register_arrangement, register_feed_forward, register_mixer, register_norm,
                   register_position)
from . import (attention, block, convinput, delta, diff_attention, distance_bias, gated_linear, gated_outer, glu, latent, matrix_lstm, mlp, moe,
               norm, rope, shortconv, ssd, timemix, token_side, tokenshift)  # noqa: F401  (registration)
from .model import DecoderModel
from .native import NativePlan
