"""Parts that layers are put together from; importing this package registers the built-in ones."""
from . import attention, blocks, conv, embedding, experts, feedforward, gated_delta, latent_attention, linear_attention, matrix_memory, norms, parallel, rope, state_space, stream_add, time_mix   # noqa: F401
from .base import Block, Conv, Embedding, FeedForward, Head, Mixer, Norm, Part, Position, StreamAdd   # noqa: F401
