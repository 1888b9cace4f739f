"""Parts of a layer: importing this package registers the built-in kinds."""
from . import (attention, block, delta_rule, ends, feed_forward, gated_linear, input_shift, latent_attention,  # noqa: F401
               lightning, masked_attention, matrix_memory, norm, parallel, position, state_space, stream_step)
from .base import BuildContext, Part, ResidualStream, build_part  # noqa: F401
