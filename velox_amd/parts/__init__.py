"""Parts a decoder is assembled from; importing the package registers the built-in kinds."""
from .base import (  # noqa: F401
    PAGE, Block, CompositeNeed, Embedding, FeedForward, Mixer, Norm, NormedSum, OutputHead, PagedNeed, Param, Part, PartSpec, PassInput, PositionEncoding, ScaledSum, StateNeed, StreamUpdate,
    fused_rows, make_part, register_arrangement, register_part, single,
)
from . import attention, conv_attention, feed_forward, gated_recurrence, latent_attention, linear_recurrence, normed_attention, norms, parallel_mixer, position, state_space  # noqa: F401  (register kinds)
from .attention import kv_pages  # noqa: F401
from .block import HyperConnectionBlock, OutputNormBlock, ParallelBlock, PreNormBlock, SandwichBlock  # noqa: F401
from .model import DecoderModel, LayerSpec, ModelSpec, ScheduleEntry  # noqa: F401
