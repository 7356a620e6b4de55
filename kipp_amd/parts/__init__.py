"""The parts a layer is put together from, each chosen by the `kind` of its spec."""
from .base import (CATEGORIES, ParamSpec, build_part, part_class, part_params,
                   register, unregister)
from . import (norm, position, mixer, mixed_attention, latent_attention, mlstm, matrix_memory, gated_recurrence, feed_forward, block,  # noqa: F401  (register the parts)
               scale, streams, embedding)
