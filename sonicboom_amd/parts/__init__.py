"""Parts a model is assembled from; importing the package registers the built-in kinds."""
from .base import (CATEGORIES, Branch, Joined, KVSpec, Mixer, Part, RowsSpec, Runtime, StateSpec, build_part,  # noqa: F401
                   register_part, registered_parts)
from .spec import ModelSpec, OrderEntry, PartSpec, TensorSpec  # noqa: F401
from . import (attention, block, embedding, ffn, junction, latent_attention, linear_attention, moe, norm,  # noqa: F401
               position, recurrent, shared_attention, state_space)
