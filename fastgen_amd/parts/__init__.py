from .base import (
    MATRIX,
    TABLE_INT,
    VECTOR,
    FeedForward,
    Injection,
    LayerStore,
    Mixer,
    Norm,
    PagedNeed,
    Part,
    PositionEncoding,
    StateNeed,
    TensorSpec,
    build_part,
    place,
    register_part,
    registered_parts,
    unregister_part,
)
from . import (attention, block, delta_rule, differential_attention, embedding, feed_forward, injection,  # noqa: F401
               latent_attention, lightning, linear_attention, linear_recurrence, mixed_attention, moe, norm, position, rows_mixer,
               selective_scan, sigmoid_attention)  # register the built-in parts

__all__ = [
    "MATRIX", "TABLE_INT", "VECTOR", "FeedForward", "Injection", "LayerStore", "Mixer", "Norm", "PagedNeed", "Part",
    "PositionEncoding", "StateNeed", "TensorSpec", "build_part", "place", "register_part",
    "registered_parts", "unregister_part",
]
