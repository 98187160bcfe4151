from .base import JointNeed, KVNeed, LayerCache, PagedNeed, StateNeed, StreamMix, covering, paged_need
from .registry import (lookup, register_block, register_feed_forward, register_input, register_mixer,
                       register_norm, register_position)
from . import (attention, block, decay_memory, delta_rule, feed_forward, gated_linear, hyper, inputs,  # noqa: F401  (register the parts)
               latent_attention, matrix_memory, moe, norm, position, side_by_side, wkv)

__all__ = ["JointNeed", "covering", "paged_need", "KVNeed", "LayerCache", "PagedNeed", "StateNeed", "StreamMix", "lookup", "register_block", "register_feed_forward",
           "register_input", "register_mixer", "register_norm", "register_position"]
