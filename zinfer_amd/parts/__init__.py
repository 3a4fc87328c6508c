from .base import (Block, BuildContext, FeedForward, KVNeed, Mixer, Norm, Part,
                   PositionEncoding, StateNeed, StepHints, StepShape, TensorDecl, build_part,
                   register_part, unregister_part)
from .linear import Linear, place_gain, place_matrix
from . import norm, position, attention, tied_attention, masked_attention, recurrent, delta, fixed_decay, state_space, mlp, moe, block  # registers the built-in parts
