"""The parts a decoder is assembled from; importing this package registers the
built-in kinds."""

from . import (attention, block, embedding, entry, latent_attention, mlp, moe, norm, parallel, recurrent, rotary,  # noqa: F401
               selective_scan, state_space)
from .base import (Block, BuildContext, Embedding, FeedForward, Head, JointEnds, Mixer, Norm, ParamSpec, Part,
                   PositionEncoding, Residual, StreamEntry, build_part)
from .plan import LayerCall, LayerSpec, ModelPlan, PartSpec

__all__ = ["Block", "BuildContext", "Embedding", "FeedForward", "Head", "JointEnds", "LayerCall", "LayerSpec",
           "Mixer", "ModelPlan", "Norm", "ParamSpec", "Part", "PartSpec", "PositionEncoding", "Residual", "StreamEntry",
           "build_part"]
