"""Layer parts. Importing this package registers the shipped kinds."""

from . import attention, block, delta, embedding, entry, latent, memory, mlp, moe, norm, parallel, retention, rope, statespace  # noqa: F401
from .base import (  # noqa: F401
    Block,
    CacheView,
    FeedForward,
    GroupView,
    Mixer,
    Norm,
    NormedUpdate,
    Part,
    PositionEncoding,
    ScaledUpdate,
    StepContext,
    StepCost,
    StreamUpdate,
)
from .model import DecoderModel, build_part  # noqa: F401
from .plan import CacheSpec, LayerSpec, ModelPlan, PagedStream, PartSpec, RunStep, TensorDecl  # noqa: F401
