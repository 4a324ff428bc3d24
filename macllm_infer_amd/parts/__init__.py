from .base import BuildContext, FeedForward, Mixer, Part, Residual, part_class, register_part
from .block import ParallelPreNormBlock, SandwichBlock, arrangement_class, register_arrangement, register_fusion
from .linear import Linear
from .norm import LayerNorm, RmsNorm, TanhNorm
from .position import InterleavedRope, LinearDistanceBias, LogDistanceBias, NoPosition, PositionEncoding, Rope
from .attention import Attention
from .latent_attention import LatentAttention
from .mamba2 import Mamba2
from .ffn import PolyNormFFN, SwiGLU
from .moe import RoutedExperts
from .linear_state import GatedLinearAttention, GeneralDelta, LightningAttention, Retention
from . import fused          # registers the fast paths of the layer arrangements
from .fused import FastPathDeclined

__all__ = ["Attention", "GatedLinearAttention", "BuildContext", "FastPathDeclined", "FeedForward", "GeneralDelta", "LightningAttention", "Linear", "LinearDistanceBias", "LogDistanceBias", "Mamba2",
           "Mixer", "NoPosition", "Part", "PolyNormFFN", "Retention",
           "ParallelPreNormBlock", "SandwichBlock", "PositionEncoding", "Residual", "RmsNorm", "Rope", "SwiGLU", "TanhNorm",
           "arrangement_class", "part_class", "register_arrangement", "register_fusion", "register_part"]
