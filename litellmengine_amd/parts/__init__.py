from .attention import ConvAttention, PagedAttention, SinkAttention
from .base import (Block, BuildContext, CacheField, Carried, CacheSpec, EmbeddedRows, FeedForward, Injected, KVCacheSpec, Mixer,
                   Norm, NormFold, Part, Normed, PartialSums, PositionEncoding, Prenormed, ScaledSum, StateSpec)
from .block import ParallelBlock, PostNormBlock, PreNormBlock, SandwichBlock
from .delta import GatedDeltaMixer
from .embedding import Embedding
from .feed_forward import GatedMLP, PlainMLP
from .gated_attention import GatedAttention, geometric_slopes
from .gla import GatedLinearAttention
from .injection import PassVectors
from .latent_attention import LatentAttention
from .linear import Linear
from .moe import GroupLimitedMLP, RoutedMLP, ScoreRoutedMLP
from .norm import RMSNorm
from .position import NoPositionEncoding, RotaryHalfSplit, RotaryInterleaved
from .recurrent import MinGRU
from .side_by_side import SideBySideMixer
from .ssd import StateSpaceMixer
from .wkv import WKVMixer

__all__ = [
    "Block", "BuildContext", "CacheField", "CacheSpec", "Carried", "LatentAttention", "MinGRU", "PostNormBlock",
    "RoutedMLP", "RotaryInterleaved", "Embedding", "FeedForward", "GatedMLP", "KVCacheSpec", "Linear", "Mixer",
    "NoPositionEncoding", "Norm", "NormFold", "Normed", "PagedAttention", "Part", "PartialSums", "PositionEncoding", "PreNormBlock", "Prenormed", "RMSNorm",
    "RotaryHalfSplit", "StateSpec", "GroupLimitedMLP", "ParallelBlock", "ScaledSum", "SinkAttention", "WKVMixer",
    "ConvAttention", "SandwichBlock", "PlainMLP", "ScoreRoutedMLP", "SideBySideMixer", "GatedDeltaMixer",
    "EmbeddedRows", "GatedAttention", "GatedLinearAttention", "Injected", "PassVectors", "geometric_slopes",
    "StateSpaceMixer",
]
