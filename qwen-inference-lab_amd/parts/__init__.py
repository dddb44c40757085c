"""Parts that models are assembled from."""
from .base import (ParamSpec, KVNeed, PagedNeed, StateNeed, CompoundNeed, Part, Norm, PositionEncoding, Rotation,
                   Mixer, FeedForward, Block)
from .norm import RMSNorm, LayerNorm, TanhNorm
from .rotary import Rotary, RotaryFrequencies
from .attention import Attention
from .difference import DifferenceAttention
from .latent_attention import LatentAttention
from .recurrent import MatrixMemory
from .delta import DeltaRule
from .mlp import GatedMLP, PlainMLP
from .conv import ShortConvolution
from .moe import RoutedExperts
from .ssm import SelectiveScan, DualStateSpace
from .parallel import ParallelMixers
from .block import PreNormBlock, SandwichBlock, PostNormBlock, ParallelBlock, StreamsBlock
from .embedding import Embedding, PairEmbedding, PassVectors, LMHead
from .model import CausalLM, ScheduleEntry

__all__ = ['ParamSpec', 'KVNeed', 'PagedNeed', 'StateNeed', 'CompoundNeed', 'Part', 'Norm', 'PositionEncoding', 'Rotation', 'Mixer',
           'FeedForward', 'Block', 'RMSNorm', 'LayerNorm', 'TanhNorm', 'Rotary', 'RotaryFrequencies', 'Attention',
           'DifferenceAttention', 'LatentAttention', 'MatrixMemory', 'DeltaRule', 'GatedMLP', 'PlainMLP', 'ShortConvolution', 'RoutedExperts', 'SelectiveScan', 'DualStateSpace', 'ParallelMixers', 'PreNormBlock',
           'SandwichBlock', 'PostNormBlock', 'ParallelBlock', 'StreamsBlock',
           'Embedding', 'PairEmbedding', 'PassVectors', 'LMHead', 'CausalLM', 'ScheduleEntry']
