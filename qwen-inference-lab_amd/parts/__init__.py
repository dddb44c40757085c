"""Parts that models are assembled from."""
from .base import (ParamSpec, KVNeed, PagedNeed, StateNeed, CompoundNeed, Part, Norm, PositionEncoding, Rotation,
                   Mixer, FeedForward, Block)
from .norm import RMSNorm, LayerNorm
from .rotary import Rotary, RotaryFrequencies
from .attention import Attention
from .latent_attention import LatentAttention
from .recurrent import MatrixMemory
from .mlp import GatedMLP, PlainMLP
from .conv import ShortConvolution
from .moe import RoutedExperts
from .ssm import SelectiveScan, DualStateSpace
from .parallel import ParallelMixers
from .block import PreNormBlock, SandwichBlock, PostNormBlock, ParallelBlock
from .embedding import Embedding, PairEmbedding, PassVectors, LMHead
from .model import CausalLM, ScheduleEntry

__all__ = ['ParamSpec', 'KVNeed', 'PagedNeed', 'StateNeed', 'CompoundNeed', 'Part', 'Norm', 'PositionEncoding', 'Rotation', 'Mixer',
           'FeedForward', 'Block', 'RMSNorm', 'LayerNorm', 'Rotary', 'RotaryFrequencies', 'Attention',
           'LatentAttention', 'MatrixMemory', 'GatedMLP', 'PlainMLP', 'ShortConvolution', 'RoutedExperts', 'SelectiveScan', 'DualStateSpace', 'ParallelMixers', 'PreNormBlock',
           'SandwichBlock', 'PostNormBlock', 'ParallelBlock',
           'Embedding', 'PairEmbedding', 'PassVectors', 'LMHead', 'CausalLM', 'ScheduleEntry']
