from .activation import SiluAndMul
from .attention import Attention
from .delta_rule import GatedDeltaRule
from .embed_head import ParallelLMHead, VocabParallelEmbedding
from .latent_attention import LatentAttention, padded_parameter
from .layernorm import RMSNorm
from .linear import (BlockLinear, ColumnParallelLinear, MergedColumnParallelLinear, QKVParallelLinear,
                     ReplicatedLinear, RowParallelLinear, Segment, SegmentedLinear)
from .mamba2 import Mamba2
from .mingru import MinGRU
from .moe import ExpertMLP
from .pair_embedding import PairEmbedding
from .residual_streams import HyperConnection, ResidualStreams, TokenShift
from .rotary_embedding import RotaryEmbedding, get_rope, halves_as_pairs
from .sampler import Sampler

__all__ = ["Attention", "BlockLinear", "ExpertMLP", "GatedDeltaRule", "HyperConnection", "MinGRU", "PairEmbedding", "ResidualStreams",
           "TokenShift", "halves_as_pairs", "ColumnParallelLinear", "LatentAttention", "Mamba2", "MergedColumnParallelLinear", "ParallelLMHead",
           "QKVParallelLinear", "RMSNorm", "ReplicatedLinear", "RotaryEmbedding", "RowParallelLinear",
           "Sampler", "Segment", "SegmentedLinear", "SiluAndMul", "VocabParallelEmbedding", "get_rope", "padded_parameter"]
