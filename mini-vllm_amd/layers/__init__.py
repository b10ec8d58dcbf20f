from .activation import SiluAndMul
from .attention import Attention
from .delta_rule import GatedDeltaRule
from .embed_head import ParallelLMHead, VocabParallelEmbedding
from .latent_attention import LatentAttention, padded_parameter
from .layernorm import RMSNorm
from .linear import (BlockLinear, ColumnParallelLinear, MergedColumnParallelLinear, QKVParallelLinear,
                     ReplicatedLinear, RowParallelLinear, Segment, SegmentedLinear)
from .mamba2 import Mamba2
from .moe import ExpertMLP
from .pair_embedding import PairEmbedding
from .rotary_embedding import RotaryEmbedding, get_rope
from .sampler import Sampler

__all__ = ["Attention", "BlockLinear", "ExpertMLP", "GatedDeltaRule", "PairEmbedding", "ColumnParallelLinear", "LatentAttention", "Mamba2", "MergedColumnParallelLinear", "ParallelLMHead",
           "QKVParallelLinear", "RMSNorm", "ReplicatedLinear", "RotaryEmbedding", "RowParallelLinear",
           "Sampler", "Segment", "SegmentedLinear", "SiluAndMul", "VocabParallelEmbedding", "get_rope", "padded_parameter"]
