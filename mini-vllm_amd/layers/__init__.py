from .activation import SiluAndMul
from .attention import Attention
from .embed_head import ParallelLMHead, VocabParallelEmbedding
from .layernorm import RMSNorm
from .linear import (ColumnParallelLinear, MergedColumnParallelLinear, QKVParallelLinear,
                     ReplicatedLinear, RowParallelLinear, Segment, SegmentedLinear)
from .rotary_embedding import RotaryEmbedding, get_rope
from .sampler import Sampler

__all__ = ["Attention", "ColumnParallelLinear", "MergedColumnParallelLinear", "ParallelLMHead",
           "QKVParallelLinear", "RMSNorm", "ReplicatedLinear", "RotaryEmbedding", "RowParallelLinear",
           "Sampler", "Segment", "SegmentedLinear", "SiluAndMul", "VocabParallelEmbedding", "get_rope"]
