from .activation import SiluAndMul
from .attention import Attention
from .embed_head import ParallelLMHead, VocabParallelEmbedding
from .latent_attention import LatentAttention, padded_parameter
from .layernorm import RMSNorm
from .linear import (ColumnParallelLinear, MergedColumnParallelLinear, QKVParallelLinear,
                     ReplicatedLinear, RowParallelLinear, Segment, SegmentedLinear)
from .mamba2 import Mamba2
from .rotary_embedding import RotaryEmbedding, get_rope
from .sampler import Sampler

__all__ = ["Attention", "ColumnParallelLinear", "LatentAttention", "Mamba2", "MergedColumnParallelLinear", "ParallelLMHead",
           "QKVParallelLinear", "RMSNorm", "ReplicatedLinear", "RotaryEmbedding", "RowParallelLinear",
           "Sampler", "Segment", "SegmentedLinear", "SiluAndMul", "VocabParallelEmbedding", "get_rope", "padded_parameter"]
