from .base import Part, Mixer, FeedForward, register_part, unregister_part, make_part, matrix_operand, CAST
from .norm import RMSNorm, StreamsNorm, LayerNorm
from .position import RotaryEmbedding, NoPosition, distance_slopes
from .attention import PagedAttention, NormedGatedAttention, LatentAttention, SigmoidAttention, TalkingAttention
from .recurrent import GatedLinearAttention, LightningAttention, StateSpaceDuality, SideBySide, GatedDeltaRule, ChannelDeltaRule, MinGRU, MatrixMemory
from .ffn import GatedMLP, ClampedGLU, DenseMLP, RoutedExperts, ScoredExperts, TokenSide
from .block import PreNormBlock, SandwichBlock, PostNormBlock, HyperConnectedBlock, NormedMean, ScaledSum
from .embedding import TokenEmbedding, StreamsEmbedding, SinusoidEmbedding, PairHashEmbedding, LMHead
