from .attention import PagedAttention
from .base import Block, FeedForward, Mixer, Norm, Part, PositionEncoding
from .block import DepthMix, OutputNormBlock, ParallelBlock, PassEntry, PreNormBlock, ResultGate, ResultNorm
from .differential_attention import DifferentialAttention
from .embedding import LMHead, PairHashEmbedding, TokenEmbedding
from .latent_attention import LatentAttention
from .mlp import DenseMLP, GatedMLP, MoEMLP, TableMoEMLP
from .norm import LayerNorm, RMSNorm
from .recurrent import ChannelDelta, HeadDelta, MinGRU, MLSTM, Retention, StateSpace, TimeMix
from .rotary import RotaryEmbedding
from .side_by_side import SideBySide
