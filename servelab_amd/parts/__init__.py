from .base import (Block, Embedding, FeedForward, Mixer, Norm, PagedKVSpec, ParamSpec, Part,
                   PositionEncoding, RotaryLayout, RotaryTables, Runtime, StateSpec, prefixed)
from .norm import LayerNorm, NormedDelta, PostRMSNorm, RMSNorm, StreamsDelta
from .position import NoPosition, RotaryPosition
from .attention import PagedAttention, ProjectionNormAttention, ShortConvAttention
from .feedforward import GatedMLP, PlainMLP
from .routed import RoutedExperts
from .recurrent import (GatedDeltaRule, GatedLinearAttention, MatrixLSTM, SelectiveStateMixer, SideBySide,
                        StateSpaceMixer)
from .streams import StreamLink
from .block import ParallelBlock, PostNormBlock, PreNormBlock, SandwichBlock, StreamReentry, StreamsBlock
from .embedding import OutputHead, TokenEmbedding
from .model import DecoderModel, LayerCall, ModelSpec, build_model_spec
