from .attention import Attention
from .base import (Block, CacheNeed, CacheView, CallInfo, FeedForward, Mixer, Norm, Part,
                   NormedRows, NormedSum, PendingRows, PoolSpec, PositionEncoding, ReadyRows, StepContext,
                   SumRows, WeightBinder, plain_rows, settle)
from .block import OutputNormBlock, ParallelBlock, PostNormBlock, PreNormBlock, SandwichBlock
from .diff_attention import DifferentialAttention
from .embedding import LMHead, TokenEmbedding
from .forget_gate import ForgetGateAttention
from .gla import GatedLinearAttention
from .latent_attention import LatentAttention
from .lightning import LightningAttention
from .matrix_memory import MatrixMemory
from .mlp import MLP, SwiGLU
from .moe import RoutedExperts, Routing, SoftmaxTopKRouter, SparseMoE, TopKRouter
from .norm import LayerNorm, OutputLayerNorm, OutputRMSNorm, ResidualRMSNorm, RMSNorm
from .rotary import NoPosition, Rotary
from .reentry import StreamReentry
from .short_conv import ShortConv
from .side_by_side import SideBySide
from .sigmoid_attention import SigmoidAttention
from .state_space import StateSpace
from .token_side import TokenSide, TokenSideTable

__all__ = ["Attention", "Block", "CacheNeed", "CacheView", "CallInfo", "FeedForward", "Mixer",
           "Norm", "Part", "PendingRows", "PoolSpec", "settle", "PositionEncoding", "StepContext", "WeightBinder", "PreNormBlock",
           "LMHead", "TokenEmbedding", "SwiGLU", "RoutedExperts", "Routing", "SoftmaxTopKRouter", "TopKRouter",
           "SparseMoE", "RMSNorm", "NoPosition", "Rotary", "OutputNormBlock", "OutputRMSNorm",
           "LatentAttention", "LightningAttention", "ShortConv", "ParallelBlock",
           "DifferentialAttention", "MLP", "StreamReentry", "GatedLinearAttention",
           "SigmoidAttention", "SandwichBlock", "LayerNorm", "OutputLayerNorm", "NormedSum",
           "ReadyRows", "plain_rows", "PostNormBlock", "ForgetGateAttention", "ResidualRMSNorm",
           "SideBySide", "SumRows", "NormedRows", "MatrixMemory", "StateSpace", "TokenSide", "TokenSideTable"]
