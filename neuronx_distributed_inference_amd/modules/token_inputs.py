"""Inputs that a decoder takes from token ids besides the plain embedding.

:class:`BigramEmbedding` adds a hashed row for the (previous, current) token
pair; the previous token of a step's first column is per-sequence state, so
prompts can be cut anywhere. :class:`TokenSideInput` feeds every layer a
slice of a second, narrow embedding of the token, gated by the stream.
"""

from __future__ import annotations

import torch
import torch.nn as nn

from neuronx_distributed_inference_amd.modules.norm import StreamRMSNorm
from neuronx_distributed_inference_amd.ops import seqmix
from neuronx_distributed_inference_amd.parallel.layers import (
    ColumnParallelLinear,
    RowParallelLinear,
)


class BigramEmbedding(nn.Module):
    """Row ``(prev * mul_prev + cur * mul_cur) mod buckets`` of a table with
    ``buckets + 1`` rows; the last row serves a sequence's first token."""

    STATE = "last_token"

    def __init__(self, buckets: int, width: int, mul_prev: int, mul_cur: int, dtype: torch.dtype):
        super().__init__()
        self.mul_prev = int(mul_prev)
        self.mul_cur = int(mul_cur)
        self.weight = nn.Parameter(torch.zeros(buckets + 1, width, dtype=dtype),
                                   requires_grad=False)

    def model_state(self):
        return {self.STATE: ((), torch.int32)}

    def forward(self, ids: torch.Tensor, embed_weight: torch.Tensor, states,
                step: seqmix.StepLayout) -> torch.Tensor:
        """Token rows + bigram rows -> fp32 stream (B,S,width), one launch;
        advances the carried token."""
        return seqmix.bigram_embedding(ids, embed_weight, self.weight, states.get(self.STATE),
                                       step, self.mul_prev, self.mul_cur)


class TokenSideInput(nn.Module):
    """``x += rms_norm(W_proj (gelu_tanh(W_gate x) * e)) * w`` with ``e`` the
    channels [index * dim, (index + 1) * dim) of the token's row in a
    (vocab, layers * dim) table shared by the layers."""

    def __init__(self, width: int, dim: int, index: int, eps: float, dtype: torch.dtype):
        super().__init__()
        self.offset = index * dim
        self.gate = ColumnParallelLinear(width, dim, dtype=dtype, tp_degree=1)
        self.proj = RowParallelLinear(dim, width, dtype=dtype, tp_degree=1)
        self.norm = StreamRMSNorm(width, eps=eps)

    def forward(self, x: torch.Tensor, h: torch.Tensor, table: torch.Tensor,
                step: seqmix.StepLayout, copy_dtype=None):
        """``x`` the fp32 stream (updated in place), ``h`` the same in the GEMM
        input dtype. Returns the new stream in ``copy_dtype`` (None: no copy)."""
        g = seqmix.token_gate_proj(h, self.gate.weight, step.tokens, table, self.offset)
        return self.norm.add_into(x, self.proj(g), copy_dtype)
