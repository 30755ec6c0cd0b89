"""Residual kept as several parallel streams with learned, static mixing.

A token's residual is ``n`` streams of the model's width, all equal to the
embedding at the start. Around a sublayer f with its pre-norm

    u    = sum_s w_in[s] x_s                     (what the sublayer reads)
    y    = f(norm(u))
    x_t <- sum_s mix[s, t] x_s + w_out[t] y      (all t from the old streams)

and the model's output is the sum of the streams. The streams are fp32 and
so are the weights. One kernel does a sublayer's write together with the next
sublayer's read and norm, so the streams are read and written once per
sublayer; the sum after the last one leaves from the same kernel.
"""

from __future__ import annotations

import torch
import torch.nn as nn

from neuronx_distributed_inference_amd.ops import seqmix


class HyperConnection(nn.Module):
    """The weights around one sublayer."""

    def __init__(self, streams: int):
        super().__init__()
        f32 = dict(dtype=torch.float32)
        self.w_in = nn.Parameter(torch.ones(streams, **f32), requires_grad=False)
        self.w_out = nn.Parameter(torch.ones(streams, **f32), requires_grad=False)
        self.mix = nn.Parameter(torch.eye(streams, **f32), requires_grad=False)

    def read(self, streams, norm, out_dtype):
        """norm(sum_s w_in[s] x_s) without a write before it; ``streams`` may
        be the (B,S,C) row that all streams still equal."""
        return seqmix.hyper_step(streams, None, self.mix, self.w_out, self.w_in, norm.weight,
                                 norm.eps, out_dtype)[1]

    def write(self, streams, y, following, eps: float, out_dtype):
        """The streams after this sublayer's result ``y``, and what follows it:
        ``following`` = (w_in, norm weight) of the next sublayer gives that
        sublayer's normed input in ``out_dtype``; None gives the sum of the
        streams in fp32 (the streams themselves are then not written)."""
        w_in, weight = following if following is not None else (None, None)
        return seqmix.hyper_step(streams, y, self.mix, self.w_out, w_in, weight, eps, out_dtype,
                                 keep=following is not None)
