"""Chunk-local GQA softmax attention with rotary positions, unit-norm queries
and keys, values mixed with an earlier layer's and one output gate per head.

Per head, queries and keys are rotated in the half-split layout on their first
``rot["dims"]`` channels and then divided by their root mean square over the
head (no weight). Query ``i`` sees key ``j <= i`` only when ``floor(i / chunk)
== floor(j / chunk)``, blocks counted from position 0 wherever a prompt was cut
(``chunk`` 0: plain causal). A module built with ``mixes_values`` blends its
values with ``v_first``, the values another layer projected for the same
tokens, ``v <- (1 - lambda) v + lambda v_first`` in fp32 with one learned lambda
per layer; the blend is what its cache holds. Each head's output is multiplied
by the sigmoid of one gate number. Every one of these is a constructor
parameter and can be switched off; key and value heads may differ in size.

The module owns lambda, the frequency table and the cache access; the q/k/v/gate
projections are the caller's (so they can be one fused GEMM). Rotation, norms,
the blend and both page scatters are one launch; then one kernel serves prompt
portions, single decoded tokens and mixed batches: every query carries its own
position.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from neuronx_distributed_inference_amd.modules.rope import half_split_inv_freq
from neuronx_distributed_inference_amd.ops import seqmix


class ChunkedRotaryAttention(nn.Module):
    def __init__(self, num_heads: int, num_kv_heads: int, qk_dim: int, v_dim: int,
                 scale: float, eps: float, chunk: int = 0, rot: Optional[dict] = None,
                 unit_norm: bool = True, mixes_values: bool = False):
        super().__init__()
        assert num_heads % num_kv_heads == 0 and chunk >= 0
        self.num_heads = num_heads
        self.num_kv_heads = num_kv_heads
        self.qk_dim = qk_dim
        self.v_dim = v_dim
        self.scale = float(scale)
        self.eps = float(eps)
        self.chunk = int(chunk)
        self.unit_norm = bool(unit_norm)
        if rot:
            dims = int(rot.get("dims", qk_dim))
            assert dims % 2 == 0 and dims <= qk_dim
            self.register_buffer("inv_freq", half_split_inv_freq(rot["base"], dims)[0],
                                 persistent=False)
        else:
            self.inv_freq = None
        self.v_lambda = nn.Parameter(torch.zeros(1, dtype=torch.float32),
                                     requires_grad=False) if mixes_values else None

    def kv_shape(self):
        """(kv_heads, key size, value size) of the pages this layer owns."""
        return (self.num_kv_heads, self.qk_dim, self.v_dim)

    def forward(self, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, kv_mgr,
                cache_idx: int, step: seqmix.StepLayout, gate: Optional[torch.Tensor] = None,
                v_first: Optional[torch.Tensor] = None) -> torch.Tensor:
        """q (B,S,H*Dk), k (B,S,G*Dk), v and v_first (B,S,G*Dv), gate (B,S,H) —
        column slices of a fused projection are fine. Returns (B,S,H*Dv)."""
        kc, vc = kv_mgr.get_cache(cache_idx)
        mixes = self.v_lambda is not None
        assert mixes == (v_first is not None)
        q = seqmix.attention_rows(q, k, v, step, self.inv_freq, self.unit_norm, self.eps, kc.data,
                                  vc.data, kv_mgr.slot_mapping, v_first, self.v_lambda)
        return seqmix.paged_attention(
            q, kc.data, vc.data, step, kv_mgr.block_table, self.scale, self.num_heads,
            chunk=self.chunk, gate=gate, gate_per_head=True, out_dtype=q.dtype)
