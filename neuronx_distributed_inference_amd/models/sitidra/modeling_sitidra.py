"""Sitidra for MI355X: a pre-norm decoder whose residual is several parallel
streams, mixing chunk-local attention with a matrix-memory recurrence, every
feed-forward a mixture of experts.

A sublayer reads a weighted sum of the streams through a layer norm (weight,
no bias) and writes back through learned static mixing
(:class:`HyperConnection`); the output is the sum of the streams. Mixers,
chosen per layer by ``type``:

- ``attention``: :class:`ChunkedRotaryAttention` — GQA, half-split rotary
  positions, queries and keys divided by their root mean square, keys visible
  only inside the query's block of ``mask.size`` positions, one sigmoid gate
  per head; in layers with ``v_mix`` but the first such layer the values are
  blended with that first layer's values of the same token;
- ``mlstm``: :class:`ExponentialGateMemory` — matrix memory with exponential
  gates, a normalizer and a running maximum.

Feed-forward (or none): silu-gated experts behind a sigmoid router (choice by
corrected scores, groups ranked by the sum of their two best, weights
renormalised) and a shared expert with weight one. Output: the model's layer
norm, an untied head, a tanh cap on the logits.

Engine integration (shared with the other hybrid decoders through
:class:`HybridDecoderModel`): fp32 streams, paged KV for attention layers,
recurrent state in the cache manager's state slots, one set of kernels for
prompt portions, decoded tokens and mixed batches. Every projection that reads
a mixer's input is one fused GEMM, all experts are two; a sublayer's write, the
next one's read and its norm are one kernel.
"""

from __future__ import annotations

import json
import os
from typing import Dict, List

import torch
import torch.nn as nn

from neuronx_distributed_inference_amd.config import InferenceConfig
from neuronx_distributed_inference_amd.models.hybrid_base import HybridDecoderModel
from neuronx_distributed_inference_amd.models.model_base import CausalLMBase
from neuronx_distributed_inference_amd.modules.attention.chunked_rotary_attention import (
    ChunkedRotaryAttention,
)
from neuronx_distributed_inference_amd.modules.hyper_connection import HyperConnection
from neuronx_distributed_inference_amd.modules.linear_recurrence import ExponentialGateMemory
from neuronx_distributed_inference_amd.modules.moe import (
    FusedGatedExperts,
    GroupRoutedFeedForward,
)
from neuronx_distributed_inference_amd.modules.norm import StreamLayerNorm
from neuronx_distributed_inference_amd.ops import seqmix
from neuronx_distributed_inference_amd.parallel.layers import (
    ColumnParallelLinear,
    RowParallelLinear,
)

MIXER_TYPES = ("attention", "mlstm")
ROUTER_NORM_EPS = 1e-20    # fixed by the design: added to the chosen scores' sum
GROUP_TOP = 2              # fixed by the design: a group scores as its two best experts


class SitidraInferenceConfig(InferenceConfig):
    """Reads the checkpoint's ``config.json`` as is (keys: architecture,
    width, vocab, streams, layers[], norm.eps, logit_softcap) and derives the
    generic attribute names the engine uses."""

    def get_required_attributes(self) -> List[str]:
        return ["width", "vocab", "streams", "layers", "norm"]

    def add_derived_config(self):
        if not hasattr(self, "layers"):
            return
        if not hasattr(self, "logit_softcap"):
            self.logit_softcap = None
        self.hidden_size = self.width
        self.vocab_size = self.vocab
        self.num_hidden_layers = len(self.layers)
        self.tie_word_embeddings = False
        if self.streams < 1:
            raise ValueError("at least one residual stream is needed")
        first = None
        for i, lc in enumerate(self.layers):
            if lc.get("type") not in MIXER_TYPES:
                raise ValueError(f"unknown Sitidra layer type {lc.get('type')!r}")
            mc, fc = lc["mixer"], lc.get("mlp")
            if lc["type"] == "attention":
                if mc["heads"] % mc["kv_heads"]:
                    raise ValueError(f"layer {i}: heads must be a multiple of kv_heads")
                if mc.get("v_mix"):
                    size = mc["kv_heads"] * mc["vdim"]
                    first = size if first is None else first
                    if size != first:
                        raise ValueError(f"layer {i}: values of another size than the first "
                                         "value-mixing layer's")
            if fc:
                if fc.get("kind") != "moe":
                    raise ValueError(f"unknown Sitidra feed-forward kind {fc.get('kind')!r}")
                rc = fc["router"]
                groups = rc.get("groups") or {"count": 1, "keep": 1}
                count, keep = groups["count"], groups["keep"]
                if count < 1 or rc["experts"] % count or not 1 <= keep <= count:
                    raise ValueError(f"layer {i}: bad expert groups {groups!r}")
                if not 1 <= rc["top"] <= rc["experts"] // count * keep:
                    raise ValueError(f"layer {i}: top exceeds the experts of the kept groups")
        ec = self.neuron_config
        if ec.tp_degree != 1:
            raise ValueError("Sitidra runs with tp_degree=1")
        ec.is_block_kv_layout = True

    def values_of(self, i: int) -> str:
        """What attention layer i does with its values: "own" (no blend),
        "first" (later layers blend them in) or "mixed"."""
        def mixes(lc):
            return lc["type"] == "attention" and bool(lc["mixer"].get("v_mix"))

        if not mixes(self.layers[i]):
            return "own"
        return "mixed" if any(mixes(lc) for lc in self.layers[:i]) else "first"

    @classmethod
    def from_hf_config(cls, model_path: str, neuron_config=None, **overrides):
        """Sizes that config.json leaves out are taken from the tensors'
        shapes in the checkpoint header, where a shape determines them."""
        with open(os.path.join(model_path, "config.json")) as f:
            hf = json.load(f)
        hf.update(overrides)
        ckpt = os.path.join(model_path, "model.safetensors")
        if os.path.exists(ckpt):
            from safetensors import safe_open

            with safe_open(ckpt, framework="pt") as st:
                names = set(st.keys())

                def shape(name):
                    return st.get_slice(name).get_shape() if name in names else None

                emb = shape("embed")
                if emb:
                    hf.setdefault("vocab", emb[0])
                    hf.setdefault("width", emb[1])
                if shape("l0.hc1.in"):
                    hf.setdefault("streams", shape("l0.hc1.in")[0])
                for i, lc in enumerate(hf["layers"]):
                    _fill_from_shapes(lc, lambda n, i=i: shape(f"l{i}.{n}"))
        return cls(neuron_config=neuron_config, **hf)


def _fill_from_shapes(lc: dict, shape):
    mc = lc.setdefault("mixer", {})
    heads = shape("mix.g") if lc["type"] == "attention" else shape("mix.i")
    if "heads" not in mc and heads:
        mc["heads"] = heads[0]
    if "dim" not in mc and "heads" in mc and shape("mix.q"):
        mc["dim"] = shape("mix.q")[0] // mc["heads"]
    if lc["type"] == "attention":
        if "kv_heads" not in mc and "dim" in mc and shape("mix.k"):
            mc["kv_heads"] = shape("mix.k")[0] // mc["dim"]
        if "vdim" not in mc and "kv_heads" in mc and shape("mix.v"):
            mc["vdim"] = shape("mix.v")[0] // mc["kv_heads"]
    elif "vdim" not in mc and "heads" in mc and shape("mix.v"):
        mc["vdim"] = shape("mix.v")[0] // mc["heads"]
    fc = lc.get("mlp")
    if not isinstance(fc, dict):
        return
    rc, xc = fc.setdefault("router", {}), fc.setdefault("expert", {})
    if "experts" not in rc and shape("mlp.router"):
        rc["experts"] = shape("mlp.router")[0]
    if "ff" not in xc and shape("mlp.e0.up"):
        xc["ff"] = shape("mlp.e0.up")[0]
    sc = fc.get("shared")
    if isinstance(sc, dict) and "ff" not in sc and shape("mlp.shared.up"):
        sc["ff"] = shape("mlp.shared.up")[0]


# ----------------------------------------------------------------- mixers
def _padded(splits: List[int]) -> List[int]:
    """Column widths of a fused projection, completed to a multiple of 8 (rows
    of its output then start on 16-byte boundaries in either dtype)."""
    pad = -sum(splits) % 8
    return splits + [pad] if pad else splits


def _stack(parts: List[torch.Tensor]) -> torch.Tensor:
    """Fused projection weight with the zero rows of :func:`_padded`."""
    pad = -sum(p.shape[0] for p in parts) % 8
    return torch.cat(parts + [parts[0].new_zeros(pad, parts[0].shape[1])], dim=0)


class SitidraAttentionMixer(nn.Module):
    def __init__(self, width: int, mc: dict, eps: float, dtype: torch.dtype, values: str):
        """``values``: as :meth:`SitidraInferenceConfig.values_of`."""
        super().__init__()
        H, G, D, Dv = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
        self.values = values
        self.core = ChunkedRotaryAttention(
            H, G, D, Dv, mc["scale"], eps, chunk=(mc.get("mask") or {}).get("size", 0),
            rot=mc.get("rot"), unit_norm=True, mixes_values=values == "mixed")
        # one GEMM for everything that reads the mixer's input
        self.splits = _padded([H * D, G * D, G * Dv, H])
        self.in_proj = ColumnParallelLinear(width, sum(self.splits), dtype=dtype, tp_degree=1)
        self.o_proj = RowParallelLinear(H * Dv, width, dtype=dtype, tp_degree=1)

    def kv_shape(self):
        return self.core.kv_shape()

    def state_shapes(self):
        return {}

    def forward(self, h, kv_mgr, run_idx: int, step):
        q, k, v, g = torch.split(self.in_proj(h), self.splits, dim=-1)[:4]
        if self.values == "first":
            step.first_values = v
        return self.o_proj(self.core(
            q, k, v, kv_mgr, run_idx, step, gate=g,
            v_first=step.first_values if self.values == "mixed" else None))

    @staticmethod
    def convert(s, d, w, f, out, values):
        out[d + "in_proj.weight"] = _stack([w(s + "q"), w(s + "k"), w(s + "v"), w(s + "g")])
        if values == "mixed":
            out[d + "core.v_lambda"] = f(s + "vmix").reshape(1)
        out[d + "o_proj.weight"] = w(s + "o")


class SitidraMemoryMixer(nn.Module):
    def __init__(self, width: int, mc: dict, eps: float, dtype: torch.dtype):
        super().__init__()
        H, D, Dv = mc["heads"], mc["dim"], mc["vdim"]
        self.core = ExponentialGateMemory(H, D, Dv, mc["gate_cap"], eps)
        # one GEMM for everything that reads the mixer's input: q, k, v, the
        # output gate, the input and the forget gates
        self.splits = _padded([H * D, H * D, H * Dv, H * Dv, H, H])
        self.in_proj = ColumnParallelLinear(width, sum(self.splits), dtype=dtype, tp_degree=1)
        self.o_proj = RowParallelLinear(H * Dv, width, dtype=dtype, tp_degree=1)

    def kv_shape(self):
        return None

    def state_shapes(self):
        return self.core.state_shapes()

    def forward(self, h, kv_mgr, run_idx: int, step):
        q, k, v, g, i, f = torch.split(self.in_proj(h), self.splits, dim=-1)[:6]
        return self.o_proj(self.core(q, k, v, g, i, f, kv_mgr.state, f"run{run_idx}", step))

    @staticmethod
    def convert(s, d, w, f, out):
        out[d + "in_proj.weight"] = _stack([w(s + n) for n in ("q", "k", "v", "g", "i", "f")])
        out[d + "core.i_bias"] = f(s + "i.b")
        out[d + "core.f_bias"] = f(s + "f.b")
        out[d + "core.norm_weight"] = f(s + "norm")
        out[d + "o_proj.weight"] = w(s + "o")


class SitidraLayer(nn.Module):
    def __init__(self, config: SitidraInferenceConfig, layer_idx: int):
        super().__init__()
        lc = config.layers[layer_idx]
        eps = float(config.norm["eps"])
        W, dt = config.width, config.neuron_config.torch_dtype
        self.dtype = dt
        self.eps = eps
        self.hc1 = HyperConnection(config.streams)
        self.norm1 = StreamLayerNorm(W, eps=eps, out_dtype=dt, bias=False)
        if lc["type"] == "attention":
            self.mixer = SitidraAttentionMixer(W, lc["mixer"], eps, dt,
                                               config.values_of(layer_idx))
        else:
            self.mixer = SitidraMemoryMixer(W, lc["mixer"], eps, dt)
        self.mlp = None
        fc = lc.get("mlp")
        if fc:
            rc = fc["router"]
            groups = rc.get("groups") or {"count": 1, "keep": 1}
            self.hc2 = HyperConnection(config.streams)
            self.norm2 = StreamLayerNorm(W, eps=eps, out_dtype=dt, bias=False)
            self.mlp = GroupRoutedFeedForward(
                W, rc["experts"], rc["top"], fc["expert"]["ff"], dt, n_groups=groups["count"],
                keep_groups=groups["keep"], scale=rc.get("scale", 1.0), normalize=True,
                shared_ff=(fc.get("shared") or {}).get("ff", 0), shared_gate=False,
                act="silu_glu", router=dict(correction=True, score="sigmoid",
                                            group_top=GROUP_TOP, norm_eps=ROUTER_NORM_EPS))

    def kv_shape(self):
        return self.mixer.kv_shape()

    def state_shapes(self) -> Dict[str, tuple]:
        return self.mixer.state_shapes()

    def entry(self):
        """What the kernel before this layer needs to make its normed input."""
        return self.hc1.w_in, self.norm1.weight

    def forward(self, x, kv_mgr, run_idx: int):
        step = kv_mgr.step
        # this layer's normed input: left by the previous layer's last write, or
        # made here for the first layer (whose streams are one row still)
        h, step.prenorm = step.prenorm, None
        if h is None:
            h = self.hc1.read(x, self.norm1, self.dtype)
        y = self.mixer(h, kv_mgr, run_idx, step)
        if self.mlp is not None:
            x, h = self.hc1.write(x, y, (self.hc2.w_in, self.norm2.weight), self.eps, self.dtype)
            last, y = self.hc2, self.mlp(h)
        else:
            last = self.hc1
        x, h = last.write(x, y, step.following, self.eps, self.dtype)
        if step.following is None:
            return h                       # the model's end: the sum of the streams
        step.prenorm = h
        return x


class SitidraModel(HybridDecoderModel):
    def build_layers(self, config) -> nn.ModuleList:
        return nn.ModuleList(SitidraLayer(config, i) for i in range(len(config.layers)))

    def build_norm(self, config) -> nn.Module:
        return StreamLayerNorm(config.width, eps=config.norm["eps"],
                               out_dtype=config.neuron_config.torch_dtype, bias=False)

    def begin_step(self, position_ids, seq_ids, block_table):
        block_table = super().begin_step(position_ids, seq_ids, block_table)
        step = self.kv_mgr.step
        step.prenorm = step.following = step.first_values = None
        return block_table

    def before_layer_run(self, run_idx, h, h_embed):
        nxt = run_idx + 1
        self.kv_mgr.step.following = self.layers[nxt].entry() if nxt < len(self.layers) else None
        return h                           # the embedding row is never written

    def finalize_logits(self, logits):
        cap = self.config.logit_softcap
        return seqmix.softcap(logits, float(cap)) if cap else logits.float()


class SitidraForCausalLM(CausalLMBase):
    _model_cls = SitidraModel
    _config_cls = SitidraInferenceConfig

    @staticmethod
    def convert_hf_to_native_state_dict(sd: Dict[str, torch.Tensor], config) -> Dict[str, torch.Tensor]:
        dt = config.neuron_config.torch_dtype
        out: Dict[str, torch.Tensor] = {}

        def w(name):                       # projection weights: engine dtype
            return sd[name].to(dt)

        def f(name):                       # 32-bit parameters
            return sd[name].float()

        out["embed_tokens.weight"] = w("embed")
        out["lm_head.weight"] = w("head")
        out["norm.weight"] = f("final.norm")
        for i, lc in enumerate(config.layers):
            s, d = f"l{i}.", f"layers.{i}."
            for q in (1, 2) if lc.get("mlp") else (1,):
                out[d + f"norm{q}.weight"] = f(s + f"norm{q}")
                for n in ("in", "out", "mix"):
                    out[d + f"hc{q}." + ("mix" if n == "mix" else "w_" + n)] = f(s + f"hc{q}.{n}")
            if lc["type"] == "attention":
                SitidraAttentionMixer.convert(s + "mix.", d + "mixer.", w, f, out,
                                              config.values_of(i))
            else:
                SitidraMemoryMixer.convert(s + "mix.", d + "mixer.", w, f, out)
            fc = lc.get("mlp")
            if not fc:
                continue
            m = s + "mlp."
            E = fc["router"]["experts"]
            shared = bool(fc.get("shared"))
            out[d + "mlp.router.weight"] = f(m + "router")
            out[d + "mlp.router.correction"] = f(m + "correction")
            out[d + "mlp.experts.gate_up.weight"] = FusedGatedExperts.stack_gate_up(
                [w(m + f"e{e}.gate") for e in range(E)], [w(m + f"e{e}.up") for e in range(E)],
                w(m + "shared.gate") if shared else None, w(m + "shared.up") if shared else None)
            out[d + "mlp.experts.down.weight"] = FusedGatedExperts.stack_down(
                [w(m + f"e{e}.down") for e in range(E)], w(m + "shared.down") if shared else None)
        return out
