"""Risutar for MI355X: a decoder that norms after each residual sum, mixes
latent attention with gated linear attention, and feeds every layer a slice
of a second token embedding.

Stream: token row + bigram row (hashed previous/current pair). Layer:
``x = norm1(alpha x + mixer(x))``, then, when the layer has a feed-forward,
``x = norm2(alpha x + ff(x))`` (layer norms with bias, ``alpha`` one constant
of the model; the sublayers read the stream itself), then the token side
input ``x += rms_norm(W_proj (gelu_tanh(W_gate x) * e_layer)) * w``. Mixers,
chosen per layer by ``type``:

- ``latent_attention``: :class:`LatentSinkAttention` (no sink, no window) —
  queries through a normed low-rank latent, keys and values expanded per head
  from a normed latent, one half-split rotated key part for all heads, one
  sigmoid gate per head; a layer with ``kv_from`` reads another layer's
  cached rows with its own up-projections;
- ``gla``: :class:`GatedLinearAttention` — matrix state with a data-dependent
  decay per key channel, normed read-out, silu output gate.

Feed-forwards, chosen by ``mlp.kind``: ``dense`` — silu-gated; ``moe`` —
two-matrix experts with the exact gelu behind a biased top-k router (softmax
over the chosen logits), and a shared expert with weight one. Output: the
model's layer norm, then an untied head.

Engine integration (shared with the other hybrid decoders through
:class:`HybridDecoderModel`): fp32 residual stream, paged latent rows (none
for borrowing and recurrent layers), recurrent state and each sequence's
newest token in the cache manager's state slots, one set of kernels for
prompt portions, decoded tokens and mixed batches. Every projection that
reads a mixer's input is one fused GEMM; each residual step is one kernel
that also emits the stream in the next GEMM's input dtype.
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
from neuronx_distributed_inference_amd.modules.attention.latent_attention import (
    LatentSinkAttention,
)
from neuronx_distributed_inference_amd.modules.linear_recurrence import GatedLinearAttention
from neuronx_distributed_inference_amd.modules.mlp import GatedMLP
from neuronx_distributed_inference_amd.modules.moe import (
    FusedUngatedExperts,
    GroupRoutedFeedForward,
)
from neuronx_distributed_inference_amd.modules.norm import StreamLayerNorm, StreamRMSNorm
from neuronx_distributed_inference_amd.modules.token_inputs import (
    BigramEmbedding,
    TokenSideInput,
)
from neuronx_distributed_inference_amd.parallel.layers import (
    ColumnParallelLinear,
    RowParallelLinear,
)

MIXER_TYPES = ("latent_attention", "gla")
FF_KINDS = ("dense", "moe")


class RisutarInferenceConfig(InferenceConfig):
    """Reads the checkpoint's ``config.json`` as is (keys: architecture,
    width, vocab, embedding.bigram, layers[], norm.eps, postln_alpha,
    token_side.dim) and derives the generic attribute names the engine uses."""

    def get_required_attributes(self) -> List[str]:
        return ["width", "vocab", "layers", "norm", "postln_alpha"]

    def add_derived_config(self):
        if not hasattr(self, "layers"):
            return
        self.embedding = getattr(self, "embedding", None) or {}
        self.token_side = getattr(self, "token_side", None)
        self.hidden_size = self.width
        self.vocab_size = self.vocab
        self.num_hidden_layers = len(self.layers)
        self.tie_word_embeddings = False
        for i, lc in enumerate(self.layers):
            if lc.get("type") not in MIXER_TYPES:
                raise ValueError(f"unknown Risutar layer type {lc.get('type')!r}")
            mc, fc = lc["mixer"], lc.get("mlp")
            if fc and fc.get("kind") not in FF_KINDS:
                raise ValueError(f"unknown Risutar feed-forward kind {fc.get('kind')!r}")
            if fc and fc["kind"] == "moe" and \
                    not 1 <= fc["router"]["top"] <= fc["router"]["experts"]:
                raise ValueError(f"layer {i}: top exceeds the number of experts")
            src = mc.get("kv_from")
            if src is not None:
                if not 0 <= src < i or lc["type"] != "latent_attention" or \
                        self.layers[src]["type"] != "latent_attention" or \
                        self.layers[src]["mixer"].get("kv_from") is not None:
                    raise ValueError(f"layer {i}: kv_from must name an earlier latent "
                                     "attention layer that stores its own rows")
                for key in ("kv_rank", "rot_dim", "rot"):
                    if self.layers[src]["mixer"][key] != mc[key]:
                        raise ValueError(f"layer {i}: {key} differs from the lender's")
            if lc["type"] == "gla" and "decay_rank" not in mc:
                raise ValueError(f"layer {i}: decay_rank (rows of mix.a1) is not known")
        ec = self.neuron_config
        if ec.tp_degree != 1:
            raise ValueError("Risutar runs with tp_degree=1")
        ec.is_block_kv_layout = True

    @classmethod
    def from_hf_config(cls, model_path: str, neuron_config=None, **overrides):
        """Sizes that config.json leaves out (the rank of the decay
        projection always) are taken from the tensors' shapes in the
        checkpoint header, where a shape determines them."""
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
                bg = (hf.get("embedding") or {}).get("bigram")
                if bg and "buckets" not in bg and shape("bigram"):
                    bg["buckets"] = shape("bigram")[0] - 1
                side = hf.get("token_side")
                if isinstance(side, dict) and "dim" not in side and shape("side.embed"):
                    side["dim"] = shape("side.embed")[1] // len(hf["layers"])
                for i, lc in enumerate(hf["layers"]):
                    _fill_from_shapes(lc, lambda n, i=i: shape(f"l{i}.{n}"))
                for lc in hf["layers"]:
                    mc = lc["mixer"]
                    if mc.get("kv_from") is not None:     # the lender's, where left out
                        for key in ("kv_rank", "rot_dim", "rot"):
                            if key not in mc and key in hf["layers"][mc["kv_from"]]["mixer"]:
                                mc[key] = hf["layers"][mc["kv_from"]]["mixer"][key]
        return cls(neuron_config=neuron_config, **hf)


def _fill_from_shapes(lc: dict, shape):
    mc = lc.setdefault("mixer", {})
    if lc["type"] == "gla":
        if shape("mix.a1"):
            mc["decay_rank"] = shape("mix.a1")[0]
        if "vdim" not in mc and shape("mix.norm"):
            mc["vdim"] = shape("mix.norm")[0]
        if "heads" not in mc and "vdim" in mc and shape("mix.v"):
            mc["heads"] = shape("mix.v")[0] // mc["vdim"]
        if "dim" not in mc and "heads" in mc and shape("mix.q"):
            mc["dim"] = shape("mix.q")[0] // mc["heads"]
    elif lc["type"] == "latent_attention":
        if "q_rank" not in mc and shape("mix.dq"):
            mc["q_rank"] = shape("mix.dq")[0]
        if "kv_rank" not in mc and shape("mix.uk"):
            mc["kv_rank"] = shape("mix.uk")[1]
        if "heads" not in mc and shape("mix.g"):
            mc["heads"] = shape("mix.g")[0]
        if "dim" not in mc and "heads" in mc and shape("mix.uk"):
            mc["dim"] = shape("mix.uk")[0] // mc["heads"]
        if "vdim" not in mc and "heads" in mc and shape("mix.uv"):
            mc["vdim"] = shape("mix.uv")[0] // mc["heads"]
        if "rot_dim" not in mc and "heads" in mc and "dim" in mc and shape("mix.uq"):
            mc["rot_dim"] = shape("mix.uq")[0] // mc["heads"] - mc["dim"]
    fc = lc.get("mlp")
    if not isinstance(fc, dict):
        return
    if fc.get("kind") == "dense":
        if "ff" not in fc and shape("mlp.up"):
            fc["ff"] = shape("mlp.up")[0]
    elif fc.get("kind") == "moe":
        rc = fc.setdefault("router", {})
        if "experts" not in rc and shape("mlp.router"):
            rc["experts"] = shape("mlp.router")[0]
        xc = fc.setdefault("expert", {})
        if "ff" not in xc and shape("mlp.e0.up"):
            xc["ff"] = shape("mlp.e0.up")[0]
        if isinstance(fc.get("shared"), dict) and "ff" not in fc["shared"] and \
                shape("mlp.shared.up"):
            fc["shared"]["ff"] = shape("mlp.shared.up")[0]


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


class RisutarLatentMixer(nn.Module):
    def __init__(self, width: int, mc: dict, eps: float, dtype: torch.dtype):
        super().__init__()
        H, D, R, Dv, C = mc["heads"], mc["dim"], mc["rot_dim"], mc["vdim"], mc["kv_rank"]
        Q = mc["q_rank"]
        rot = mc["rot"]
        self.source = mc.get("kv_from")
        self.core = LatentSinkAttention(
            H, D, R, Dv, C, mc["scale"], eps, rot["base"], rot.get("dims", R), dtype, sink=False,
            half_split=True, gate_per_head=True, owns_kv=self.source is None)
        # one GEMM for everything that reads the mixer's input: the query
        # latent, the head gates and (unless the rows are another layer's) the
        # key/value latent with the rotated key part
        self.splits = _padded([Q] + ([C + R] if self.source is None else []) + [H])
        self.in_proj = ColumnParallelLinear(width, sum(self.splits), dtype=dtype, tp_degree=1)
        self.q_norm = StreamRMSNorm(Q, eps=eps, out_dtype=dtype)
        self.q_up = ColumnParallelLinear(Q, H * (D + R), dtype=dtype, tp_degree=1)
        self.o_proj = RowParallelLinear(H * Dv, width, dtype=dtype, tp_degree=1)

    def kv_shape(self):
        return self.core.kv_shape()

    def state_shapes(self):
        return {}

    def forward(self, h, kv_mgr, run_idx: int, step):
        parts = torch.split(self.in_proj(h), self.splits, dim=-1)
        dkv, gate = (parts[1], parts[2]) if self.source is None else (None, parts[1])
        q = self.q_up(self.q_norm(parts[0]))
        return self.o_proj(self.core(q, dkv, kv_mgr, run_idx, step, gate=gate))

    @staticmethod
    def convert(sd, s, d, w, f, out, mc):
        own = mc.get("kv_from") is None
        out[d + "in_proj.weight"] = _stack(
            [w(s + "dq")] + ([w(s + "dkv")] if own else []) + [w(s + "g")])
        out[d + "q_norm.weight"] = f(s + "dq.norm")
        out[d + "q_up.weight"] = w(s + "uq")
        if own:
            out[d + "core.latent_norm.weight"] = f(s + "dkv.norm")
        uk, uv = w(s + "uk"), w(s + "uv")
        H, C = mc["heads"], uk.shape[1]
        out[d + "core.uk"] = uk.view(H, -1, C).contiguous()                   # (H, dim, C)
        out[d + "core.uv"] = uv.view(H, -1, C).contiguous()                   # (H, vdim, C)
        out[d + "o_proj.weight"] = w(s + "o")


class RisutarLinearMixer(nn.Module):
    source = None

    def __init__(self, width: int, mc: dict, eps: float, dtype: torch.dtype):
        super().__init__()
        H, D, Dv, r = mc["heads"], mc["dim"], mc["vdim"], mc["decay_rank"]
        self.core = GatedLinearAttention(H, D, Dv, mc["tau"], r, eps, dtype)
        # one GEMM for everything that reads the mixer's input: q, k, v, the
        # output gate, the first stage of the decay projection
        self.splits = _padded([H * D, H * D, H * Dv, H * Dv, r])
        self.in_proj = ColumnParallelLinear(width, sum(self.splits), dtype=dtype, tp_degree=1)
        self.o_proj = RowParallelLinear(H * Dv, width, dtype=dtype, tp_degree=1)

    def kv_shape(self):
        return None

    def state_shapes(self):
        return self.core.state_shapes()

    def forward(self, h, kv_mgr, run_idx: int, step):
        q, k, v, g, a = torch.split(self.in_proj(h), self.splits, dim=-1)[:5]
        return self.o_proj(self.core(q, k, v, g, a, kv_mgr.state, f"run{run_idx}", step))

    @staticmethod
    def convert(sd, s, d, w, f, out, mc):
        out[d + "in_proj.weight"] = _stack(
            [w(s + "q"), w(s + "k"), w(s + "v"), w(s + "g"), w(s + "a1")])
        out[d + "core.decay_up.weight"] = w(s + "a2")
        out[d + "core.decay_bias"] = f(s + "a2.b")
        out[d + "core.norm_weight"] = f(s + "norm")
        out[d + "o_proj.weight"] = w(s + "o")


_MIXERS = {"latent_attention": RisutarLatentMixer, "gla": RisutarLinearMixer}


class RisutarLayer(nn.Module):
    def __init__(self, config: RisutarInferenceConfig, layer_idx: int):
        super().__init__()
        lc = config.layers[layer_idx]
        eps = float(config.norm["eps"])
        W, dt = config.width, config.neuron_config.torch_dtype
        self.dtype = dt
        self.alpha = float(config.postln_alpha)
        self.last = layer_idx == len(config.layers) - 1
        self.mixer = _MIXERS[lc["type"]](W, lc["mixer"], eps, dt)
        self.norm1 = StreamLayerNorm(W, eps=eps)
        self.mlp = None
        fc = lc.get("mlp")
        if fc:
            self.norm2 = StreamLayerNorm(W, eps=eps)
            if fc["kind"] == "dense":
                self.mlp = GatedMLP(W, fc["ff"], tp_degree=1, dtype=dt,
                                    hidden_act="stream_silu", fused_gate_up=True)
            else:
                rc = fc["router"]
                self.mlp = GroupRoutedFeedForward(
                    W, rc["experts"], rc["top"], fc["expert"]["ff"], dt, normalize=True,
                    shared_ff=(fc.get("shared") or {}).get("ff", 0), shared_gate=False,
                    act="gelu", router_bias=True)
        self.side = None
        if config.token_side:
            self.side = TokenSideInput(W, config.token_side["dim"], layer_idx, eps, dt)

    def kv_shape(self):
        return self.mixer.kv_shape()

    def kv_source(self):
        return self.mixer.source

    def state_shapes(self) -> Dict[str, tuple]:
        return self.mixer.state_shapes()

    def forward(self, x, kv_mgr, run_idx: int):
        step = kv_mgr.step
        # the stream in the GEMM input dtype: left by the previous residual
        # kernel, or cast here for the first layer
        h = step.stream_copy if step.stream_copy is not None else x.to(self.dtype)
        h = self.norm1.sum_into(x, self.mixer(h, kv_mgr, run_idx, step), self.alpha, self.dtype)
        if self.mlp is not None:
            h = self.norm2.sum_into(x, self.mlp(h), self.alpha, self.dtype)
        if self.side is not None:
            h = self.side(x, h, step.side_table, step, None if self.last else self.dtype)
        step.stream_copy = h
        return x


class RisutarModel(HybridDecoderModel):
    def __init__(self, config):
        super().__init__(config)
        dt = config.neuron_config.torch_dtype
        self.side_embed = None
        if config.token_side:
            self.side_embed = nn.Parameter(
                torch.zeros(config.vocab, len(config.layers) * config.token_side["dim"], dtype=dt),
                requires_grad=False)

    def build_layers(self, config) -> nn.ModuleList:
        return nn.ModuleList(RisutarLayer(config, i) for i in range(len(config.layers)))

    def build_norm(self, config) -> nn.Module:
        return StreamLayerNorm(config.width, eps=config.norm["eps"],
                               out_dtype=config.neuron_config.torch_dtype)

    def build_kv_manager(self, config) -> nn.Module:
        bg = config.embedding.get("bigram")
        self.bigram = None
        if bg:
            self.bigram = BigramEmbedding(bg["buckets"], config.width, bg["mul_prev"],
                                          bg["mul_cur"], config.neuron_config.torch_dtype)
        return super().build_kv_manager(config)

    def model_state(self):
        return self.bigram.model_state() if self.bigram is not None else {}

    def embed(self, input_ids):
        ids = input_ids.long().contiguous()
        step = self.kv_mgr.step
        step.tokens = ids
        step.side_table = self.side_embed
        if self.bigram is None:
            return super().embed(input_ids)
        return self.bigram(ids, self.embed_tokens.weight, self.kv_mgr.state, step)

    def prepare_hidden(self, h):
        return h if h.dtype == torch.float32 and self.bigram is not None else h.float()

    def before_layer_run(self, run_idx, h, h_embed):
        # the bigram kernel's fresh rows are this model's to update in place
        return h if self.bigram is not None else super().before_layer_run(run_idx, h, h_embed)

    def finalize_logits(self, logits):
        return logits.float()


class RisutarForCausalLM(CausalLMBase):
    _model_cls = RisutarModel
    _config_cls = RisutarInferenceConfig

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
        out["norm.bias"] = f("final.norm.b")
        if config.embedding.get("bigram"):
            out["bigram.weight"] = w("bigram")
        if config.token_side:
            out["side_embed"] = w("side.embed")
        for i, lc in enumerate(config.layers):
            s, d = f"l{i}.", f"layers.{i}."
            for n in ("norm1", "norm2") if lc.get("mlp") else ("norm1",):
                out[d + n + ".weight"] = f(s + n)
                out[d + n + ".bias"] = f(s + n + ".b")
            _MIXERS[lc["type"]].convert(sd, s + "mix.", d + "mixer.", w, f, out, lc["mixer"])
            if config.token_side:
                out[d + "side.gate.weight"] = w(s + "side.gate")
                out[d + "side.proj.weight"] = w(s + "side.proj")
                out[d + "side.norm.weight"] = f(s + "side.norm")
            fc = lc.get("mlp")
            if not fc:
                continue
            m = s + "mlp."
            if fc["kind"] == "dense":
                out[d + "mlp.gate_up_proj.weight"] = torch.cat([w(m + "gate"), w(m + "up")], dim=0)
                out[d + "mlp.down_proj.weight"] = w(m + "down")
                continue
            E = fc["router"]["experts"]
            shared = bool(fc.get("shared"))
            out[d + "mlp.router.weight"] = f(m + "router")
            out[d + "mlp.router.bias"] = f(m + "router.b")
            out[d + "mlp.experts.up.weight"] = FusedUngatedExperts.stack_up(
                [w(m + f"e{e}.up") for e in range(E)], w(m + "shared.up") if shared else None)
            out[d + "mlp.experts.down.weight"] = FusedUngatedExperts.stack_down(
                [w(m + f"e{e}.down") for e in range(E)], w(m + "shared.down") if shared else None)
        return out
