"""Sequence-mixing ops of hybrid (windowed attention + linear recurrence)
models: dispatch between the gfx950 kernels of ``csrc/seqmix.hip`` and the
torch references in ``ops.ref`` (CPU execution and numerics oracle).

The kernels live in their own small shared library ``_nxdi_seqmix.so`` with
a C ABI, loaded through ctypes: it has no torch headers, so a fresh checkout
compiles it with one ``hipcc`` call in seconds and a model that needs only
these ops never waits for the large extension. Launches go to torch's
current HIP stream. On a GPU tensor the library is required — there is no
silent fallback.
"""

from __future__ import annotations

import ctypes
import os
import subprocess
import threading
from typing import Optional

import torch

from neuronx_distributed_inference_amd.ops import ref

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "_nxdi_seqmix.so")
SRC_PATH = os.path.join(_HERE, "csrc", "seqmix.hip")
HIPCC_FLAGS = [
    "-O3", "-std=c++17", "--offload-arch=gfx950", "-shared", "-fPIC",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
]

_lib = None
_lib_error: Optional[BaseException] = None
_lock = threading.Lock()


def _compile(dst: str) -> str:
    hipcc = os.environ.get("HIPCC") or (
        "/opt/rocm/bin/hipcc" if os.path.exists("/opt/rocm/bin/hipcc") else "hipcc")
    tmp = dst + ".%d.tmp" % os.getpid()
    try:
        subprocess.run([hipcc] + HIPCC_FLAGS + ["-o", tmp, SRC_PATH], check=True,
                       stdout=subprocess.DEVNULL, stderr=subprocess.PIPE)
        os.replace(tmp, dst)
    finally:
        if os.path.exists(tmp):
            os.unlink(tmp)
    return dst


def build(force: bool = False) -> str:
    """Compile the library in-tree (cross-compiles without a GPU). When the
    package directory is read-only the library goes to the user's temp
    directory, named after the source's modification time."""
    global LIB_PATH
    if not force and os.path.exists(LIB_PATH) and \
            os.path.getmtime(LIB_PATH) >= os.path.getmtime(SRC_PATH):
        return LIB_PATH
    try:
        return _compile(LIB_PATH)
    except (OSError, subprocess.CalledProcessError):
        if os.access(os.path.dirname(LIB_PATH), os.W_OK):
            raise                      # a real compile error, not a read-only tree
        import tempfile

        alt = os.path.join(tempfile.gettempdir(), "nxdi_seqmix_%d_%d.so" % (
            os.getuid(), int(os.path.getmtime(SRC_PATH))))
        if force or not os.path.exists(alt):
            _compile(alt)
        LIB_PATH = alt
        return LIB_PATH


def _load():
    global _lib, _lib_error
    if _lib is not None:
        return _lib
    with _lock:
        if _lib is not None:
            return _lib
        try:
            build()
            _lib = ctypes.CDLL(LIB_PATH)
        except BaseException as e:  # noqa: BLE001
            _lib_error = e
            raise RuntimeError(
                "sequence-mixing op called on a GPU tensor but _nxdi_seqmix.so "
                f"could not be built/loaded: {e!r}") from e
    return _lib


def library_available() -> bool:
    try:
        _load()
        return True
    except RuntimeError:
        return False


def _p(t: Optional[torch.Tensor]):
    return ctypes.c_void_p(0 if t is None else t.data_ptr())


def _stream():
    return ctypes.c_void_p(torch.cuda.current_stream().cuda_stream)


def _is_bf16(t: torch.Tensor) -> int:
    if t.dtype == torch.bfloat16:
        return 1
    if t.dtype == torch.float32:
        return 0
    raise TypeError(f"seqmix ops take float32 or bfloat16, got {t.dtype}")


def _check(rc: int, name: str):
    if rc != 0:
        raise RuntimeError(f"{name}: launch failed / unsupported shape (code {rc})")


def _i32(t: torch.Tensor) -> torch.Tensor:
    return t if t.dtype == torch.int32 and t.is_contiguous() else t.to(torch.int32).contiguous()


def _f32(t: torch.Tensor) -> torch.Tensor:
    return t if t.dtype == torch.float32 and t.is_contiguous() else t.float().contiguous()


def _rows_view(t: torch.Tensor):
    """(..., C) tensor whose leading dims collapse to rows with one stride
    (a column slice of a fused GEMM output qualifies): returns row stride."""
    assert t.stride(-1) == 1, "innermost dim must be contiguous"
    if t.dim() == 3:
        return _token_stride(t)
    return t.stride(0)


def _token_stride(t: torch.Tensor) -> int:
    """Stride between consecutive tokens of a (B, S, ...) tensor whose
    tokens are uniformly strided (a size-1 axis has no stride of its own)."""
    B, S = t.shape[0], t.shape[1]
    if S == 1:
        return t.stride(0) if B > 1 else max(t.stride(0), t.stride(1))
    assert B == 1 or t.stride(0) == t.stride(1) * S, "rows must be uniformly strided"
    return t.stride(1)


class StepLayout:
    """Per-step ragged-batch descriptors shared by every layer's kernels:
    int32 positions (B,S), state slots (B,), valid-token counts (B,)."""

    def __init__(self, positions: torch.Tensor, seq_ids: torch.Tensor):
        self.positions = _i32(positions)
        self.seq_ids = _i32(seq_ids)
        self.nvalid = (self.positions >= 0).sum(-1).to(torch.int32)
        self._i32 = {}
        # the residual stream in the GEMM input dtype, handed from one
        # sublayer's residual kernel to the next sublayer (None: not yet made)
        self.stream_copy = None
        # True when every row of the step starts its sequence (a whole prompt)
        self.fresh = False
        # dense rows of latent layers whose cache a later layer reads (whole
        # prompts only), by the owner's cache index
        self.latent_rows = {}
        # the step's token ids and the (vocab, layers * dim) table that layers
        # read them from, for models that use ids past the embedding
        self.tokens = None
        self.side_table = None

    def i32(self, t: torch.Tensor) -> torch.Tensor:
        """int32 copy of a per-step index tensor (block table, slot mapping),
        converted once per step instead of once per layer."""
        key = (t.data_ptr(), tuple(t.shape), t.dtype)
        hit = self._i32.get(key)
        if hit is None:
            hit = self._i32[key] = (t, _i32(t))      # keeps `t` alive: the pointer stays its
        return hit[1]


# ----------------------------------------------------------------------
def layer_norm(x, weight, eps: float, out_dtype: torch.dtype, bias=None):
    """LayerNorm (optional bias) of an fp32 stream, fp32 statistics."""
    if x.is_cuda:
        lib = _load()
        x = _f32(x)
        out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
        C = x.shape[-1]
        _check(lib.nx_layer_norm(_p(x), _p(_f32(weight)),
                                 _p(None if bias is None else _f32(bias)), _p(out), _is_bf16(out),
                                 ctypes.c_long(x.numel() // C), C,
                                 ctypes.c_float(eps), _stream()), "layer_norm")
        return out
    return ref.layer_norm(x, weight, eps, out_dtype, bias)


def add_layer_norm(stream, y, alpha: float, weight, bias, eps: float, copy_dtype=None):
    """Residual step with the norm after the sum, in place on the fp32 stream:
    stream = layer_norm(alpha * stream + y) * weight + bias. Returns the new
    stream in ``copy_dtype`` (the next sublayer's GEMM input; the stream
    itself for float32), None without one."""
    if stream.is_cuda:
        lib = _load()
        assert stream.dtype == torch.float32 and stream.is_contiguous()
        y = y.contiguous()
        assert y.numel() == stream.numel()
        C = stream.shape[-1]
        copy = None
        if copy_dtype is not None and copy_dtype != torch.float32:
            copy = torch.empty(stream.shape, dtype=copy_dtype, device=stream.device)
        _check(lib.nx_add_layer_norm(
            _p(stream), _p(y), _is_bf16(y), ctypes.c_float(alpha), _p(_f32(weight)),
            _p(_f32(bias)), ctypes.c_float(eps), _p(copy), 0 if copy is None else 1,
            ctypes.c_long(stream.numel() // C), C, _stream()), "add_layer_norm")
    else:
        stream.copy_(ref.layer_norm(alpha * stream + y.float(), weight, eps, torch.float32, bias))
        copy = None if copy_dtype in (None, torch.float32) else stream.to(copy_dtype)
    return stream if copy_dtype == torch.float32 else copy


def short_conv(x, w, tail, step: StepLayout, activation: str = "none",
               residual: bool = False, out_dtype=torch.float32, bias=None):
    """Depthwise causal conv over time with a carried tail and an optional
    per-channel bias (see ref.short_conv). Does not advance the tail: call
    short_conv_commit."""
    if x.is_cuda:
        lib = _load()
        B, S, C = x.shape
        y = torch.empty(B, S, C, dtype=out_dtype, device=x.device)
        _check(lib.nx_short_conv(
            _p(x), ctypes.c_long(_rows_view(x)), _is_bf16(x), _p(_f32(w)), _p(tail), _p(step.positions),
            _p(step.seq_ids), _p(step.nvalid), _p(y), _is_bf16(y), B, S, C, w.shape[1],
            int(activation == "silu"), int(residual),
            _p(None if bias is None else _f32(bias)), _stream()), "short_conv")
        return y
    return ref.short_conv(x, w, tail, step.positions, step.seq_ids,
                          activation, residual, out_dtype, bias)


def short_conv_commit(x, tail, step: StepLayout):
    if x.is_cuda:
        lib = _load()
        B, S, C = x.shape
        assert tail.dtype == torch.float32 and tail.is_contiguous()
        _check(lib.nx_short_conv_commit(
            _p(x), ctypes.c_long(_rows_view(x)), _is_bf16(x), _p(tail), _p(step.positions), _p(step.seq_ids),
            _p(step.nvalid), B, S, C, tail.shape[1], _stream()), "short_conv_commit")
        return
    ref.short_conv_commit(x, tail, step.positions, step.seq_ids)


def paged_kv_write(k_cache, v_cache, k_new, v_new, slot_mapping, step: "StepLayout" = None):
    """Scatter k_new (N, G*Dk) / v_new (N, G*Dv) rows (row-strided views
    allowed) into paged caches (blocks, block, G, D*). ``v_cache``/``v_new``
    may be None for caches whose values live inside the key rows."""
    if k_cache.is_cuda:
        lib = _load()
        N = k_new.shape[0]
        GDk = k_cache.shape[2] * k_cache.shape[3]
        GDv = 0 if v_cache is None else v_cache.shape[2] * v_cache.shape[3]
        assert k_new.shape[1] == GDk and k_new.dtype == k_cache.dtype and k_new.stride(1) == 1
        assert k_cache.is_contiguous()
        if v_cache is not None:
            assert v_new.shape[1] == GDv and v_new.dtype == v_cache.dtype == k_cache.dtype
            assert v_new.stride(1) == 1 and v_cache.is_contiguous()
        _check(lib.nx_paged_kv_write(
            _p(k_cache), _p(v_cache), _p(k_new), ctypes.c_long(k_new.stride(0)),
            _p(v_new), ctypes.c_long(0 if v_new is None else v_new.stride(0)),
            _is_bf16(k_cache),
            _p(_i32(slot_mapping) if step is None else step.i32(slot_mapping)),
            ctypes.c_long(N), GDk, GDv,
            ctypes.c_long(k_cache.shape[0] * k_cache.shape[1]), _stream()),
            "paged_kv_write")
        return
    G = k_cache.shape[2]
    ref.paged_kv_write(k_cache, v_cache, k_new.reshape(k_new.shape[0], G, -1),
                       None if v_new is None else v_new.reshape(v_new.shape[0], G, -1),
                       slot_mapping)


def paged_attention(q, k_cache, v_cache, step: StepLayout, block_table, scale: float,
                    num_heads: int, window: Optional[int] = None, keep_first: int = 0,
                    r1=None, r2=None, gate=None, softcap: float = 0.0, sink=None,
                    q_temp=None, out_dtype=None, gate_per_head: bool = False,
                    chunk: int = 0, slopes=None):
    """q (B,S,H*Dk) (row-strided view allowed) against the paged cache ->
    (B,S,H*Dv). Options (see ref.paged_attention): sliding ``window`` with
    ``keep_first`` always-visible tokens (None = plain causal), ``chunk`` > 0
    = only keys of the query's own block of that many positions, log-distance
    penalty ``r1``/``r2`` or linear distance penalty ``slopes`` (H,), tanh
    score cap, per-head softmax ``sink``, query
    temperature ``q_temp`` = (coef, every), sigmoid output ``gate``
    ((B,S,H*Dv), or (B,S,H) with ``gate_per_head``).
    ``v_cache`` may be ``k_cache[..., :Dv]`` (values inside the key rows)."""
    B, S = q.shape[0], q.shape[1]
    H = num_heads
    G, Dk = k_cache.shape[2], k_cache.shape[3]
    Dv = v_cache.shape[3]
    out_dtype = out_dtype or q.dtype
    assert slopes is None or r1 is None, "one distance penalty at a time"
    if q.is_cuda:
        lib = _load()
        out = torch.empty(B, S, H * Dv, dtype=out_dtype, device=q.device)
        bt = step.i32(block_table)
        if slopes is not None:
            r1, r2 = slopes, None          # the kernels read a lone r1 as slopes
        assert k_cache.stride(3) == 1 and v_cache.stride(3) == 1
        assert k_cache.stride(1) == k_cache.stride(2) * G and v_cache.stride(1) == v_cache.stride(2) * G
        assert k_cache.stride(0) == k_cache.stride(1) * k_cache.shape[1]
        assert v_cache.stride(0) == v_cache.stride(1) * v_cache.shape[1]
        assert k_cache.dtype == v_cache.dtype == q.dtype
        coef, every = (0.0, 0) if q_temp is None else (float(q_temp[0]), int(q_temp[1]))
        # single-token steps over latent caches (values inside the one key
        # row): few workgroups per step, so the keys are split over several
        # and merged; the partials need a workspace
        ws, nks = None, 1
        if S == 1 and G == 1 and q.dtype == torch.bfloat16 and \
                v_cache.data_ptr() == k_cache.data_ptr():
            groups = B * ((H + 15) // 16) * ((Dv + 511) // 512)
            span = bt.shape[1] * k_cache.shape[1]           # most keys a token can see
            if window is not None:
                span = min(span, int(window) + 31)
            if chunk:
                span = min(span, int(chunk) + 31)
            nks = max(1, min(8, 256 // max(groups, 1), span // 128))
            if nks > 1:
                ws = torch.empty(B * H * nks * (Dv + 2), dtype=torch.float32, device=q.device)
        _check(lib.nx_paged_attn(
            _p(q), ctypes.c_long(_rows_view(q)), _p(k_cache), ctypes.c_long(k_cache.stride(1)),
            ctypes.c_long(k_cache.stride(2)), _p(v_cache), ctypes.c_long(v_cache.stride(1)),
            ctypes.c_long(v_cache.stride(2)),
            _p(step.positions), _p(step.seq_ids), _p(bt), bt.shape[1],
            _p(None if r1 is None else _f32(r1)), _p(None if r2 is None else _f32(r2)),
            _p(None if sink is None else _f32(sink)),
            _p(gate), ctypes.c_long(0 if gate is None else _rows_view(gate)),
            _p(out), _is_bf16(q), _is_bf16(out), B, S, H, G, Dk, Dv,
            k_cache.shape[1], ctypes.c_float(scale),
            int(window) if window is not None else 0x7fffffff, int(keep_first),
            ctypes.c_float(softcap or 0.0), ctypes.c_float(coef), every,
            _p(ws), nks, int(bool(gate_per_head)), int(chunk or 0), _stream()),
            "paged_attention")
        return out
    return ref.paged_attention(
        q.reshape(B, S, H, Dk), k_cache, v_cache, step.positions, block_table, scale,
        window=window, keep_first=keep_first, r1=r1, r2=r2, gate=gate,
        softcap=softcap or 0.0, sink=sink, q_temp=q_temp, out_dtype=out_dtype,
        gate_per_head=gate_per_head, chunk=int(chunk or 0), slopes=slopes)


def window_bias_attention(q, k_cache, v_cache, step: StepLayout, block_table,
                          r1, r2, scale: float, window: int, keep_first: int,
                          num_heads: int, gate=None, out_dtype=None):
    """Sliding window + kept first tokens with a log-distance penalty."""
    return paged_attention(q, k_cache, v_cache, step, block_table, scale, num_heads,
                           window=window, keep_first=keep_first, r1=r1, r2=r2,
                           gate=gate, out_dtype=out_dtype)


def gated_delta_rule(qkv, beta, a, dt_bias, a_log, gate, norm_w, eps: float,
                     state, step: StepLayout, kv_heads: int, dim: int, vdim: int,
                     out_dtype=torch.float32, gate_act: str = "sigmoid"):
    """Gated delta-rule recurrence over the step's tokens, state carried in
    `state` (slots, H, vdim, dim) fp32; see ref.gated_delta_rule. ``a`` is
    (B,S,H*dim) for a decay per key channel or (B,S,H) for one per head."""
    assert gate_act in ("sigmoid", "silu")
    if qkv.is_cuda:
        lib = _load()
        B, S = qkv.shape[0], qkv.shape[1]
        H = beta.shape[-1]
        per_head = a.shape[-1] == H and dim != 1
        assert a.shape[-1] == (H if per_head else H * dim)
        assert dt_bias.numel() == a.shape[-1]
        assert qkv.dtype == torch.float32 and state.dtype == torch.float32
        assert beta.dtype == a.dtype == gate.dtype == out_dtype
        out = torch.empty(B, S, H * vdim, dtype=out_dtype, device=qkv.device)
        obuf = torch.empty(B, S, H * vdim, dtype=torch.float32, device=qkv.device)
        PS = (2 * kv_heads + H) * dim + H + kv_heads
        prep = torch.empty(B, S, PS, dtype=torch.float32, device=qkv.device)
        _check(lib.nx_gated_delta(
            _p(qkv), ctypes.c_long(_rows_view(qkv)), _p(beta),
            ctypes.c_long(_rows_view(beta)), _p(a), ctypes.c_long(_rows_view(a)),
            _p(gate), ctypes.c_long(_rows_view(gate)), _p(_f32(dt_bias)),
            _p(_f32(a_log)), _p(_f32(norm_w)), ctypes.c_float(eps), _p(state),
            _p(step.positions), _p(step.seq_ids), _p(step.nvalid), _p(prep),
            ctypes.c_long(PS), _p(obuf), _p(out),
            _is_bf16(beta), B, S, H, kv_heads, dim, vdim, int(per_head),
            int(gate_act == "silu"), _stream()),
            "gated_delta_rule")
        return out
    return ref.gated_delta_rule(qkv, beta, a, dt_bias, a_log, gate, norm_w, eps,
                                state, step.positions, step.seq_ids, kv_heads,
                                dim, vdim, out_dtype, gate_act)


HEAD_PRODUCT_MAX_TOKENS = 256


def head_product(a, w):
    """Per-head product a (T,H,K) x w (H,N,K)^T -> (T,H,N), 32-bit sums."""
    T, H, K = a.shape
    out = torch.empty(T, H, w.shape[1], dtype=a.dtype, device=a.device)
    if a.is_cuda and a.dtype == torch.bfloat16 and K % 8 == 0 and T <= HEAD_PRODUCT_MAX_TOKENS \
            and a.is_contiguous() and w.is_contiguous():
        assert w.dtype == a.dtype and w.shape[0] == H and w.shape[2] == K
        _check(_load().nx_head_product(_p(a), _p(w), _p(out), T, H, K, w.shape[1], _stream()),
               "head_product")
        return out
    # (the library's batched product gets no transposed right operand)
    torch.bmm(a.transpose(0, 1), w.transpose(1, 2).contiguous(), out=out.transpose(0, 1))
    return out


def softcap(logits, cap: float):
    """cap * tanh(logits / cap) in fp32."""
    if logits.is_cuda:
        lib = _load()
        x = logits.contiguous()
        out = torch.empty(x.shape, dtype=torch.float32, device=x.device)
        _check(lib.nx_softcap(_p(x), _is_bf16(x), _p(out), ctypes.c_long(x.numel()),
                              ctypes.c_float(cap), _stream()), "softcap")
        return out
    return ref.softcap(logits, cap)


def residual_add(x, a, sa: float = 1.0, b=None, sb: float = 1.0):
    """In place on the fp32 stream: x += sa*a (+ sb*b)."""
    if x.is_cuda:
        lib = _load()
        assert x.dtype == torch.float32 and x.is_contiguous()
        a = a.contiguous()
        if b is not None:
            b = b.contiguous()
            assert b.dtype == a.dtype
        _check(lib.nx_residual_add(_p(x), _p(a), ctypes.c_float(sa), _p(b),
                                   ctypes.c_float(sb), _is_bf16(a),
                                   ctypes.c_long(x.numel()), _stream()), "residual_add")
        return x
    x.add_(a.float(), alpha=sa)
    if b is not None:
        x.add_(b.float(), alpha=sb)
    return x


def _gated_unit(gate_up, silu: bool):
    I = gate_up.shape[-1] // 2
    lib = _load()
    gu = gate_up.contiguous()
    out = torch.empty(gu.shape[:-1] + (I,), dtype=gu.dtype, device=gu.device)
    _check(lib.nx_gelu_mul(_p(gu), _p(out), _is_bf16(gu),
                           ctypes.c_long(gu.numel() // (2 * I)), I, int(silu), _stream()),
           "gated_unit")
    return out


def gelu_tanh_mul_fused(gate_up):
    """(rows, 2I) [gate | up] -> gelu_tanh(gate) * up."""
    if gate_up.is_cuda:
        return _gated_unit(gate_up, False)
    g, u = gate_up.float().chunk(2, dim=-1)
    return ref.gelu_tanh_mul(g, u).to(gate_up.dtype)


def silu_mul_fused(gate_up):
    """(rows, 2I) [gate | up] -> silu(gate) * up."""
    if gate_up.is_cuda:
        return _gated_unit(gate_up, True)
    g, u = gate_up.float().chunk(2, dim=-1)
    return (torch.nn.functional.silu(g) * u).to(gate_up.dtype)


def rms_norm(x, weight, eps: float, one_plus: bool = False, out_dtype=None, out=None):
    """RMS norm over the last axis with fp32 statistics: x / sqrt(mean(x^2)
    + eps) * w (or * (1 + w) for weights stored around zero). ``x`` may be a
    column slice of a wider tensor; ``out`` may be a column slice to fill."""
    out_dtype = out_dtype or (out.dtype if out is not None else x.dtype)
    if x.is_cuda:
        lib = _load()
        C = x.shape[-1]
        if out is None:
            out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
        assert out.shape == x.shape and out.dtype == out_dtype
        rows = x.numel() // C
        _check(lib.nx_rms_norm(
            _p(x), ctypes.c_long(_rows_view(x)), _is_bf16(x), _p(_f32(weight)), int(one_plus),
            ctypes.c_float(eps), _p(out), ctypes.c_long(_rows_view(out)), _is_bf16(out),
            ctypes.c_long(rows), C, _stream()), "rms_norm")
        return out
    y = ref.rms_norm_rows(x, weight, eps, one_plus, out_dtype)
    if out is not None:
        out.copy_(y)
        return out
    return y


def add_rms_norm(stream, y, weight, eps: float, one_plus: bool = True, copy_dtype=None,
                 extra=None, coef=None, next_weight=None):
    """Post-norm residual step on the fp32 stream, in place:
    stream += rms_norm(y) * w (``one_plus``: * (1 + w)). With ``extra``
    (same shape as y) and ``coef`` (rows, n) fp32, the normed vector is
    y + sum(coef[row]) * extra[row] (experts that pass their input through).
    Returns the updated stream cast to ``copy_dtype`` (the next sublayer's
    GEMM input), or, with ``next_weight``, the next sublayer's pre-norm
    rms_norm(stream) * next_weight in ``copy_dtype``; None without a
    ``copy_dtype``."""
    assert (extra is None) == (coef is None)
    if stream.is_cuda:
        lib = _load()
        assert stream.dtype == torch.float32 and stream.is_contiguous()
        y = y.contiguous()
        C = stream.shape[-1]
        rows = stream.numel() // C
        copy = None
        if copy_dtype is not None and (copy_dtype != torch.float32 or next_weight is not None):
            copy = torch.empty(stream.shape, dtype=copy_dtype, device=stream.device)
        nc, cs = 0, 0
        if extra is not None:
            extra = extra.contiguous()
            assert extra.dtype == y.dtype and extra.numel() == y.numel()
            assert coef.dtype == torch.float32 and coef.stride(-1) == 1 and coef.dim() == 2
            assert coef.shape[0] == rows
            nc, cs = coef.shape[1], coef.stride(0)
        _check(lib.nx_add_rms_norm(
            _p(stream), _p(y), _is_bf16(y), _p(_f32(weight)), int(one_plus),
            ctypes.c_float(eps), _p(copy), 0 if copy is None else _is_bf16(copy),
            _p(extra), _p(coef), ctypes.c_long(cs), nc,
            _p(None if next_weight is None else _f32(next_weight)),
            ctypes.c_long(rows), C, _stream()), "add_rms_norm")
        if copy_dtype == torch.float32 and next_weight is None:
            return stream
        return copy
    v = y.float()
    if extra is not None:
        v = v + coef.float().sum(-1).view(*y.shape[:-1], 1) * extra.float()
    stream.add_(ref.rms_norm_rows(v, weight, eps, one_plus, torch.float32))
    if copy_dtype is None:
        return None
    if next_weight is not None:
        return ref.rms_norm_rows(stream, next_weight, eps, False, copy_dtype)
    return stream if copy_dtype == torch.float32 else stream.to(copy_dtype)


def rotate_interleaved(x, step: StepLayout, inv_freq, out=None, out_dtype=None,
                       half_split: bool = False):
    """Rotary positions on interleaved channel pairs (2i, 2i+1) — or, with
    ``half_split``, pairs (i, i + len(inv_freq)) — of the first
    2*len(inv_freq) channels of every head; angles p * inv_freq[i] in fp32.
    x (B,S,N,C), possibly a strided view; ``out`` likewise (may be a slice of
    a wider buffer). Channels past the rotated ones are copied."""
    out_dtype = out_dtype or (out.dtype if out is not None else x.dtype)
    if x.is_cuda:
        lib = _load()
        B, S, N, C = x.shape
        if out is None:
            out = torch.empty(B, S, N, C, dtype=out_dtype, device=x.device)
        assert x.stride(3) == 1 and out.stride(3) == 1
        assert 2 * inv_freq.numel() <= C
        _check(lib.nx_rope_pairs(
            _p(x), ctypes.c_long(_token_stride(x)), ctypes.c_long(x.stride(2)), _is_bf16(x),
            _p(out), ctypes.c_long(_token_stride(out)), ctypes.c_long(out.stride(2)),
            _is_bf16(out),
            _p(step.positions), _p(_f32(inv_freq)), inv_freq.numel(), int(half_split),
            ctypes.c_long(B * S), N, C, _stream()), "rotate_interleaved")
        return out
    y = ref.rotate_pairs(x, step.positions, inv_freq, half_split).to(out_dtype)
    if out is not None:
        out.copy_(y)
        return out
    return y


def clamped_glu_fused(gate_up, limit: float, alpha: float = 1.702):
    """(rows, 2I) [gate | up] -> g*sigmoid(alpha*g)*(u+1) with g = min(gate,
    limit), u = clamp(up, -limit, limit)."""
    I = gate_up.shape[-1] // 2
    if gate_up.is_cuda:
        lib = _load()
        gu = gate_up.contiguous()
        out = torch.empty(gu.shape[:-1] + (I,), dtype=gu.dtype, device=gu.device)
        _check(lib.nx_clamped_glu(_p(gu), _p(out), _is_bf16(gu),
                                  ctypes.c_long(gu.numel() // (2 * I)), I,
                                  ctypes.c_float(limit), ctypes.c_float(alpha), _stream()),
               "clamped_glu_fused")
        return out
    g, u = gate_up.chunk(2, dim=-1)
    return ref.clamped_glu(g, u, limit, alpha).to(gate_up.dtype)


def scaled_embedding(h, scale: float):
    """Embedding rows -> fp32 residual stream, times a constant."""
    return h.float().mul_(scale) if h.dtype != torch.float32 else h * scale


def head_norm_rotate(x, step: StepLayout, norm_weight, eps: float, inv_freq,
                     mscale: float = 1.0, out_dtype=None):
    """Per-head RMS norm (weight shared by the heads, None = none) and
    half-split rotary positions (channel i pairs with i + len(inv_freq), cos
    and sin times ``mscale``; None = no rotation) in one pass, statistics and
    angles in fp32. x (B,S,N,C), possibly a strided view of a fused
    projection; returns a dense (B,S,N*C) tensor."""
    out_dtype = out_dtype or x.dtype
    B, S, N, C = x.shape
    if x.is_cuda:
        lib = _load()
        out = torch.empty(B, S, N * C, dtype=out_dtype, device=x.device)
        assert x.stride(3) == 1
        half = 0 if inv_freq is None else inv_freq.numel()
        assert 2 * half <= C
        _check(lib.nx_head_norm_rope(
            _p(x), ctypes.c_long(_token_stride(x)), ctypes.c_long(x.stride(2)), _is_bf16(x),
            _p(out), _is_bf16(out), _p(step.positions),
            _p(None if norm_weight is None else _f32(norm_weight)), ctypes.c_float(eps),
            _p(None if half == 0 else _f32(inv_freq)), half, ctypes.c_float(mscale),
            ctypes.c_long(B * S), N, C, _stream()), "head_norm_rotate")
        return out
    return ref.head_norm_rotate(x, step.positions, norm_weight, eps, inv_freq,
                                mscale).reshape(B, S, N * C).to(out_dtype)


def low_rank_decay(low, weight, bias, tau: float):
    """Logarithms of per-channel decays from a low-rank projection:
    log(sigmoid(low @ weight.T + bias)) / tau in fp32. low (B,S,rank) may be a
    column slice; weight (C, rank) in the same dtype, bias (C,) fp32."""
    if low.is_cuda:
        lib = _load()
        C, rank = weight.shape
        assert low.shape[-1] == rank and low.dtype == weight.dtype and weight.is_contiguous()
        assert bias.numel() == C
        out = torch.empty(low.shape[:-1] + (C,), dtype=torch.float32, device=low.device)
        _check(lib.nx_low_rank_decay(
            _p(low), ctypes.c_long(_rows_view(low)), _p(weight), _is_bf16(low), _p(_f32(bias)),
            ctypes.c_float(1.0 / tau), _p(out), ctypes.c_long(low.numel() // rank), C, rank,
            _stream()), "low_rank_decay")
        return out
    return ref.low_rank_decay(low, weight, bias, tau)


def decay_scan(q, k, v, state, step: StepLayout, dim: int, vdim: int, dt=None,
               dt_bias=None, a_log=None, head_decay=None, k_scale: float = 1.0, skip=None,
               log_decay=None, weight=None):
    """Decayed linear recurrence with matrix state (see ref.decay_scan):
    selective state spaces (``dt``/``dt_bias``/``a_log``), fixed per-head
    decays (``head_decay``), a decay per key channel (its logarithm
    ``log_decay`` (B,S,H*dim) fp32) or, with ``weight`` (B,S,H) fp32, given
    log decays (B,S,H) and write weights per head and token; the state then
    has one more row per head, of a value channel that is always one (a
    normalizer), and so has the output. q, k (B,S,G*dim), v (B,S,H*vdim) may
    be column slices of wider tensors; ``state`` (slots, H, vdim [+ 1], dim)
    fp32 is read (unless the row starts at position 0) and advanced. Returns
    fp32."""
    assert sum(x is not None for x in (dt, head_decay, log_decay)) == 1
    assert weight is None or log_decay is not None
    if v.is_cuda:
        lib = _load()
        B, S = v.shape[0], v.shape[1]
        H = v.shape[-1] // vdim
        G = q.shape[-1] // dim
        assert q.dtype == k.dtype == v.dtype and state.dtype == torch.float32
        rows = vdim + int(weight is not None)
        assert state.is_contiguous() and tuple(state.shape[1:]) == (H, rows, dim)
        assert H % G == 0 and q.shape[-1] == G * dim and k.shape[-1] == G * dim
        out = torch.empty(B, S, H * rows, dtype=torch.float32, device=v.device)
        channel, dch = log_decay is not None and weight is None, 1
        if weight is not None:
            assert log_decay.dtype == weight.dtype == torch.float32
            assert tuple(log_decay.shape) == tuple(weight.shape) == (B, S, H)
            assert log_decay.is_contiguous() and weight.is_contiguous()
            dt = log_decay
        if channel:
            assert G == H and skip is None and log_decay.shape[-1] == H * dim
            assert log_decay.dtype == torch.float32
            dt, dch = log_decay, dim
        # a long row with few (row, head, channel block) workgroups is cut into
        # segments that scan side by side (two passes joined by a short serial
        # link over the segments' end states)
        groups = B * H * ((rows + 15) // 16)
        nseg, seglen, ws, wdec = 1, S, None, None
        if S >= 256 and groups < 1024:
            nseg = 1
            while nseg * 2 <= min(S // 64, max(1, 2048 // groups)):
                nseg *= 2
            if nseg > 1:
                seglen = ((S + nseg - 1) // nseg + 15) // 16 * 16
                ws = torch.empty(B * nseg * H * rows * dim, dtype=torch.float32, device=v.device)
                wdec = torch.empty(B * nseg * H * dch, dtype=torch.float32, device=v.device)
        _check(lib.nx_decay_scan(
            _p(q), ctypes.c_long(_rows_view(q)), _p(k), ctypes.c_long(_rows_view(k)),
            _p(v), ctypes.c_long(_rows_view(v)), _is_bf16(v),
            _p(dt), ctypes.c_long(0 if dt is None else _rows_view(dt)),
            0 if dt is None else _is_bf16(dt),
            _p(None if dt_bias is None else _f32(dt_bias)),
            _p(None if a_log is None else _f32(a_log)),
            _p(None if head_decay is None else _f32(head_decay)),
            ctypes.c_float(k_scale), _p(None if skip is None else _f32(skip)),
            _p(state), _p(step.positions), _p(step.seq_ids), _p(step.nvalid), _p(out),
            B, S, H, G, dim, rows, _p(ws), _p(wdec), nseg, seglen,
            2 if weight is not None else int(channel), _p(weight), _stream()), "decay_scan")
        return out
    return ref.decay_scan(q, k, v, state, step.positions, step.seq_ids, dim, vdim,
                          dt=dt, dt_bias=dt_bias, a_log=a_log, head_decay=head_decay,
                          k_scale=k_scale, skip=skip, log_decay=log_decay, weight=weight)


CHUNKED_GLA_MIN_TOKENS = 96


def gated_linear_attention(q, k, v, log_decay, gate, norm_weight, eps: float, state,
                           step: StepLayout, dim: int, vdim: int, k_scale: float = 1.0):
    """Recurrence with a decay per key channel and its gated read-out norm:
    decay_scan(log_decay) -> RMS norm per head (weight shared by the heads) ->
    times silu(gate), in the gate's dtype. Long bf16 rows run in chunks on the
    matrix cores with the norm and gate fused; everything else is the scan
    and the norm kernel."""
    B, S = v.shape[0], v.shape[1]
    H = v.shape[-1] // vdim
    if v.is_cuda and S >= CHUNKED_GLA_MIN_TOKENS and dim <= 128 and vdim <= 128 and \
            dim % 8 == 0 and vdim % 8 == 0 and \
            all(t.dtype == torch.bfloat16 for t in (q, k, v, gate)) and \
            all(_rows_view(t) % 8 == 0 and t.data_ptr() % 16 == 0 for t in (q, k, v)):
        lib = _load()
        assert log_decay.dtype == torch.float32 and log_decay.is_contiguous()
        assert log_decay.shape[-1] == H * dim == q.shape[-1] == k.shape[-1]
        assert state.dtype == torch.float32 and state.is_contiguous()
        assert tuple(state.shape[1:]) == (H, vdim, dim) and norm_weight.numel() == vdim
        nc = (S + 63) // 64
        ws = torch.empty(B * nc * H * vdim * dim, dtype=torch.float32, device=v.device)
        wdec = torch.empty(B * nc * H * dim, dtype=torch.float32, device=v.device)
        out = torch.empty(B, S, H * vdim, dtype=torch.bfloat16, device=v.device)
        _check(lib.nx_gla_chunked(
            _p(q), ctypes.c_long(_rows_view(q)), _p(k), ctypes.c_long(_rows_view(k)),
            _p(v), ctypes.c_long(_rows_view(v)), _p(log_decay), ctypes.c_float(k_scale),
            _p(gate), ctypes.c_long(_rows_view(gate)), _p(_f32(norm_weight)), ctypes.c_float(eps),
            _p(state), _p(step.positions), _p(step.seq_ids), _p(step.nvalid), _p(ws), _p(wdec),
            _p(out), B, S, H, dim, vdim, _stream()), "gated_linear_attention")
        return out
    o = decay_scan(q, k, v, state, step, dim, vdim, log_decay=log_decay, k_scale=k_scale)
    return group_gated_norm(o, gate, norm_weight, eps, H, gate_first=False, out_dtype=gate.dtype)


def group_gated_norm(y, gate, weight, eps: float, groups: int, gate_first: bool,
                     out_dtype=torch.float32):
    """RMS norm of fp32 rows in ``groups`` equal parts with a silu gate before
    or after it and an optional weight, of the row's width or of one part's
    (shared by the parts) (see ref.group_gated_norm). ``gate`` may be a column
    slice of a wider tensor."""
    if y.is_cuda:
        lib = _load()
        C = y.shape[-1]
        assert y.dtype == torch.float32 and y.is_contiguous() and C % groups == 0
        out = torch.empty(y.shape, dtype=out_dtype, device=y.device)
        assert weight is None or weight.numel() in (C, C // groups)
        _check(lib.nx_group_gated_norm(
            _p(y), _p(gate), ctypes.c_long(_rows_view(gate)), _is_bf16(gate),
            _p(None if weight is None else _f32(weight)), ctypes.c_float(eps), groups,
            int(gate_first), int(weight is not None and weight.numel() != C), _p(out),
            _is_bf16(out), ctypes.c_long(y.numel() // C), C,
            _stream()), "group_gated_norm")
        return out
    return ref.group_gated_norm(y, gate, weight, eps, groups, gate_first, out_dtype)


CHUNKED_MLSTM_MIN_TOKENS = 64


def mlstm(q, k, v, i_gate, f_gate, gate, i_bias, f_bias, gate_cap: float, norm_weight, eps: float,
          state, max_state, step: StepLayout, dim: int, vdim: int):
    """Matrix memory with exponential gates and its gated read-out norm (see
    ref.mlstm). q, k (B,S,H*dim), v, gate (B,S,H*vdim), i_gate, f_gate
    (B,S,H): raw projections, column slices of one GEMM output are fine;
    ``state`` (slots, H, vdim + 1, dim) and ``max_state`` (slots, H) fp32 are
    read (unless the row starts at position 0) and advanced. Returns
    (B,S,H*vdim) in the gate's dtype. Single-token steps are one launch; long
    bf16 rows run in chunks on the matrix cores; everything else is gates,
    scan and read-out."""
    B, S = v.shape[0], v.shape[1]
    H = v.shape[-1] // vdim
    k_scale = dim ** -0.5
    if not v.is_cuda:
        return ref.mlstm(q, k, v, i_gate, f_gate, gate, i_bias, f_bias, gate_cap, norm_weight, eps,
                         state, max_state, step.positions, step.seq_ids, dim, vdim)
    lib = _load()
    assert q.dtype == k.dtype == v.dtype == gate.dtype == i_gate.dtype == f_gate.dtype
    assert q.shape[-1] == k.shape[-1] == H * dim and gate.shape[-1] == H * vdim
    assert i_gate.shape[-1] == f_gate.shape[-1] == i_bias.numel() == f_bias.numel() == H
    assert state.dtype == max_state.dtype == torch.float32 and norm_weight.numel() == H * vdim
    assert state.is_contiguous() and tuple(state.shape[1:]) == (H, vdim + 1, dim)
    assert max_state.is_contiguous() and tuple(max_state.shape[1:]) == (H,)
    bi, bf, nw = _f32(i_bias), _f32(f_bias), _f32(norm_weight)

    def rows(t):
        return _p(t), ctypes.c_long(_rows_view(t))

    if S == 1 and dim <= 256:
        out = torch.empty(B, S, H * vdim, dtype=gate.dtype, device=v.device)
        _check(lib.nx_mlstm_decode(
            *rows(q), *rows(k), *rows(v), *rows(i_gate), *rows(f_gate), _is_bf16(v), _p(bi), _p(bf),
            ctypes.c_float(gate_cap), ctypes.c_float(k_scale), *rows(gate), _p(nw),
            ctypes.c_float(eps), _p(state), _p(max_state), _p(step.positions), _p(step.seq_ids),
            _p(out), B, H, dim, vdim, _stream()), "mlstm_decode")
        return out
    log_a, w, mx = torch.empty(3, B, S, H, dtype=torch.float32, device=v.device).unbind(0)
    _check(lib.nx_mlstm_gates(
        *rows(i_gate), *rows(f_gate), _is_bf16(i_gate), _p(bi), _p(bf), ctypes.c_float(gate_cap),
        _p(max_state), _p(step.positions), _p(step.seq_ids), _p(step.nvalid), _p(log_a), _p(w),
        _p(mx), B, S, H, _stream()), "mlstm_gates")
    if S >= CHUNKED_MLSTM_MIN_TOKENS and dim <= 128 and vdim <= 128 and dim % 8 == 0 and \
            vdim % 8 == 0 and v.dtype == torch.bfloat16 and \
            all(_rows_view(t) % 8 == 0 and t.data_ptr() % 16 == 0 for t in (q, k, v, gate)):
        nc = (S + 63) // 64
        ws = torch.empty(B * nc * H * (vdim + 1) * dim, dtype=torch.float32, device=v.device)
        wdec = torch.empty(B * nc * H, dtype=torch.float32, device=v.device)
        out = torch.empty(B, S, H * vdim, dtype=torch.bfloat16, device=v.device)
        _check(lib.nx_mlstm_chunked(
            *rows(q), *rows(k), *rows(v), _p(log_a), _p(w), _p(mx), ctypes.c_float(k_scale),
            *rows(gate), _p(nw), ctypes.c_float(eps), _p(state), _p(step.positions),
            _p(step.seq_ids), _p(step.nvalid), _p(ws), _p(wdec), _p(out), B, S, H, dim, vdim,
            _stream()), "mlstm_chunked")
        return out
    o = decay_scan(q, k, v, state, step, dim, vdim, k_scale=k_scale, log_decay=log_a, weight=w)
    out = torch.empty(B, S, H * vdim, dtype=gate.dtype, device=v.device)
    _check(lib.nx_mlstm_readout(
        _p(o), _p(mx), *rows(gate), _is_bf16(gate), _p(nw), ctypes.c_float(eps),
        _p(step.positions), _p(out), ctypes.c_long(B * S), H, vdim, _stream()), "mlstm_readout")
    return out


def group_limited_router(logits, num_experts: int, top_k: int, n_groups: int = 1,
                         keep_groups: int = 1, scale: float = 1.0, normalize: bool = False,
                         correction=None, score: str = "softmax", group_top: int = 1,
                         norm_eps: float = 0.0):
    """Group-limited top-k routing on fp32 logits (T, E + extra) (see
    ref.group_limited_router; ``correction`` (E,) shifts the scores for the
    choice only; ``score``: softmax or sigmoid; a group scores as the sum of
    its ``group_top`` (1 or 2) best): returns (dense (T, E + extra) weights with
    sigmoid gates in the extra columns, idx (T, top_k) int32, weights)."""
    assert score in ("softmax", "sigmoid") and group_top in (1, 2)
    if logits.is_cuda:
        lib = _load()
        T, C = logits.shape
        E = num_experts
        assert logits.dtype == torch.float32 and logits.stride(1) == 1
        assert E % max(n_groups, 1) == 0 and top_k <= E
        dense = torch.empty(T, C, dtype=torch.float32, device=logits.device)
        idx = torch.empty(T, top_k, dtype=torch.int32, device=logits.device)
        wts = torch.empty(T, top_k, dtype=torch.float32, device=logits.device)
        _check(lib.nx_group_router(
            _p(logits), ctypes.c_long(logits.stride(0)), E, C - E, top_k, max(n_groups, 1),
            max(min(keep_groups, n_groups), 1), ctypes.c_float(scale), int(normalize),
            _p(None if correction is None else _f32(correction)), int(score == "sigmoid"),
            int(group_top == 2), ctypes.c_float(norm_eps),
            _p(dense), _p(idx), _p(wts), ctypes.c_long(T), _stream()), "group_limited_router")
        return dense, idx, wts
    return ref.group_limited_router(logits, num_experts, top_k, max(n_groups, 1),
                                    max(min(keep_groups, n_groups), 1), scale, normalize,
                                    correction, score, group_top, norm_eps)


FUSED_ROUTER_MAX_TOKENS = 512


def route_tokens(x, weight, num_experts: int, top_k: int, n_groups: int = 1,
                 keep_groups: int = 1, scale: float = 1.0, normalize: bool = False,
                 correction=None, bias=None, score: str = "softmax", group_top: int = 1,
                 norm_eps: float = 0.0):
    """Router product and selection: fp32 logits ``x.float() @ weight.T + bias``
    (x (T, hidden) in any dtype, weight (E + extra, hidden) fp32), then
    :func:`group_limited_router`. Steps of few tokens do both in one launch;
    larger ones take the library product first."""
    T = x.shape[0]
    assert score in ("softmax", "sigmoid") and group_top in (1, 2)
    if x.is_cuda and 0 < T <= FUSED_ROUTER_MAX_TOKENS and x.stride(-1) == 1:
        lib = _load()
        E, C = num_experts, weight.shape[0]
        assert weight.dtype == torch.float32 and weight.is_contiguous()
        assert weight.shape[1] == x.shape[1] and E % max(n_groups, 1) == 0 and top_k <= E
        dense = torch.empty(T, C, dtype=torch.float32, device=x.device)
        idx = torch.empty(T, top_k, dtype=torch.int32, device=x.device)
        wts = torch.empty(T, top_k, dtype=torch.float32, device=x.device)
        _check(lib.nx_router_fused(
            _p(x), ctypes.c_long(x.stride(0)), _is_bf16(x), _p(weight), weight.shape[1], E, C - E,
            top_k, max(n_groups, 1), max(min(keep_groups, n_groups), 1), ctypes.c_float(scale),
            int(normalize), _p(None if correction is None else _f32(correction)),
            _p(None if bias is None else _f32(bias)), int(score == "sigmoid"),
            int(group_top == 2), ctypes.c_float(norm_eps), _p(dense), _p(idx), _p(wts), ctypes.c_long(T), _stream()), "route_tokens")
        return dense, idx, wts
    logits = torch.nn.functional.linear(x.float(), weight, bias)
    return group_limited_router(logits, num_experts, top_k, n_groups, keep_groups, scale,
                                normalize, correction=correction, score=score,
                                group_top=group_top, norm_eps=norm_eps)


def latent_row_write(x, norm_weight, eps: float, inv_freq, step: StepLayout, k_cache,
                     slot_mapping, kv_rank: int, row=None, half_split: bool = False):
    """Cache row of a latent layer in one pass: x (B,S,kv_rank + rot) (a column
    slice is fine) -> [rms_norm(x[..., :kv_rank]) * w | rotary of the rest in
    interleaved or ``half_split`` pairs] scattered into the paged ``k_cache`` (blocks, block, 1,
    kv_rank + rot) at ``slot_mapping``; ``row`` (B,S,kv_rank + rot, dense)
    also receives it when given."""
    B, S, CR = x.shape
    C, R = kv_rank, CR - kv_rank
    if x.is_cuda:
        lib = _load()
        assert k_cache.is_contiguous() and k_cache.shape[2] * k_cache.shape[3] == CR
        assert k_cache.dtype == x.dtype and x.stride(2) == 1
        assert row is None or (row.is_contiguous() and row.dtype == x.dtype and row.shape == x.shape)
        _check(lib.nx_latent_row(
            _p(x), ctypes.c_long(_token_stride(x)), _is_bf16(x), _p(_f32(norm_weight)),
            ctypes.c_float(eps), _p(_f32(inv_freq)), inv_freq.numel(), int(half_split),
            _p(step.positions), _p(step.i32(slot_mapping)), _p(k_cache),
            ctypes.c_long(k_cache.shape[0] * k_cache.shape[1]), _p(row),
            ctypes.c_long(0 if row is None else CR), ctypes.c_long(B * S), C, R, _stream()),
            "latent_row_write")
        return row
    r = torch.empty(B, S, CR, dtype=x.dtype, device=x.device)
    r[..., :C] = ref.rms_norm_rows(x[..., :C], norm_weight, eps, False, x.dtype)
    r[..., C:] = ref.rotate_pairs(x[..., C:].unsqueeze(2), step.positions, inv_freq,
                                  half_split).squeeze(2).to(x.dtype)
    ref.paged_kv_write(k_cache, None, r.view(B * S, 1, CR), None, slot_mapping)
    if row is not None:
        row.copy_(r)
    return row


EXPERT_ACTS = {"relu2": 0, "gelu": 1}


def act_scale(hid, gates, expert_ff: int, num_experts: int, act: str = "relu2", out_dtype=None):
    """act(x) of (T, E*ff + rest) pre-activations times the token's gate of the
    column's expert; the remaining columns take gate column E, or one when
    ``gates`` has only E columns (see ref.act_scale). ``act``: relu2 (squared
    relu) or gelu (the exact one). ``gates`` None: plain act(x)."""
    out_dtype = out_dtype or hid.dtype
    if hid.is_cuda:
        lib = _load()
        T, C = hid.shape
        assert hid.is_contiguous() and out_dtype == hid.dtype
        out = torch.empty(T, C, dtype=out_dtype, device=hid.device)
        code = EXPERT_ACTS[act]
        if gates is None:
            _check(lib.nx_act_scale(_p(hid), _is_bf16(hid), _p(None), 0, max(C, 1), 1, code,
                                    _p(out), ctypes.c_long(T), C, _stream()), "act_scale")
            return out
        assert gates.dtype == torch.float32 and gates.is_contiguous() and gates.shape[0] == T
        _check(lib.nx_act_scale(_p(hid), _is_bf16(hid), _p(gates), gates.shape[1], expert_ff,
                                num_experts, code, _p(out), ctypes.c_long(T), C, _stream()),
               "act_scale")
        return out
    return ref.act_scale(hid, gates, expert_ff, num_experts, act, out_dtype)


def relu2_scale(hid, gates, expert_ff: int, num_experts: int, out_dtype=None):
    """:func:`act_scale` with the squared relu."""
    return act_scale(hid, gates, expert_ff, num_experts, "relu2", out_dtype)


def clamped_glu_scale(hid, gates, expert_ff: int, num_experts: int, limit: float,
                      shared_limit: float = 0.0, alpha: float = 1.702, out_dtype=None):
    """Clamped gated units of stacked experts (see ref.clamped_glu_scale):
    hid (T, 2*C) = [gate | up] of C = E*ff + shared columns -> (T, C), an
    expert's columns times the token's routing weight ``gates[t, e]`` (fp32,
    (T, >= E), row-strided), the shared columns with their own clamp."""
    if hid.is_cuda:
        return _glu_scale(hid, gates, expert_ff, num_experts, 0, limit, shared_limit, alpha,
                          out_dtype)
    return ref.clamped_glu_scale(hid, gates, expert_ff, num_experts, limit, shared_limit,
                                 alpha, out_dtype or hid.dtype)


def silu_glu_scale(hid, gates, expert_ff: int, num_experts: int, out_dtype=None):
    """silu(gate) * up of stacked experts, times the token's routing weight (see
    :func:`clamped_glu_scale` for the layout)."""
    if hid.is_cuda:
        return _glu_scale(hid, gates, expert_ff, num_experts, 1, 0.0, 0.0, 0.0, out_dtype)
    return ref.silu_glu_scale(hid, gates, expert_ff, num_experts, out_dtype or hid.dtype)


def _glu_scale(hid, gates, expert_ff, num_experts, act, limit, shared_limit, alpha, out_dtype):
    lib = _load()
    T, C2 = hid.shape
    C = C2 // 2
    assert hid.is_contiguous() and out_dtype in (None, hid.dtype) and C2 == 2 * C
    assert num_experts * expert_ff <= C
    if num_experts:
        assert gates.dtype == torch.float32 and gates.stride(1) == 1
        assert gates.shape[0] == T and gates.shape[1] >= num_experts
    out = torch.empty(T, C, dtype=hid.dtype, device=hid.device)
    _check(lib.nx_glu_scale(
        _p(hid), _is_bf16(hid), _p(gates if num_experts else None),
        ctypes.c_long(gates.stride(0) if num_experts else 0), expert_ff, num_experts, act,
        ctypes.c_float(limit), ctypes.c_float(shared_limit), ctypes.c_float(alpha),
        _p(out), ctypes.c_long(T), C, _stream()), "glu_scale")
    return out


def sigmoid_gate_(y, gate):
    """In place: y *= sigmoid(gate). y (..., C) contiguous; ``gate`` of the
    same shape may be a column slice of a wider tensor."""
    if y.is_cuda:
        lib = _load()
        C = y.shape[-1]
        assert y.is_contiguous() and gate.shape == y.shape and gate.dtype == y.dtype
        _check(lib.nx_sigmoid_gate(_p(y), _p(gate), ctypes.c_long(_rows_view(gate)), _is_bf16(y),
                                   ctypes.c_long(y.numel() // C), C, _stream()), "sigmoid_gate")
        return y
    return y.copy_(y.float() * torch.sigmoid(gate.float()))


def scaled_residual(x, terms, eps: float = 0.0):
    """In place on the fp32 stream: x += sum_i f_i(y_i) * w_i for up to three
    terms (y (..., C) in one dtype, w (C,) fp32, normed): f_i is an RMS norm
    over the row (with ``eps``) when ``normed`` else the identity."""
    assert 1 <= len(terms) <= 3
    if x.is_cuda:
        lib = _load()
        C = x.shape[-1]
        assert x.dtype == torch.float32 and x.is_contiguous()
        args = []
        keep = []
        for i in range(3):
            if i < len(terms):
                y, w, normed = terms[i]
                y = y.contiguous()
                assert y.dtype == terms[0][0].dtype and y.numel() == x.numel()
                wf = _f32(w)
                keep += [y, wf]
                args += [_p(y), _p(wf), int(bool(normed))]
            else:
                args += [_p(None), _p(None), 0]
        _check(lib.nx_scaled_residual(_p(x), *args, _is_bf16(terms[0][0]), ctypes.c_float(eps),
                                      ctypes.c_long(x.numel() // C), C, _stream()),
               "scaled_residual")
        return x
    return ref.scaled_residual(x, [(y, w, eps if normed else None) for y, w, normed in terms])


def embed_positions(h, pos_table, step: StepLayout):
    """Token embedding rows (B,S,W) plus a learned position row per token ->
    fp32 residual stream; pad tokens (position -1) take row 0."""
    if h.is_cuda:
        lib = _load()
        h = h.contiguous()
        assert pos_table.dtype == h.dtype and pos_table.is_contiguous()
        W = h.shape[-1]
        out = torch.empty(h.shape, dtype=torch.float32, device=h.device)
        _check(lib.nx_embed_pos(_p(h), _p(pos_table), _is_bf16(h), _p(step.positions), _p(out),
                                ctypes.c_long(h.numel() // W), W, pos_table.shape[0], _stream()),
               "embed_positions")
        return out
    p = step.positions.long().clamp(min=0, max=pos_table.shape[0] - 1)
    return h.float() + pos_table[p].float()


def bigram_embedding(ids, embed, table, last, step: StepLayout, mul_prev: int, mul_cur: int):
    """Token embedding rows plus a bigram row per token -> fp32 residual stream
    (see ref.bigram_embedding). ids (B,S) int64; ``table`` has one more row
    than buckets (the last serves a sequence's first token); ``last`` (slots,)
    int32 carries each sequence's newest token and is advanced."""
    if embed.is_cuda:
        lib = _load()
        B, S = ids.shape
        assert ids.dtype == torch.int64 and ids.is_contiguous() and last.dtype == torch.int32
        assert embed.dtype == table.dtype and embed.is_contiguous() and table.is_contiguous()
        V, W = embed.shape
        out = torch.empty(B, S, W, dtype=torch.float32, device=embed.device)
        _check(lib.nx_bigram_embed(
            _p(ids), _p(step.positions), _p(step.seq_ids), _p(step.nvalid), _p(embed), _p(table),
            _is_bf16(embed), _p(last), ctypes.c_longlong(int(mul_prev)),
            ctypes.c_longlong(int(mul_cur)), ctypes.c_longlong(table.shape[0] - 1), V, _p(out),
            B, S, W, _stream()), "bigram_embedding")
        return out
    return ref.bigram_embedding(ids, embed, table, last, step.positions, step.seq_ids,
                                mul_prev, mul_cur)


def token_gate(z, ids, table, offset: int):
    """gelu_tanh(z) times the token's channels [offset, offset + C) of ``table``
    (vocab, >= offset + C). z (B,S,C) may be a column slice; ids (B,S) int64."""
    C = z.shape[-1]
    if z.is_cuda:
        lib = _load()
        assert ids.dtype == torch.int64 and ids.is_contiguous() and table.dtype == z.dtype
        assert table.is_contiguous() and ids.numel() * C == z.numel()
        out = torch.empty(z.shape, dtype=z.dtype, device=z.device)
        _check(lib.nx_token_gate(_p(z), ctypes.c_long(_rows_view(z)), _p(ids), _p(table),
                                 ctypes.c_long(table.stride(0)), int(offset), table.shape[0],
                                 _is_bf16(z), _p(out), ctypes.c_long(ids.numel()), C, _stream()),
               "token_gate")
        return out
    return ref.token_gate(z, ids, table, offset).to(z.dtype)


def token_gate_proj(h, weight, ids, table, offset: int):
    """:func:`token_gate` of the projection z = h @ weight.T; narrow bf16
    projections of few tokens take one launch for product, gelu and gate."""
    C, K = weight.shape
    if h.is_cuda and h.dtype == torch.bfloat16 and K % 8 == 0 and C <= 256 and \
            h.is_contiguous() and weight.is_contiguous() and ids.numel() <= 1024:
        lib = _load()
        assert ids.dtype == torch.int64 and ids.is_contiguous() and h.shape[-1] == K
        assert table.dtype == weight.dtype == h.dtype and table.is_contiguous()
        out = torch.empty(h.shape[:-1] + (C,), dtype=h.dtype, device=h.device)
        assert ids.numel() * C == out.numel()
        _check(lib.nx_token_gate_proj(
            _p(h), ctypes.c_long(K), _p(weight), K, _p(ids), _p(table),
            ctypes.c_long(table.stride(0)), int(offset), table.shape[0], _p(out),
            ctypes.c_long(ids.numel()), C, _stream()), "token_gate_proj")
        return out
    return token_gate(torch.nn.functional.linear(h, weight), ids, table, offset)


def hyper_step(streams, y, mix, w_out, w_in, norm_weight, eps: float, out_dtype,
               keep: bool = True):
    """One step of a residual kept as parallel streams (fp32): stream t becomes
    sum_s mix[s, t] streams_s + w_out[t] * y, then their weighted sum
    u = sum_t w_in[t] x_t is normed for the next sublayer (layer norm with a
    weight, fp32 statistics). ``streams`` (B,S,n,C), or (B,S,C) when all of
    them still equal one row; ``y`` None reads the streams without changing
    them; ``w_in`` None is the plain sum and ``norm_weight`` None returns u
    itself in fp32. Returns (streams, the normed u in ``out_dtype``);
    ``streams`` is updated in place where it can be, and not made anew
    without ``keep``."""
    n = mix.shape[0]
    B, S, C = streams.shape[0], streams.shape[1], streams.shape[-1]
    shared = streams.dim() == 3
    if streams.is_cuda:
        lib = _load()
        assert streams.dtype == torch.float32 and streams.is_contiguous()
        assert shared or streams.shape[2] == n
        assert tuple(mix.shape) == (n, n) and w_out.numel() == n
        assert w_in is None or w_in.numel() == n
        keep = keep and y is not None
        vec = n <= 4 and C % 4 == 0 and C <= 8192
        if y is not None:
            y = y.contiguous()
            assert y.numel() == B * S * C
        new = streams
        if keep and (shared or not vec):
            new = torch.empty(B, S, n, C, dtype=torch.float32, device=streams.device)
        dt = y.dtype if y is not None else out_dtype
        assert norm_weight is None or out_dtype == dt
        h = torch.empty(B, S, C, dtype=torch.float32 if norm_weight is None else out_dtype,
                        device=streams.device)
        scratch = None
        if norm_weight is not None and not vec:
            scratch = torch.empty(B * S * C, dtype=torch.float32, device=streams.device)
        _check(lib.nx_hyper_step(
            _p(streams), ctypes.c_long(C if shared else n * C), ctypes.c_long(0 if shared else C),
            _p(y), int(dt == torch.bfloat16), _p(_f32(mix)), _p(_f32(w_out)),
            _p(new if keep else None), _p(None if w_in is None else _f32(w_in)),
            _p(None if norm_weight is None else _f32(norm_weight)), ctypes.c_float(eps),
            _p(None if norm_weight is None else h), _p(h if norm_weight is None else None),
            _p(scratch), ctypes.c_long(B * S), n, C, _stream()), "hyper_step")
        return new, h
    new, u = ref.hyper_step(streams, y, mix, w_out, w_in)
    if norm_weight is not None:
        u = ref.layer_norm(u, norm_weight, eps, out_dtype)
    return new, u


def attention_rows(q, k, v, step: StepLayout, inv_freq, unit_norm: bool, eps: float, k_cache,
                   v_cache, slot_mapping, v_first=None, v_lambda=None):
    """Query, key and value rows of a step in one launch: q (B,S,H*D) and k
    (B,S,G*D) rotated (half-split pairs of the first 2*len(inv_freq)
    channels, fp32 angles; None = not) and, with ``unit_norm``, divided by
    their root mean square per head; keys and values (B,S,G*Dv) scattered into
    the paged caches (blocks, block, G, D*) at ``slot_mapping``; with
    ``v_first`` (same shape as v) the values are (1 - lambda) v + lambda
    v_first, ``v_lambda`` a one-element fp32 tensor. Column slices of a fused
    projection are fine. Returns the queries, dense."""
    B, S = q.shape[0], q.shape[1]
    G, D = k_cache.shape[2], k_cache.shape[3]
    Dv = v_cache.shape[3]
    H = q.shape[-1] // D
    assert k.shape[-1] == G * D and v.shape[-1] == G * Dv and q.shape[-1] == H * D
    assert v_first is None or (v_first.shape == v.shape and v_lambda is not None)
    if q.is_cuda:
        lib = _load()
        assert q.dtype == k.dtype == v.dtype == k_cache.dtype == v_cache.dtype
        assert k_cache.is_contiguous() and v_cache.is_contiguous()
        half = 0 if inv_freq is None else inv_freq.numel()
        if v_first is not None:
            assert v_first.dtype == v.dtype and v_lambda.dtype == torch.float32
            assert v_lambda.numel() == 1
        out = torch.empty(B, S, H * D, dtype=q.dtype, device=q.device)
        _check(lib.nx_qkv_rows(
            _p(q), ctypes.c_long(_rows_view(q)), _p(k), ctypes.c_long(_rows_view(k)),
            _p(v), ctypes.c_long(_rows_view(v)), _p(v_first),
            ctypes.c_long(0 if v_first is None else _rows_view(v_first)),
            _p(v_lambda if v_first is not None else None), _is_bf16(q), _p(step.positions),
            _p(step.i32(slot_mapping)), _p(_f32(inv_freq) if half else None), half,
            int(bool(unit_norm)), ctypes.c_float(eps), _p(out), _p(k_cache), _p(v_cache),
            ctypes.c_long(k_cache.shape[0] * k_cache.shape[1]), ctypes.c_long(B * S), H, G, D, Dv,
            _stream()), "attention_rows")
        return out

    def rows(x, n):
        x = ref.head_norm_rotate(x.reshape(B, S, n, D), step.positions, None, 0.0, inv_freq)
        if unit_norm:
            x = x * torch.rsqrt((x * x).mean(-1, keepdim=True) + eps)
        return x.to(q.dtype)

    if v_first is not None:
        lam = v_lambda.float().reshape(())
        v = ((1.0 - lam) * v.float() + lam * v_first.float()).to(v.dtype)
    ref.paged_kv_write(k_cache, v_cache, rows(k, G).view(B * S, G, D), v.reshape(B * S, G, Dv),
                       slot_mapping)
    return rows(q, H).view(B, S, H * D)
