"""Risutar (norm after the residual sum, latent attention with borrowed rows
and per-head gates, gated linear attention, biased top-k experts, bigram and
per-layer token inputs) against the plain float64 oracle in
``risutar_oracle.py``.

Every test builds its own small configuration and weights. The
device-parametrized tests run the torch reference ops on the CPU and the
gfx950 kernels on the GPU (``-m gpu``) through the same engine code.
"""

import copy
import json
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import risutar_oracle as oracle  # noqa: E402

from neuronx_distributed_inference_amd.config import EngineConfig  # noqa: E402
from neuronx_distributed_inference_amd.models.risutar.modeling_risutar import (  # noqa: E402
    RisutarForCausalLM,
    RisutarInferenceConfig,
)
from neuronx_distributed_inference_amd.modules.attention.latent_attention import (  # noqa: E402
    LatentSinkAttention,
)
from neuronx_distributed_inference_amd.modules.kvcache.block_kv_cache_manager import (  # noqa: E402
    BlockKVCacheManager,
    RecurrentStateManager,
    generate_slot_mapping,
)
from neuronx_distributed_inference_amd.modules.linear_recurrence import (  # noqa: E402
    GatedLinearAttention,
)
from neuronx_distributed_inference_amd.modules.mlp import GatedMLP  # noqa: E402
from neuronx_distributed_inference_amd.modules.moe import (  # noqa: E402
    FusedUngatedExperts,
    GroupRoutedFeedForward,
)
from neuronx_distributed_inference_amd.modules.norm import StreamLayerNorm  # noqa: E402
from neuronx_distributed_inference_amd.modules.rope import half_split_inv_freq  # noqa: E402
from neuronx_distributed_inference_amd.modules.token_inputs import TokenSideInput  # noqa: E402
from neuronx_distributed_inference_amd.ops import seqmix  # noqa: E402
from neuronx_distributed_inference_amd.serving import ServingEngine  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32 = torch.float32
BF16 = torch.bfloat16
EPS = 1e-5


# ---------------------------------------------------------------- builders
def latent_cfg(heads=3, dim=8, rot_dim=4, vdim=6, kv_rank=10, q_rank=12, scale=0.3, base=50.0,
               kv_from=None):
    mc = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
          "q_rank": q_rank, "scale": scale, "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        mc["kv_from"] = kv_from
    return mc


def gla_cfg(heads=3, dim=5, vdim=8, tau=4.0, decay_rank=3):
    """``decay_rank`` is no key of the checkpoint's file (the tensors tell)."""
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": decay_rank}


def dense(ff=24):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=8, shared_ff=12):
    fc = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared_ff:
        fc["shared"] = {"ff": shared_ff}
    return fc


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def model_cfg(layers=None, width=16, vocab=37, side=4, buckets=31, mul_prev=7, mul_cur=3,
              alpha=1.7, eps=EPS):
    layers = layers or [
        layer("latent_attention", latent_cfg(), dense()),
        layer("gla", gla_cfg(), moe()),
        layer("latent_attention", latent_cfg(kv_from=0, heads=2, dim=5, vdim=9, q_rank=7,
                                             scale=0.5), moe()),
        layer("gla", gla_cfg(), moe()),
    ]
    return {"architecture": "Risutar", "width": width, "vocab": vocab,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev,
                                     "mul_cur": mul_cur}},
            "token_side": {"dim": side}, "postln_alpha": alpha, "norm": {"eps": eps},
            "layers": layers}


def varied_cfg():
    """Other sizes and another order: the recurrence first, two layers that
    borrow the same rows and one lender nobody borrows from, a layer without
    feed-forward, no shared expert, one expert, every expert chosen, sizes that
    are no powers of two, one head, tau of one (decays far from 1), a rotation
    of two channels, one bucket, large multipliers."""
    la = dict(kv_rank=12, rot_dim=6, base=9.0)
    return model_cfg(layers=[
        layer("gla", gla_cfg(2, 7, 3, tau=1.0, decay_rank=5), moe(3, 3, ff=6, shared_ff=0)),
        layer("latent_attention", latent_cfg(2, 6, vdim=10, q_rank=9, scale=0.5, **la), None),
        layer("latent_attention", latent_cfg(4, 3, vdim=4, q_rank=5, scale=0.7, kv_from=1, **la),
              dense(20)),
        layer("gla", gla_cfg(3, 12, 20, tau=30.0, decay_rank=1), dense(9)),
        layer("latent_attention", latent_cfg(1, 9, 2, 5, 7, q_rank=11, scale=0.4, base=100.0),
              moe(1, 1, ff=10, shared_ff=4)),
        layer("latent_attention", latent_cfg(3, 6, vdim=2, q_rank=13, scale=0.2, kv_from=1, **la),
              moe(7, 3, ff=5, shared_ff=3)),
    ], width=24, vocab=29, side=5, buckets=1, mul_prev=1000003, mul_cur=998244353, alpha=1.3,
        eps=1e-3)


def make_weights(cfg, seed=0):
    """Checkpoint-named tensors, values exactly representable in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    Wd = cfg["width"]

    def rnd(*shape, std=1.0):
        return (torch.randn(*shape, generator=g) * std).bfloat16().float()

    def lin(o, i, gain=1.0):
        return rnd(o, i, std=gain / i ** 0.5)

    def nw(n):
        return (1 + rnd(n, std=0.3)).bfloat16().float()

    W["embed"] = rnd(cfg["vocab"], Wd)
    W["bigram"] = rnd(cfg["embedding"]["bigram"]["buckets"] + 1, Wd)
    side = cfg["token_side"]["dim"]
    W["side.embed"] = rnd(cfg["vocab"], side * len(cfg["layers"]))
    W["head"] = lin(cfg["vocab"], Wd)
    W["final.norm"], W["final.norm.b"] = nw(Wd), rnd(Wd, std=0.2)
    for i, lc in enumerate(cfg["layers"]):
        p = "l%d." % i
        m = p + "mix."
        mc, fc = lc["mixer"], lc["mlp"]
        for n in ("norm1", "norm2") if fc else ("norm1",):
            W[p + n], W[p + n + ".b"] = nw(Wd), rnd(Wd, std=0.2)
        W[p + "side.gate"], W[p + "side.proj"] = lin(side, Wd, 2.0), lin(Wd, side)
        W[p + "side.norm"] = rnd(Wd, std=0.2)
        if lc["type"] == "latent_attention":
            H, D, R, Dv, C = mc["heads"], mc["dim"], mc["rot_dim"], mc["vdim"], mc["kv_rank"]
            W[m + "dq"], W[m + "dq.norm"] = lin(mc["q_rank"], Wd), nw(mc["q_rank"])
            W[m + "uq"] = lin(H * (D + R), mc["q_rank"], 2.0)
            if mc.get("kv_from") is None:
                W[m + "dkv"], W[m + "dkv.norm"] = lin(C + R, Wd), nw(C)
            W[m + "uk"], W[m + "uv"] = lin(H * D, C, 2.0), lin(H * Dv, C)
            W[m + "g"], W[m + "o"] = lin(H, Wd, 2.0), lin(Wd, H * Dv)
        else:
            H, D, Dv, r = mc["heads"], mc["dim"], mc["vdim"], mc["decay_rank"]
            W[m + "q"], W[m + "k"] = lin(H * D, Wd), lin(H * D, Wd)
            W[m + "v"], W[m + "g"] = lin(H * Dv, Wd), lin(H * Dv, Wd, 2.0)
            W[m + "a1"], W[m + "a2"] = lin(r, Wd, 2.0), lin(H * D, r, 2.0)
            W[m + "a2.b"] = rnd(H * D)
            W[m + "norm"], W[m + "o"] = nw(Dv), lin(Wd, H * Dv)
        if not fc:
            continue
        f = p + "mlp."
        if fc["kind"] == "dense":
            W[f + "gate"], W[f + "up"] = lin(fc["ff"], Wd), lin(fc["ff"], Wd)
            W[f + "down"] = lin(Wd, fc["ff"])
            continue
        E, ff = fc["router"]["experts"], fc["expert"]["ff"]
        W[f + "router"], W[f + "router.b"] = lin(E, Wd, 3.0), rnd(E, std=2.0)
        for e in range(E):
            W[f + f"e{e}.up"], W[f + f"e{e}.down"] = lin(ff, Wd), lin(Wd, ff, 2.0)
        if fc.get("shared"):
            sf = fc["shared"]["ff"]
            W[f + "shared.up"], W[f + "shared.down"] = lin(sf, Wd, 2.0), lin(Wd, sf, 2.0)
    return W


def make_engine(cfg, W, device="cpu", dtype="float32", slots=3, page=4, pages=40,
                max_len=96, **engine_kw):
    ec = EngineConfig(batch_size=slots, max_batch_size=slots, kv_cache_batch_size=slots,
                      seq_len=max_len, max_length=max_len, torch_dtype=dtype, tp_degree=1,
                      is_block_kv_layout=True, pa_block_size=page, pa_num_blocks=pages,
                      enable_hip_graphs=False)
    config = RisutarInferenceConfig(neuron_config=ec, **copy.deepcopy(cfg))
    model = RisutarForCausalLM(config)
    sd = RisutarForCausalLM.convert_hf_to_native_state_dict(W, config)
    missing, unexpected = model.model.load_state_dict(sd, strict=False)
    assert not unexpected and all(m.startswith("kv_mgr.") for m in missing), (missing, unexpected)
    model = model.to(device).eval()
    engine_kw.setdefault("capture_decode", False)
    engine_kw.setdefault("async_depth", 1)
    return ServingEngine(model, max_slots=slots, **engine_kw)


def feed(engine, tokens, cuts):
    """One request alone, fed in portions of the given sizes; logits (T, V)."""
    req = engine.admit()
    out, at = [], 0
    for n in cuts:
        lg = engine.forced_step([(req, torch.tensor(tokens[at:at + n]))])
        out.append(lg[0, :n].float().cpu())
        at += n
    assert at == len(tokens)
    engine.release(req)
    return torch.cat(out)


def tokens_for(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def close(got, want, tol, rtol=0.0):
    """|got - want| <= tol + rtol * |want| everywhere."""
    excess = ((got.double() - want.double()).abs() - rtol * want.double().abs()).max().item()
    assert excess < tol, excess


def step_of(positions, seq_ids, device):
    return seqmix.StepLayout(torch.as_tensor(positions).to(device),
                             torch.as_tensor(seq_ids).to(device))


# ------------------------------------------------------------ norms
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n", [20, 32, 264, 2056, 4104, 8200])   # scalar / register forms
def test_residual_step_with_norm_after_the_sum(device, n):
    torch.manual_seed(1)
    x, y = torch.randn(3, 2, n) * 3 + 1.5, torch.randn(3, 2, n)
    norm = StreamLayerNorm(n, eps=1e-3)
    norm.weight.data, norm.bias.data = 1 + 0.3 * torch.randn(n), torch.randn(n)
    want = oracle.post_norm(x.double(), y.double(), 1.7, norm.weight.double(),
                            norm.bias.double(), 1e-3)
    norm = norm.to(device)
    s = x.clone().to(device)
    out = norm.sum_into(s, y.to(device), 1.7, F32)
    assert out is s
    close(s.cpu(), want, 2e-5)
    s = x.clone().to(device)
    cp = norm.sum_into(s, y.to(device), 1.7, BF16)
    close(s.cpu(), want, 2e-5)
    assert cp.dtype == BF16 and torch.equal(cp, s.to(BF16))
    assert norm.sum_into(s, y.to(device), 1.7) is None
    # the plain call (the model's last norm)
    plain = oracle.layer_norm(x.double(), norm.weight.double().cpu(), norm.bias.double().cpu(), 1e-3)
    close(norm(x.to(device)).cpu(), plain, 2e-5)


@pytest.mark.gpu
def test_residual_step_bf16_terms_gpu():
    torch.manual_seed(2)
    x, y = torch.randn(5, 520), torch.randn(5, 520).bfloat16()
    w, b = 1 + 0.3 * torch.randn(520), torch.randn(520)
    want = oracle.post_norm(x.double(), y.double(), 0.8, w.double(), b.double(), EPS)
    s = x.cuda()
    cp = seqmix.add_layer_norm(s, y.cuda(), 0.8, w.cuda(), b.cuda(), EPS, BF16)
    close(s.cpu(), want, 2e-5)
    assert torch.equal(cp, s.bfloat16())


# ------------------------------------------------------------ token inputs
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W,buckets,mul", [(16, 31, (7, 3)), (12, 1, (5, 9)), (40, 97, (1, 1)),
                                           (520, 1009, (2000000011, 1999999973))])
def test_bigram_rows_across_portions_and_slots(device, W, buckets, mul):
    """Every way of cutting gives the whole sequence's rows: the token before
    a portion is the slot's state; a slot's stale token is never read at
    position 0; pad tokens and pad rows change nothing."""
    torch.manual_seed(3)
    V = 50
    weights = {"embed": torch.randn(V, W), "bigram": torch.randn(buckets + 1, W)}
    bg = {"buckets": buckets, "mul_prev": mul[0], "mul_cur": mul[1]}
    a = torch.randint(0, V, (11,)).tolist()
    b = torch.randint(0, V, (6,)).tolist()
    wa, wb = oracle.embed(a, weights, bg), oracle.embed(b, weights, bg)
    emb, tab = weights["embed"].to(device), weights["bigram"].to(device)
    last = torch.full((4,), 49, dtype=torch.int32, device=device)

    def run(ids, pos, seq):
        return seqmix.bigram_embedding(torch.tensor(ids).to(device), emb, tab, last,
                                       step_of(pos, seq, device), *mul).cpu()

    # slot 2 takes a in portions of 4, 1, 6 beside b in slot 1 (1, 3, 2) and a pad row
    y = run([a[:4], [b[0], 0, 0, 0], [5] * 4], [[0, 1, 2, 3], [0, -1, -1, -1], [-1] * 4], [2, 1, -1])
    close(y[0], wa[:4], 1e-6)
    close(y[1, :1], wb[:1], 1e-6)
    assert last[2] == a[3] and last[1] == b[0] and last[0] == 49 and last[3] == 49
    y = run([[a[4], 0, 0], b[1:4]], [[4, -1, -1], [1, 2, 3]], [2, 1])
    close(y[0, :1], wa[4:5], 1e-6)
    close(y[1], wb[1:4], 1e-6)
    y = run([b[4:] + [0] * 4, a[5:]], [[4, 5, -1, -1, -1, -1], list(range(5, 11))], [1, 2])
    close(y[0, :2], wb[4:], 1e-6)
    close(y[1], wa[5:], 1e-6)
    y = run([[b[0]]], [[0]], [2])                       # slot 2 again, for another sequence
    close(y[0], wb[:1], 1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W,dim,index", [(16, 4, 2), (24, 5, 0), (64, 32, 1), (40, 1, 3)])
def test_per_layer_token_input(device, W, dim, index):
    torch.manual_seed(4)
    V, L, T = 30, 4, 7
    toks = torch.randint(0, V, (T,))
    p = f"l{index}.side."
    weights = {"side.embed": torch.randn(V, L * dim), p + "gate": torch.randn(dim, W) * 0.3,
               p + "proj": torch.randn(W, dim), p + "norm": torch.randn(W)}
    x = torch.randn(1, T, W)
    want = oracle.token_side(x[0].double(), toks.tolist(), weights, index, dim, EPS)
    m = TokenSideInput(W, dim, index, EPS, F32)
    m.gate.weight.data, m.proj.weight.data = weights[p + "gate"], weights[p + "proj"]
    m.norm.weight.data = weights[p + "norm"]
    m = m.to(device)
    st = step_of(torch.arange(T).view(1, T), [0], device)
    st.tokens = toks.view(1, T).to(device)
    with torch.no_grad():
        s = x.clone().to(device)
        out = m(s, s.clone(), weights["side.embed"].to(device), st, F32)
        assert out is s
        close(s[0].cpu(), want, 2e-5)
        assert m(s, s, weights["side.embed"].to(device), st, None) is None


@pytest.mark.gpu
def test_per_layer_token_input_bf16_gpu():
    """Token counts below, at and above one tile, narrow and wide sides."""
    torch.manual_seed(5)
    for T, W, dim in [(1, 256, 16), (16, 512, 24), (67, 320, 64), (130, 1024, 48), (3, 72, 9)]:
        V, L, index = 40, 3, 1
        toks = torch.randint(0, V, (T,))
        p = f"l{index}.side."
        weights = {"side.embed": torch.randn(V, L * dim).bfloat16(),
                   p + "gate": (torch.randn(dim, W) * W ** -0.5).bfloat16(),
                   p + "proj": (torch.randn(W, dim) * dim ** -0.5).bfloat16(),
                   p + "norm": torch.randn(W)}
        x = torch.randn(T, 1, W).bfloat16().float()
        want = oracle.token_side(x[:, 0].double(), toks.tolist(), weights, index, dim, EPS)
        m = TokenSideInput(W, dim, index, EPS, BF16)
        m.gate.weight.data, m.proj.weight.data = weights[p + "gate"], weights[p + "proj"]
        m.norm.weight.data = weights[p + "norm"]
        m = m.cuda()
        st = step_of(torch.zeros(T, 1, dtype=torch.long), torch.arange(T), "cuda")
        st.tokens = toks.view(T, 1).cuda()
        with torch.no_grad():
            s = x.cuda()
            m(s, x.bfloat16().cuda(), weights["side.embed"].cuda(), st, BF16)
        assert (s[:, 0].cpu().double() - want).std().item() < 0.01 * want.std().item(), (T, W, dim)


# ------------------------------------------------------------ rotation, latent rows
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("C,dims", [(4, 4), (8, 8), (10, 6), (64, 64)])
def test_half_split_rotation_of_a_slice(device, C, dims):
    torch.manual_seed(6)
    x = torch.randn(2, 5, 3, C + 3)
    pos = torch.tensor([[700, 701, 702, 703, 704], [0, 1, 2, -1, -1]])
    st = step_of(pos, [0, 1], device)
    inv, _ = half_split_inv_freq(77.0, dims)
    got = seqmix.rotate_interleaved(x.to(device)[..., 3:], st, inv.to(device), half_split=True).cpu()
    for b, n in ((0, 5), (1, 3)):
        want = oracle.rotate_halves(x[b, :n, :, 3:].double(), pos[b, :n], 77.0, dims)
        close(got[b, :n], want, 3e-4)                    # fp32 angles near position 700
    inter = seqmix.rotate_interleaved(x.to(device)[..., 3:], st, inv.to(device)).cpu()
    assert dims == 2 or not torch.allclose(inter[0], got[0], atol=1e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("C,R", [(10, 4), (12, 6), (64, 32), (5, 2)])
def test_latent_cache_row_half_split(device, C, R):
    torch.manual_seed(9)
    B, S, page, nblk = 2, 5, 4, 6
    wide = torch.randn(B, S, C + R + 3) * 2
    w = 1 + 0.3 * torch.randn(C)
    pos = torch.tensor([[900, 901, 902, 903, 904], [0, 1, 2, -1, -1]])
    slots = torch.tensor([[17, 18, 19, 4, 5], [9, 10, 11, -1, -1]])
    cache = torch.randn(nblk, page, 1, C + R)
    inv, _ = half_split_inv_freq(100.0, R)
    cd = cache.clone().to(device)
    row = torch.zeros(B, S, C + R, device=device)
    seqmix.latent_row_write(wide.to(device)[..., 3:], w.to(device), EPS, inv.to(device),
                            step_of(pos, [0, 1], device), cd, slots.view(-1).to(device), C,
                            row=row, half_split=True)
    flat = cd.cpu().view(-1, C + R)
    for b in range(B):
        for t in range(S):
            if pos[b, t] < 0:
                continue
            x = wide[b, t, 3:].double()
            want = torch.cat([oracle.rms(x[:C], EPS) * w.double(), oracle.rotate_halves(
                x[C:].view(1, 1, R), pos[b, t:t + 1], 100.0, R).view(R)])
            close(flat[slots[b, t]], want, 3e-4)
            close(row[b, t].cpu(), want, 3e-4)
    untouched = torch.ones(nblk * page, dtype=torch.bool)
    untouched[slots[slots >= 0]] = False
    assert torch.equal(flat[untouched], cache.view(-1, C + R)[untouched])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype,T,H,K,N", [
    (F32, 5, 3, 10, 6), (BF16, 1, 16, 512, 128), (BF16, 7, 4, 64, 40), (BF16, 64, 5, 96, 24),
    (BF16, 33, 2, 72, 16), (BF16, 100, 2, 32, 48), (BF16, 9, 3, 20, 7)])
def test_per_head_product(device, dtype, T, H, K, N):
    if device == "cpu" and dtype == BF16 and T > 40:
        T = 40
    torch.manual_seed(10)
    a = torch.randn(T, H, K).to(dtype)
    w = torch.randn(H, N, K).to(dtype)
    want = torch.stack([a[:, h].double() @ w[h].double().T for h in range(H)], dim=1)
    got = seqmix.head_product(a.to(device), w.to(device)).cpu()
    assert got.dtype == dtype and got.shape == (T, H, N)
    close(got, want, 1e-4 if dtype == F32 else 0.05, 0.0 if dtype == F32 else 0.01)


# ------------------------------------------------------------ latent attention
def _latent_inputs(L, T, dtype, spikes, Wd=14, own=True):
    H, D, R, Dv, C, Q = (L[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
    h = torch.randn(T, Wd).double()
    q = oracle.rms(h @ torch.randn(Wd, Q).double(), EPS) @ (torch.randn(Q, H * (D + R)) * 0.5).double()
    dkv = h @ (torch.randn(Wd, C + R) * 0.6).double()
    gate = h @ torch.randn(Wd, H).double()
    for i, j in spikes:                       # one score stands out, through the rotated part
        dkv[j, C:] *= 5.0
        q.view(T, H, D + R)[i, :, D:] *= 5.0
    W = {"norm": (1 + 0.3 * torch.randn(C)).double(),
         "uk": (torch.randn(H * D, C) * 0.5).bfloat16().double(),
         "uv": (torch.randn(H * Dv, C) * 0.5).bfloat16().double()}
    if dtype != F32:
        q, dkv, gate = (t.to(dtype).double() for t in (q, dkv, gate))
    return q, dkv, gate, W


def _latent_module(L, W, dtype, device, owns=True):
    H, D, R, Dv, C = (L[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    att = LatentSinkAttention(H, D, R, Dv, C, L["scale"], EPS, L["rot"]["base"], R, dtype,
                              sink=False, half_split=True, gate_per_head=True, owns_kv=owns)
    if owns:
        att.latent_norm.weight.data = W["norm"].float()
    att.uk.data, att.uv.data = W["uk"].view(H, D, C).to(dtype), W["uv"].view(H, Dv, C).to(dtype)
    return att.to(device)


def _latent_alone(device, L, T, cuts=None, page=4, dtype=F32, tol=5e-5, spikes=(), fresh=False,
                  borrower=None):
    """A latent layer (and, given ``borrower``, a second one that reads its
    rows with projections of its own) against the oracle."""
    torch.manual_seed(5)
    q, dkv, gate, W = _latent_inputs(L, T, dtype, spikes)
    c, kr = oracle.latent_rows(dkv, W["norm"], L, EPS)
    want = [oracle.latent_attend(q.clone(), c, kr, W["uk"], W["uv"], L, gate)]
    ins = [(q, dkv, gate)]
    mods = [_latent_module(L, W, dtype, device)]
    if borrower is not None:
        q2, _, g2, W2 = _latent_inputs(borrower, T, dtype, spikes)
        want.append(oracle.latent_attend(q2.clone(), c, kr, W2["uk"], W2["uv"], borrower, g2))
        ins.append((q2, None, g2))
        mods.append(_latent_module(borrower, W2, dtype, device, owns=False))
    nblk = (T + page - 1) // page
    mgr = BlockKVCacheManager(len(mods), 1, 1, num_blocks=nblk + 2, block_size=page, dtype=dtype,
                              tp_degree=1, layer_kv_shapes=[m.kv_shape() for m in mods],
                              layer_kv_source=[None, 0][:len(mods)]).to(device)
    assert all(v.numel() == 0 for v in mgr.v_caches) and sum(k.numel() > 0 for k in mgr.k_caches) == 1
    mgr.k_caches[0].data.normal_()                      # stale pages
    bt = torch.randperm(nblk + 2)[:nblk].view(1, nblk).to(device)
    got, at = [[] for _ in mods], 0
    for n in cuts or [T]:
        pos = torch.arange(at, at + n).view(1, n).to(device)
        mgr.set_step_context(bt, generate_slot_mapping(bt, pos, page))
        st = seqmix.StepLayout(pos, torch.zeros(1, dtype=torch.long, device=device))
        st.fresh = fresh and at == 0          # whole-prompt form for the first portion
        for i, m in enumerate(mods):
            a, d, g = (None if t is None else t[at:at + n].view(1, n, -1).to(device, dtype)
                       for t in ins[i])
            got[i].append(m(a, d, mgr, i, st, gate=g)[0].float().cpu())
        at += n
    for g, w in zip(got, want):
        g = torch.cat(g)
        if dtype == F32:
            close(g, w, tol)
        else:
            assert (g.double() - w).std().item() < tol * w.std().item()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("L", [latent_cfg(), latent_cfg(2, 6, 8, 10, 12, base=9.0),
                               latent_cfg(5, 4, 2, 3, 5), latent_cfg(1, 16, 16, 24, 40)])
def test_latent_attention_in_portions(device, L):
    # far keys, page borders, the first tokens, the query itself
    spikes = [(25, 0), (25, 4), (24, 3), (17, 16), (1, 0), (20, 20)]
    _latent_alone(device, L, 26, spikes=spikes)
    _latent_alone(device, L, 26, spikes=spikes, cuts=[1, 2, 7, 1, 1, 1, 13])
    _latent_alone(device, L, 26, spikes=spikes, cuts=[3] + [1] * 23, page=8)
    _latent_alone(device, L, 26, spikes=spikes, cuts=[2] * 13)
    _latent_alone(device, L, 26, spikes=spikes, fresh=True)
    _latent_alone(device, L, 26, spikes=spikes, cuts=[17, 1, 1, 7], fresh=True)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("fresh", [False, True])
def test_borrowed_rows(device, fresh):
    """A second layer with other heads, head sizes and projections reads the
    first one's rows; it stores none itself."""
    L = latent_cfg(2, 6, 8, 10, 12, base=9.0)
    other = latent_cfg(5, 3, 8, 4, 12, scale=0.6, base=9.0)
    spikes = [(25, 0), (24, 7), (12, 11)]
    for cuts in (None, [11, 2, 1, 1, 11], [5] + [1] * 21):
        _latent_alone(device, L, 26, cuts=cuts, spikes=spikes, fresh=fresh, borrower=other)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [None, [250] + [1] * 30, [100, 100, 60, 20]])
def test_latent_attention_far_key_among_hundreds(device, cuts):
    L = latent_cfg(2, 8, 8, 6, 12, scale=0.4, base=10000.0)
    _latent_alone(device, L, 280, cuts=cuts, page=16, tol=2e-4,
                  spikes=[(279, 0), (270, 15), (260, 16), (100, 1), (265, 128), (16, 0)])


@pytest.mark.gpu
@pytest.mark.parametrize("L,cuts", [
    (latent_cfg(4, 32, 16, 32, 64, scale=0.1), None),
    (latent_cfg(6, 24, 8, 40, 72, scale=0.1), [3, 60, 1, 66]),                 # 80-wide rows
    (latent_cfg(8, 64, 32, 64, 96, scale=0.08), [64, 66]),
    # wide rows: 32-key tiles, values split over workgroups, also when decoding
    (latent_cfg(8, 32, 32, 48, 224, scale=0.1), [70, 50] + [1] * 10),
    (latent_cfg(16, 64, 64, 64, 512, scale=0.07), [100] + [1] * 30),
    (latent_cfg(3, 12, 6, 10, 20, scale=0.2), [100, 29, 1]),                   # vector kernel
])
def test_latent_attention_bf16_matrix_path_gpu(L, cuts):
    spikes = [(129, 0), (129, 64), (110, 63), (110, 15), (128, 127)]
    other = dict(L, heads=L["heads"] + 1, scale=L["scale"] * 0.8)
    _latent_alone("cuda", L, 130, spikes=spikes, cuts=cuts, page=16, dtype=BF16, tol=0.03,
                  borrower=other)
    _latent_alone("cuda", L, 130, spikes=spikes, cuts=[100] + [1] * 30, page=16, dtype=BF16,
                  tol=0.03, fresh=True, borrower=other)


@pytest.mark.gpu
@pytest.mark.parametrize("L", [latent_cfg(16, 64, 64, 64, 512, scale=0.07),
                               latent_cfg(20, 32, 32, 48, 224, scale=0.1),
                               latent_cfg(8, 32, 32, 32, 128, scale=0.1)])
def test_latent_attention_decode_key_splits_gpu(L):
    """Single-token steps: the keys are split over several workgroups whose
    partial softmaxes are merged, with the head gates in the merge."""
    spikes = [(619, 0), (619, 300), (605, 127), (605, 511), (610, 609)]
    _latent_alone("cuda", L, 620, spikes=spikes, cuts=[600] + [1] * 20, page=16, dtype=BF16,
                  tol=0.03)


# ------------------------------------------------------------ gated linear attention
def _scan_alone(device, H, D, Dv, T, cuts, tau, dtype=F32, tol=3e-5, shift=0.0, rows=1, zgain=2.0, normed=False):
    """The recurrence from given projections, carried over ``cuts``, state slot
    2 holding garbage at the start."""
    torch.manual_seed(12)
    q, k, z = (torch.randn(rows, T, H * D) for _ in range(3))
    v = torch.randn(rows, T, H * Dv)
    z = z * zgain
    bias = torch.randn(H * D) + shift
    if dtype != F32:
        q, k, v = (t.to(dtype).float() for t in (q, k, v))
    want, state = [], []
    for b in range(rows):
        o, S = oracle.gla_scan(
            q[b].double().view(T, H, D) * D ** -0.5, k[b].double().view(T, H, D),
            v[b].double().view(T, H, Dv),
            oracle.gla_decay((z[b].double() + bias.double()).view(T, H, D), tau))
        want.append(o.reshape(T, H * Dv))
        state.append(S)
    want = torch.stack(want)
    mem = torch.randn(rows + 2, H, Dv, D, device=device)
    keep = mem[:2].clone()
    gate, nw = torch.randn(rows, T, H * Dv), 1 + 0.3 * torch.randn(Dv)
    if dtype != F32:
        gate = gate.to(dtype).float()
    eye = torch.eye(H * D, device=device)
    got, at = [], 0
    for n in cuts:
        pos = torch.arange(at, at + n).view(1, n).expand(rows, n)
        st = step_of(pos, torch.arange(2, 2 + rows), device)
        part = [t[:, at:at + n].to(device, dtype) for t in (q, k, v, gate)]
        ld = seqmix.low_rank_decay(z[:, at:at + n].to(device), eye, bias.to(device), tau)
        if normed:
            got.append(seqmix.gated_linear_attention(
                part[0], part[1], part[2], ld, part[3], nw.to(device), EPS, mem, st, D, Dv,
                k_scale=D ** -0.5).float().cpu())
        else:
            got.append(seqmix.decay_scan(part[0], part[1], part[2], mem, st, D, Dv, log_decay=ld,
                                         k_scale=D ** -0.5).cpu())
        at += n
    assert at == T
    assert torch.equal(mem[:2], keep)                   # other slots are left alone
    got = torch.cat(got, dim=1)
    if normed:
        gd = gate.double()
        want = (oracle.rms(want.view(rows, T, H, Dv), EPS) * nw.double()).view(rows, T, H * Dv)
        want = want * gd * torch.sigmoid(gd)
        if dtype == F32:
            close(got, want, 10 * tol, 10 * tol)
        else:                                           # one rounding of the result
            close(got, want, 3e-3, 5e-3)
    else:
        close(got, want, tol * max(want.abs().max().item(), 1.0))
    S = torch.stack(state)                              # carried for the next step
    close(mem[2:].cpu().transpose(-1, -2) / D ** -0.5, S, tol * max(S.abs().max().item(), 1.0))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,Dv,tau", [(3, 5, 8, 4.0), (1, 12, 20, 16.0), (2, 33, 3, 1.0),
                                        (2, 64, 17, 2.0), (1, 1, 1, 8.0)])
def test_channel_decay_scan_in_portions(device, H, D, Dv, tau):
    for cuts in ([40], [1] * 40, [2, 15, 1, 16, 6], [17, 2, 21]):
        _scan_alone(device, H, D, Dv, 40, cuts, tau)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("zgain,shift,tau", [(30.0, 0.0, 1.0), (2.0, 40.0, 16.0), (60.0, -80.0, 2.0)])
def test_channel_decay_extremes(device, zgain, shift, tau):
    """Decays of nearly one (nothing forgotten), of nearly zero, and both in
    one chunk: no overflow, no loss."""
    _scan_alone(device, 2, 16, 8, 90, [90], tau, shift=shift, zgain=zgain)
    _scan_alone(device, 2, 16, 8, 90, [50, 2, 1, 37], tau, shift=shift, zgain=zgain)


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,Dv,T,cuts", [
    (2, 64, 48, 300, [300]), (3, 128, 128, 700, [700]), (2, 32, 64, 520, [257, 1, 262]),
    (1, 256, 40, 530, [530]), (2, 20, 24, 400, [398, 2]), (4, 128, 64, 193, [97, 96]),
    (2, 96, 80, 333, [64, 128, 141]), (2, 8, 8, 230, [113, 117]), (3, 40, 104, 200, [100, 100]),
    (1, 72, 72, 1100, [1100]), (2, 64, 136, 150, [150])])
def test_channel_decay_scan_long_rows_gpu(H, D, Dv, T, cuts):
    """Rows that are scanned in segments side by side or, in bf16 with the gated
    norm, in chunks on the matrix cores; memory that reaches across all of them;
    decays of nearly zero beside nearly one; the state is exact either way."""
    for dtype, normed in ((F32, False), (BF16, False), (F32, True), (BF16, True)):
        kw = dict(dtype=dtype, normed=normed)
        _scan_alone("cuda", H, D, Dv, T, cuts, 16.0, shift=3.0, **kw)
        _scan_alone("cuda", H, D, Dv, T, cuts, 1.0, zgain=8.0, **kw)
        _scan_alone("cuda", H, D, Dv, T, cuts, 2.0, zgain=60.0, shift=-20.0, **kw)
    _scan_alone("cuda", H, D, Dv, T, cuts, 16.0, dtype=BF16, shift=1.0, rows=3, normed=True)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("C,rank,T", [(24, 3, 5), (300, 16, 33), (16, 70, 17), (8, 128, 2)])
def test_low_rank_log_decay(device, C, rank, T):
    torch.manual_seed(19)
    wide = torch.randn(2, T, rank + 5) * 3
    w, bias = torch.randn(C, rank), torch.randn(C) * 5
    got = seqmix.low_rank_decay(wide.to(device)[..., 5:], w.to(device), bias.to(device), 7.0).cpu()
    z = wide[..., 5:].double() @ w.double().T + bias.double()
    close(got.exp(), oracle.gla_decay(z, 7.0), 2e-5)
    close(got, torch.nn.functional.logsigmoid(z) / 7.0, 1e-4)


@pytest.mark.parametrize("device,lens,chunked", [
    ("cpu", [9, 1, 0, 70], False),
    pytest.param("cuda", [9, 1, 0, 70], False, marks=pytest.mark.gpu),
    pytest.param("cuda", [64, 1, 0, 130], True, marks=pytest.mark.gpu)])   # bf16, matrix cores
def test_scan_of_unequal_rows_and_pads(device, lens, chunked):
    torch.manual_seed(13)
    H, D, Dv, tau = (2, 16, 24, 3.0) if chunked else (2, 6, 5, 3.0)
    S = max(lens)
    q, k, z = (torch.randn(4, S, H * D) for _ in range(3))
    v = torch.randn(4, S, H * Dv)
    bias = torch.randn(H * D)
    pos = torch.full((4, S), -1)
    for b, n in enumerate(lens):
        pos[b, :n] = torch.arange(n)
    mem = torch.randn(4, H, Dv, D, device=device)
    keep = mem[3].clone()
    st = step_of(pos, [2, 0, -1, 1], device)
    ld = seqmix.low_rank_decay(z.to(device), torch.eye(H * D, device=device), bias.to(device), tau)
    if chunked:
        q, k, v = (t.bfloat16().float() for t in (q, k, v))
        gate, nw = torch.randn(4, S, H * Dv).bfloat16(), torch.ones(Dv)
        got = seqmix.gated_linear_attention(
            *(t.to(device, BF16) for t in (q, k, v)), ld, gate.to(device), nw.to(device), EPS, mem,
            st, D, Dv, k_scale=D ** -0.5).float().cpu()
    else:
        got = seqmix.decay_scan(q.to(device), k.to(device), v.to(device), mem, st, D, Dv,
                                log_decay=ld, k_scale=D ** -0.5).cpu()
    for b, n in enumerate(lens):
        if n:
            o, _ = oracle.gla_scan(q[b, :n].double().view(n, H, D) * D ** -0.5,
                                   k[b, :n].double().view(n, H, D), v[b, :n].double().view(n, H, Dv),
                                   oracle.gla_decay((z[b, :n].double() + bias).view(n, H, D), tau))
            if chunked:
                gd = gate[b, :n].double()
                close(got[b, :n], oracle.rms(o, EPS).reshape(n, H * Dv) * gd * torch.sigmoid(gd),
                      3e-3, 5e-3)
            else:
                close(got[b, :n], o.reshape(n, H * Dv), 3e-5)
    assert torch.equal(mem[3], keep)


def _gla_alone(device, mc, T, cuts, Wd=12, dtype=F32, tol=3e-5):
    torch.manual_seed(14)
    cfg = model_cfg(layers=[layer("gla", mc, None)], width=Wd)
    W = make_weights(cfg, seed=15)
    W["l0.mix.o"] = torch.eye(mc["heads"] * mc["vdim"])
    h = torch.randn(T, Wd)
    want = oracle.gla_mixer(h.double(), W, "l0.mix.", mc, EPS)
    H, D, Dv = mc["heads"], mc["dim"], mc["vdim"]
    m = GatedLinearAttention(H, D, Dv, mc["tau"], mc["decay_rank"], EPS, dtype)
    m.decay_up.weight.data = W["l0.mix.a2"].to(dtype)
    m.decay_bias.data, m.norm_weight.data = W["l0.mix.a2.b"], W["l0.mix.norm"]
    m = m.to(device)
    states = RecurrentStateManager(2)
    states.register("x.mem", m.state_shapes()["mem"])
    states.tensors["x_mem"].data.normal_()
    states = states.to(device)
    wide = torch.cat([h @ W["l0.mix." + n].T for n in ("q", "k", "v", "g", "a1")], dim=-1)
    got, at = [], 0
    with torch.no_grad():
        for n in cuts:
            st = step_of(torch.arange(at, at + n).view(1, n), [1], device)
            parts = torch.split(wide[None, at:at + n].to(device, dtype),
                                [H * D, H * D, H * Dv, H * Dv, mc["decay_rank"]], dim=-1)
            got.append(m(*parts, states, "x", st)[0].float().cpu())
            at += n
    got = torch.cat(got)
    if dtype == F32:
        close(got, want, tol)
    else:
        assert (got.double() - want).std().item() < tol * want.std().item()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("mc", [gla_cfg(), gla_cfg(2, 7, 3, tau=1.0, decay_rank=5),
                                gla_cfg(1, 16, 24, tau=16.0, decay_rank=16)])
def test_gated_linear_attention_alone(device, mc):
    for cuts in ([30], [1] * 30, [2] * 15, [13, 1, 1, 15]):
        _gla_alone(device, mc, 30, cuts)


@pytest.mark.gpu
@pytest.mark.parametrize("mc", [gla_cfg(4, 64, 48, 16.0, 16), gla_cfg(2, 128, 128, 8.0, 24),
                                gla_cfg(2, 32, 96, 16.0, 70)])
def test_gated_linear_attention_bf16_gpu(mc):
    for cuts in ([300], [120, 2, 130, 1, 1, 46]):
        _gla_alone("cuda", mc, 300, cuts, Wd=64, dtype=BF16, tol=0.03)


@pytest.mark.parametrize("device", DEVICES)
def test_head_norm_weight_is_shared_by_the_heads(device):
    torch.manual_seed(16)
    y, g, w = torch.randn(2, 3, 4 * 6), torch.randn(2, 3, 4 * 6), torch.randn(6)
    got = seqmix.group_gated_norm(y.to(device), g.to(device), w.to(device), EPS, 4, False).cpu()
    want = (oracle.rms(y.double().view(2, 3, 4, 6), EPS) * w.double()).view(2, 3, 24)
    gd = g.double()
    close(got, want * gd * torch.sigmoid(gd), 1e-5)


# ------------------------------------------------------------ feed-forwards
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,ff,rest", [(3, 5, 7), (4, 8, 16), (2, 16, 0), (1, 8, 8)])
@pytest.mark.parametrize("column", [False, True])
def test_exact_gelu_times_routing_weight(device, E, ff, rest, column):
    """With a gate column the shared expert's columns take it, without one
    they take one; unchosen experts give exact zeros."""
    torch.manual_seed(17)
    T, C = 9, E * ff + rest
    hid = torch.randn(T, C) * 2
    gates = torch.rand(T, E + int(column))
    gates[:, 0] = 0.0
    got = seqmix.act_scale(hid.to(device), gates.to(device), ff, E, act="gelu").cpu()
    full = gates if column else torch.cat([gates, torch.ones(T, 1)], dim=1)
    cols = (torch.arange(C) // ff).clamp(max=E)
    close(got, oracle.gelu_erf(hid.double()) * full.double()[:, cols], 2e-6)
    assert (got[:, :ff] == 0).all()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T,W,E,top", [(5, 24, 7, 2), (64, 64, 16, 4), (9, 136, 3, 3), (6, 10, 1, 1),
                                       (600, 32, 9, 3)])
def test_router_bias_and_softmax_over_the_chosen(device, T, W, E, top):
    """The bias is part of the logits: it moves choice and weights. Weights
    are a softmax over the chosen logits only; few and many tokens."""
    torch.manual_seed(18)
    weights = {"r.router": torch.randn(E, W) * 0.5, "r.router.b": torch.randn(E) * 3}
    x = torch.randn(T, W)
    want_idx, want_w = oracle.route(x.double(), weights, "r.", top)
    dense_w, idx, wts = seqmix.route_tokens(
        x.to(device), weights["r.router"].to(device), E, top, normalize=True,
        bias=weights["r.router.b"].to(device))
    want = torch.zeros(T, E, dtype=torch.float64).scatter(1, want_idx, want_w)
    close(dense_w.cpu(), want, 5e-6)
    close(wts.sum(-1).cpu(), torch.ones(T), 1e-5)
    if E > top:
        unbiased, _, _ = seqmix.route_tokens(x.to(device), weights["r.router"].to(device), E, top,
                                             normalize=True)
        assert ((unbiased.cpu() > 0) != (want > 0)).any()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("fc", [dense(24), dense(7), moe(), moe(3, 3, ff=6, shared_ff=0),
                                moe(1, 1, ff=10, shared_ff=4), moe(8, 2, ff=16, shared_ff=24)])
def test_feed_forwards_alone(device, fc, T=19, Wd=16):
    torch.manual_seed(6)
    W = make_weights(model_cfg(layers=[layer("gla", gla_cfg(), fc)], width=Wd), seed=6)
    h = torch.randn(T, Wd)
    p = "l0.mlp."
    if fc["kind"] == "dense":
        want = oracle.dense_ff(h.double(), W, p)
        m = GatedMLP(Wd, fc["ff"], tp_degree=1, dtype=F32, hidden_act="stream_silu",
                     fused_gate_up=True)
        m.gate_up_proj.weight.data = torch.cat([W[p + "gate"], W[p + "up"]])
        m.down_proj.weight.data = W[p + "down"]
    else:
        want = oracle.moe_ff(h.double(), W, p, fc)
        E, sh = fc["router"]["experts"], bool(fc.get("shared"))
        m = GroupRoutedFeedForward(Wd, E, fc["router"]["top"], fc["expert"]["ff"], F32,
                                   normalize=True, shared_ff=fc["shared"]["ff"] if sh else 0,
                                   shared_gate=False, act="gelu", router_bias=True)
        m.router.weight.data, m.router.bias.data = W[p + "router"], W[p + "router.b"]
        m.experts.up.weight.data = FusedUngatedExperts.stack_up(
            [W[p + f"e{e}.up"] for e in range(E)], W[p + "shared.up"] if sh else None)
        m.experts.down.weight.data = FusedUngatedExperts.stack_down(
            [W[p + f"e{e}.down"] for e in range(E)], W[p + "shared.down"] if sh else None)
    with torch.no_grad():
        got = m.to(device)(h.view(1, T, Wd).to(device))[0].cpu()
    close(got, want, 1e-4)


# ------------------------------------------------------------ whole model
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("make", [model_cfg, varied_cfg])
def test_prefill_decode_portions_match_oracle(device, make):
    cfg = make()
    W = make_weights(cfg, seed=5)
    toks = tokens_for(cfg, 41, seed=6)
    want = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, device)
    close(feed(eng, toks, [41]), want, 3e-4)
    close(feed(eng, toks, [1] * 41), want, 3e-4)          # token by token from the start
    close(feed(eng, toks, [2, 5, 2, 1, 9, 3, 2, 16, 1]), want, 3e-4)
    close(feed(eng, toks, [2] * 20 + [1]), want, 3e-4)
    close(feed(eng, toks, [11] + [1] * 30), want, 3e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_across_many_pages(device):
    cfg = model_cfg()
    W = make_weights(cfg, seed=21)
    toks = tokens_for(cfg, 90, seed=22)
    eng = make_engine(cfg, W, device, pages=30, max_len=96)
    close(feed(eng, toks, [3] + [1] * 87), oracle.forward(cfg, W, toks), 3e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_a_far_token_decides_through_each_mechanism(device):
    """Changing only the FIRST token of a long sequence moves the last logits,
    as much as the oracle says: through a key that stands out (latent
    attention) and through a state that forgets little (recurrence)."""
    for kind in ("latent_attention", "gla"):
        mixer = latent_cfg(2, 8, 4, 12, 12, scale=1.5) if kind == "latent_attention" \
            else gla_cfg(2, 8, 8, tau=64.0)
        cfg = model_cfg(layers=[layer(kind, mixer, None)])
        W = make_weights(cfg, seed=33)
        if kind == "gla":
            W["l0.mix.a2.b"] += 6.0
        toks = tokens_for(cfg, 80, seed=34)
        other = [(toks[0] + 11) % cfg["vocab"]] + toks[1:]
        a, b = oracle.forward(cfg, W, toks), oracle.forward(cfg, W, other)
        assert (a[-1] - b[-1]).abs().max() > 3e-3, kind
        eng = make_engine(cfg, W, device, pages=24, max_len=96)
        for cuts in ([80], [60, 2] + [1] * 18):
            close(feed(eng, toks, cuts)[-1], a[-1], 3e-4)
            close(feed(eng, other, cuts)[-1], b[-1], 3e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("make", [model_cfg, varied_cfg])
def test_residual_stream_per_layer(device, make):
    cfg = make()
    W = make_weights(cfg, seed=7)
    toks = tokens_for(cfg, 9, seed=8)
    streams = []
    oracle.forward(cfg, W, toks, streams)
    eng = make_engine(cfg, W, device)
    seen = []
    hooks = [l.register_forward_hook(lambda m, a, out: seen.append(out.detach().clone().cpu()))
             for l in eng.model.model.layers]
    feed(eng, toks, [9])
    for hk in hooks:
        hk.remove()
    assert len(seen) == len(streams) == len(cfg["layers"])
    for r, s in enumerate(seen):
        close(s[0], streams[r], 1e-4)


def test_only_owners_hold_pages_and_only_recurrences_hold_state():
    cfg = varied_cfg()
    eng = make_engine(cfg, make_weights(cfg, seed=16))
    mgr = eng.kv_mgr
    for i, lc in enumerate(cfg["layers"]):
        mc = lc["mixer"]
        own = lc["type"] == "latent_attention" and mc.get("kv_from") is None
        assert (mgr.k_caches[i].numel() > 0) == own
        assert mgr.v_caches[i].numel() == 0
        if mc.get("kv_from") is not None:
            assert mgr.get_cache(i)[0] is mgr.k_caches[mc["kv_from"]]
    keys = set(mgr.state.tensors.keys())
    assert keys == {"run0_mem", "run3_mem", "last_token"}
    assert mgr.state.get("last_token").dtype == torch.int32
    assert not eng.prefix_caching                 # state is not page-addressable


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("make", [model_cfg, varied_cfg])
def test_mixed_batches_and_reuse(device, make):
    """Unequal requests side by side (portions beside single tokens, one
    request pausing) equal each request alone; slots and pages are handed
    back and used again with stale contents."""
    cfg = make()
    W = make_weights(cfg, seed=9)
    seqs = {n: tokens_for(cfg, L, seed=10 + i)
            for i, (n, L) in enumerate([("a", 30), ("b", 7), ("c", 19), ("d", 26), ("e", 12)])}
    want = {n: oracle.forward(cfg, W, t) for n, t in seqs.items()}
    eng = make_engine(cfg, W, device, slots=3, page=4, pages=18, max_len=32)
    for t in list(eng.kv_mgr.k_caches):
        t.data.normal_()
    for n, t in eng.kv_mgr.state.tensors.items():
        t.data.fill_(5) if t.dtype == torch.int32 else t.data.normal_()
    plan = [                                   # (name, count) per step
        [("a", 6), ("b", 1), ("c", 2)],
        [("a", 1), ("b", 3), ("c", 9)],
        [("a", 11), ("c", 1)],                 # b pauses
        [("a", 1), ("b", 3), ("c", 7)],        # b, c end
        [("a", 1), ("d", 13), ("e", 2)],       # d, e take the freed slots/pages
        [("a", 10), ("d", 1), ("e", 1)],       # a ends
        [("d", 12), ("e", 9)],
    ]
    live, at, got = {}, {n: 0 for n in seqs}, {n: [] for n in seqs}
    for step in plan:
        parts = []
        for n, c in step:
            if n not in live:
                live[n] = eng.admit()
            parts.append((live[n], torch.tensor(seqs[n][at[n]:at[n] + c])))
        lg = eng.forced_step(parts)
        for i, (n, c) in enumerate(step):
            got[n].append(lg[i, :c].float().cpu())
            at[n] += c
            if at[n] == len(seqs[n]):
                eng.release(live.pop(n))
    assert not live and eng.allocator.available() == 18 and len(eng.free_slots) == 3
    for n in seqs:
        close(torch.cat(got[n]), want[n], 3e-4)


def _oracle_greedy(cfg, W, prompt, n_new):
    toks = list(prompt)
    for _ in range(n_new):
        toks.append(int(oracle.forward(cfg, W, toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [dict(), dict(chunk_size=4), dict(chunk_size=4, mixed_chunking=True)])
def test_greedy_generation_through_scheduler(device, kw):
    """Queue -> slots -> (chunked / mixed) prefill -> batched decode; more
    requests than slots, so slots and pages are recycled."""
    cfg = model_cfg()
    W = make_weights(cfg, seed=11)
    prompts = [tokens_for(cfg, n, seed=20 + n) for n in (9, 5, 14, 1)]
    want = [_oracle_greedy(cfg, W, p, 7) for p in prompts]
    eng = make_engine(cfg, W, device, slots=2, page=4, pages=14, max_len=28, **kw)
    rids = [eng.add_request(torch.tensor(p), max_new_tokens=7) for p in prompts]
    out = eng.run()
    assert [out[r] for r in rids] == want


@pytest.mark.gpu
def test_greedy_generation_captured_decode_gpu():
    """The engine's default GPU configuration: hipGraph-captured decode,
    replayed many times beside eager prefills; the carried token and the
    recurrent state survive the capture's warm-up runs."""
    cfg = model_cfg()
    W = make_weights(cfg, seed=11)
    prompts = [tokens_for(cfg, n, seed=20 + n) for n in (9, 5, 14, 6)]
    want = [_oracle_greedy(cfg, W, p, 12) for p in prompts]
    eng = make_engine(cfg, W, "cuda", slots=2, page=4, pages=14, max_len=28,
                      capture_decode=True, async_depth=2)
    rids = [eng.add_request(torch.tensor(p), max_new_tokens=12) for p in prompts]
    out = eng.run()
    assert [out[r] for r in rids] == want


@pytest.mark.gpu
def test_bfloat16_serving_precision_gpu():
    """bf16 projections, fp32 stream/scores/norms/router/recurrence: close to
    the oracle and independent of how the prompt is cut, beyond rounding."""
    lat = dict(heads=8, dim=32, rot_dim=16, vdim=48, kv_rank=64, q_rank=96, scale=0.12)
    cfg = model_cfg(layers=[
        layer("latent_attention", latent_cfg(**lat), dense(256)),
        layer("gla", gla_cfg(4, 32, 40, tau=16.0, decay_rank=12), moe(6, 6, ff=64, shared_ff=48)),
        layer("latent_attention", latent_cfg(kv_from=0, **lat), moe(6, 6, ff=64, shared_ff=48)),
        layer("gla", gla_cfg(4, 32, 40, tau=16.0, decay_rank=12), None),
    ], width=128, vocab=96, side=24, buckets=101)
    W = make_weights(cfg, seed=12)
    toks = tokens_for(cfg, 100, seed=13)
    want = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, "cuda", dtype="bfloat16", page=16, pages=12, max_len=128)
    a = feed(eng, toks, [100])
    b = feed(eng, toks, [7, 30, 2, 1, 1, 59])
    scale = want.std().item()
    assert (a.double() - want).std().item() < 0.04 * scale
    assert (b.double() - want).std().item() < 0.04 * scale
    assert (a - b).double().std().item() < 0.04 * scale


@pytest.mark.gpu
def test_float32_kernels_at_larger_sizes_gpu():
    lat = dict(heads=4, dim=48, rot_dim=24, vdim=40, kv_rank=96, q_rank=112, scale=0.1,
               base=10000.0)
    cfg = model_cfg(layers=[
        layer("gla", gla_cfg(5, 64, 48, tau=8.0, decay_rank=20), moe(8, 3, ff=32, shared_ff=48)),
        layer("latent_attention", latent_cfg(**lat), dense(288)),
        layer("latent_attention", latent_cfg(kv_from=1, **dict(lat, heads=6)), moe(8, 3, ff=40)),
    ], width=160, vocab=101, side=32, buckets=211)
    W = make_weights(cfg, seed=30)
    toks = tokens_for(cfg, 310, seed=31)
    want = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, "cuda", page=16, pages=24, max_len=320, slots=2)
    close(feed(eng, toks, [310]), want, 5e-4)
    close(feed(eng, toks, [100, 7, 2, 160] + [1] * 41), want, 5e-4)


def _write_checkpoint(path, cfg, W):
    from safetensors.torch import save_file

    disk = copy.deepcopy(cfg)
    for lc in disk["layers"]:
        lc["mixer"].pop("decay_rank", None)
    path.mkdir()
    (path / "config.json").write_text(json.dumps(disk))
    save_file({k: v.bfloat16() for k, v in W.items()}, str(path / "model.safetensors"))
    return disk


def test_checkpoint_folder_and_schedule_replay(tmp_path):
    """config.json + model.safetensors on disk -> registry lookup by the
    config's architecture -> schedule replay writes the wanted logits. Sizes
    the file leaves out come from the tensors' shapes."""
    import numpy as np

    from neuronx_distributed_inference_amd import trace_replay
    from neuronx_distributed_inference_amd.registry import model_type_from_config

    cfg = varied_cfg()
    W = make_weights(cfg, seed=14)
    mdir = tmp_path / "model"
    disk = _write_checkpoint(mdir, cfg, W)
    del disk["vocab"], disk["width"], disk["token_side"]["dim"]
    del disk["embedding"]["bigram"]["buckets"]
    for lc in disk["layers"]:
        mc, fc = lc["mixer"], lc["mlp"]
        drop = ("heads", "dim", "vdim") + (() if lc["type"] == "gla" else
                                           ("q_rank", "kv_rank", "rot_dim"))
        for key in drop:
            del mc[key]
        if fc and fc["kind"] == "dense":
            del fc["ff"]
        elif fc:
            del fc["expert"]["ff"], fc["router"]["experts"]
            if fc.get("shared"):
                del fc["shared"]["ff"]
    (mdir / "config.json").write_text(json.dumps(disk))
    assert model_type_from_config(str(mdir)) == "risutar"
    a, b = tokens_for(cfg, 21, 30), tokens_for(cfg, 9, 31)
    lines = [
        {"step": 0, "entries": [{"id": "x", "tokens": a[:8], "want": [0, 7]}], "end": []},
        {"step": 1, "entries": [{"id": "x", "tokens": a[8:20], "want": []},
                                {"id": "y", "tokens": b[:1], "want": [0]}], "end": []},
        {"step": 2, "entries": [{"id": "y", "tokens": b[1:], "want": [7]},
                                {"id": "x", "tokens": a[20:], "want": [0]}], "end": ["x", "y"]},
    ]
    out = tmp_path / "out"
    out.mkdir()
    eng = trace_replay.build_engine(str(mdir), "float32", 128, device=torch.device("cpu"))
    said = []
    trace_replay.replay(eng, [json.dumps(x) for x in lines], str(out), said.append)
    assert said == ["done 0", "done 1", "done 2"]
    wa, wb = oracle.forward(cfg, W, a), oracle.forward(cfg, W, b)
    g = [torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
         for i in range(3)]
    close(g[0], wa[[0, 7]], 3e-4)
    close(g[1], wb[[0]], 3e-4)
    close(g[2], torch.stack([wb[8], wa[20]]), 3e-4)


def test_command_line_generation(tmp_path, capsys):
    """inference_demo --model-type risutar: checkpoint folder -> compile ->
    load -> greedy generation, the same path as every other family."""
    from neuronx_distributed_inference_amd.inference_demo import main

    cfg = model_cfg()
    W = make_weights(cfg, seed=3)
    mdir = tmp_path / "model"
    _write_checkpoint(mdir, cfg, W)
    prompt = tokens_for(cfg, 9, seed=1)
    rc = main(["--model-type", "risutar", "run", "--model-path", str(mdir),
               "--compiled-model-path", str(tmp_path / "compiled"),
               "--prompt-ids", json.dumps([prompt]), "--max-new-tokens", "6",
               "--torch-dtype", "float32", "--on-cpu", "--seq-len", "32",
               "--max-context-length", "16"])
    assert rc == 0
    printed = [json.loads(l) for l in capsys.readouterr().out.splitlines() if l.startswith("[[")]
    assert printed and printed[-1][0] == prompt + _oracle_greedy(cfg, W, prompt, 6)


def test_config_rejects_what_it_does_not_know():
    cfg = model_cfg()
    for change in (lambda c: c["layers"][1].update(type="window"),
                   lambda c: c["layers"][0]["mlp"].update(kind="experts"),
                   lambda c: c["layers"][2]["mixer"].update(kv_from=2),       # itself
                   lambda c: c["layers"][2]["mixer"].update(kv_from=1),       # a recurrence
                   lambda c: c["layers"][2]["mixer"].update(kv_from=9),       # no such layer
                   lambda c: c["layers"][2]["mixer"].update(kv_rank=11),      # not the lender's
                   lambda c: c["layers"][3]["mixer"].pop("decay_rank"),
                   lambda c: c["layers"][1]["mlp"]["router"].update(top=9)):
        bad = copy.deepcopy(cfg)
        change(bad)
        with pytest.raises(ValueError):
            RisutarInferenceConfig(neuron_config=EngineConfig(tp_degree=1), **bad)


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_generate_adapter(device):
    """The plain generate() entry point (no page table passed: the model
    lays its slots out linearly over the page pool)."""
    from neuronx_distributed_inference_amd.utils.hf_adapter import (
        GenerationConfig,
        HuggingFaceGenerationAdapter,
    )

    cfg = model_cfg()
    W = make_weights(cfg, seed=15)
    prompts = [tokens_for(cfg, 8, seed=40), tokens_for(cfg, 8, seed=41)]
    want = [_oracle_greedy(cfg, W, p, 6) for p in prompts]
    eng = make_engine(cfg, W, device, slots=2, page=4, pages=16, max_len=32)
    out = HuggingFaceGenerationAdapter(eng.model).generate(
        torch.tensor(prompts, device=device),
        generation_config=GenerationConfig(max_new_tokens=6))
    assert out[:, 8:].tolist() == want
