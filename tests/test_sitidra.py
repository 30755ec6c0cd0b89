"""Sitidra (parallel residual streams, chunk-local rotary attention with unit
norms, blended values and per-head gates, matrix memory with exponential gates,
sigmoid-scored group-routed experts) against the plain float64 oracle in
``sitidra_oracle.py``.

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
import sitidra_oracle as oracle  # noqa: E402

from neuronx_distributed_inference_amd.config import EngineConfig  # noqa: E402
from neuronx_distributed_inference_amd.models.sitidra.modeling_sitidra import (  # noqa: E402
    SitidraForCausalLM,
    SitidraInferenceConfig,
)
from neuronx_distributed_inference_amd.modules.attention.chunked_rotary_attention import (  # noqa: E402
    ChunkedRotaryAttention,
)
from neuronx_distributed_inference_amd.modules.hyper_connection import (  # noqa: E402
    HyperConnection,
)
from neuronx_distributed_inference_amd.modules.kvcache.block_kv_cache_manager import (  # noqa: E402
    BlockKVCacheManager,
    RecurrentStateManager,
    generate_slot_mapping,
)
from neuronx_distributed_inference_amd.modules.linear_recurrence import (  # noqa: E402
    ExponentialGateMemory,
)
from neuronx_distributed_inference_amd.modules.moe import (  # noqa: E402
    FusedGatedExperts,
    GroupRoutedFeedForward,
)
from neuronx_distributed_inference_amd.modules.norm import StreamLayerNorm  # noqa: E402
from neuronx_distributed_inference_amd.modules.rope import half_split_inv_freq  # noqa: E402
from neuronx_distributed_inference_amd.ops import seqmix  # noqa: E402
from neuronx_distributed_inference_amd.serving import ServingEngine  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32 = torch.float32
BF16 = torch.bfloat16
EPS = 1e-5
ROUTER = dict(correction=True, score="sigmoid", group_top=2, norm_eps=1e-20)


# ---------------------------------------------------------------- builders
def att_cfg(heads=6, kv_heads=3, dim=8, vdim=5, size=11, scale=0.9, base=60.0, dims=6,
            v_mix=True):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
            "mask": {"size": size}, "rot": {"base": base, "dims": dims}, "v_mix": v_mix}


def mem_cfg(heads=3, dim=5, vdim=7, gate_cap=4.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}


def moe(experts=6, top=2, ff=8, shared_ff=12, count=3, keep=2, scale=1.7):
    fc = {"kind": "moe", "expert": {"ff": ff},
          "router": {"experts": experts, "top": top, "scale": scale,
                     "groups": {"count": count, "keep": keep}}}
    if shared_ff:
        fc["shared"] = {"ff": shared_ff}
    return fc


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def model_cfg(layers=None, width=20, vocab=37, streams=2, cap=9.0, eps=EPS):
    layers = layers or [
        layer("attention", att_cfg(), moe()),
        layer("mlstm", mem_cfg(), moe()),
        layer("attention", att_cfg(), moe()),
        layer("mlstm", mem_cfg(), moe()),
    ]
    return {"architecture": "Sitidra", "width": width, "vocab": vocab, "streams": streams,
            "norm": {"eps": eps}, "logit_softcap": cap, "layers": layers}


def varied_cfg():
    """Other sizes and another order: the recurrence first, an attention layer
    outside the value mixing before its first layer, blocks of one position
    and longer than the sequence, a layer without feed-forward, no shared
    expert, one expert, every expert chosen, one group, groups of one expert,
    as many key/value heads as heads and a single one, a rotation of two
    channels and of the whole head, equal key and value sizes, a low and a
    high gate cap, five streams, no cap on the logits."""
    return model_cfg(layers=[
        layer("mlstm", mem_cfg(2, 6, 3, gate_cap=0.7), moe(3, 3, ff=6, shared_ff=0, count=1, keep=1)),
        layer("attention", att_cfg(2, 2, 6, 6, size=500, dims=2, scale=0.4, v_mix=False), None),
        layer("attention", att_cfg(4, 1, 10, 6, size=7, dims=10, scale=1.3), moe(4, 2, ff=5, count=4,
                                                                                 keep=3, shared_ff=3)),
        layer("mlstm", mem_cfg(1, 12, 20, gate_cap=30.0), None),
        layer("attention", att_cfg(3, 3, 4, 2, size=1, dims=4), moe(1, 1, ff=10, shared_ff=4, count=1,
                                                                    keep=1, scale=0.6)),
        layer("attention", att_cfg(2, 2, 6, 3, size=16, dims=4, base=9.0, scale=2.0),
              moe(8, 3, ff=5, shared_ff=7, count=2, keep=1, scale=3.0)),
    ], width=28, vocab=29, streams=5, cap=None, eps=1e-3)


def make_weights(cfg, seed=0):
    """Checkpoint-named tensors, values exactly representable in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    Wd, n = cfg["width"], cfg["streams"]

    def rnd(*shape, std=1.0):
        return (torch.randn(*shape, generator=g) * std).bfloat16().float()

    def lin(o, i, gain=1.0):
        return rnd(o, i, std=gain / i ** 0.5)

    def nw(m):
        return (1 + rnd(m, std=0.3)).bfloat16().float()

    W["embed"] = rnd(cfg["vocab"], Wd)
    W["head"] = lin(cfg["vocab"], Wd, 2.0)
    W["final.norm"] = nw(Wd)
    for i, lc in enumerate(cfg["layers"]):
        p = "l%d." % i
        m = p + "mix."
        mc, fc = lc["mixer"], lc["mlp"]
        for q in (1, 2) if fc else (1,):
            W[p + f"norm{q}"] = nw(Wd)
            W[p + f"hc{q}.in"] = (1.0 / n + rnd(n, std=0.3)).bfloat16().float()
            W[p + f"hc{q}.out"] = (1.0 + rnd(n, std=0.4)).bfloat16().float()
            W[p + f"hc{q}.mix"] = (0.8 * torch.eye(n) + rnd(n, n, std=0.3 / n)).bfloat16().float()
        if lc["type"] == "attention":
            H, G, D, Dv = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
            W[m + "q"], W[m + "k"] = lin(H * D, Wd), lin(G * D, Wd)
            W[m + "v"], W[m + "vmix"] = lin(G * Dv, Wd), rnd(1, std=0.5).reshape(())
            W[m + "g"], W[m + "o"] = lin(H, Wd, 2.0), lin(Wd, H * Dv, 2.0)
        else:
            H, D, Dv = mc["heads"], mc["dim"], mc["vdim"]
            W[m + "q"], W[m + "k"] = lin(H * D, Wd), lin(H * D, Wd)
            W[m + "v"], W[m + "g"] = lin(H * Dv, Wd), lin(H * Dv, Wd, 2.0)
            W[m + "i"], W[m + "i.b"] = lin(H, Wd, 2.0), rnd(H)
            W[m + "f"], W[m + "f.b"] = lin(H, Wd, 2.0), (2.0 + rnd(H)).bfloat16().float()
            W[m + "norm"], W[m + "o"] = nw(H * Dv), lin(Wd, H * Dv, 2.0)
        if not fc:
            continue
        f = p + "mlp."
        E, ff = fc["router"]["experts"], fc["expert"]["ff"]
        W[f + "router"], W[f + "correction"] = lin(E, Wd, 3.0), rnd(E, std=0.5)
        for e in range(E):
            W[f + f"e{e}.gate"], W[f + f"e{e}.up"] = lin(ff, Wd, 2.0), lin(ff, Wd)
            W[f + f"e{e}.down"] = lin(Wd, ff, 2.0)
        if fc.get("shared"):
            sf = fc["shared"]["ff"]
            W[f + "shared.gate"], W[f + "shared.up"] = lin(sf, Wd, 2.0), lin(sf, Wd)
            W[f + "shared.down"] = lin(Wd, sf, 2.0)
    return W


def make_engine(cfg, W, device="cpu", dtype="float32", slots=3, page=4, pages=40,
                max_len=96, **engine_kw):
    ec = EngineConfig(batch_size=slots, max_batch_size=slots, kv_cache_batch_size=slots,
                      seq_len=max_len, max_length=max_len, torch_dtype=dtype, tp_degree=1,
                      is_block_kv_layout=True, pa_block_size=page, pa_num_blocks=pages,
                      enable_hip_graphs=False)
    config = SitidraInferenceConfig(neuron_config=ec, **copy.deepcopy(cfg))
    model = SitidraForCausalLM(config)
    sd = SitidraForCausalLM.convert_hf_to_native_state_dict(W, config)
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


# ------------------------------------------------------------ parallel streams
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n,C", [(1, 24), (2, 20), (3, 7), (4, 1028), (3, 2052), (2, 4100), (4, 8192),
                                 (5, 16), (7, 33), (2, 8200)])      # register / scalar forms
def test_streams_read_write_and_sum(device, n, C):
    torch.manual_seed(1)
    xs = torch.randn(2, 3, n, C) * 2 + 0.5
    y, y2 = torch.randn(2, 3, C), torch.randn(2, 3, C)
    a, b = HyperConnection(n), HyperConnection(n)
    for h in (a, b):
        h.w_in.data, h.w_out.data = torch.randn(n), torch.randn(n)
        h.mix.data = torch.randn(n, n)                  # not symmetric: [from, to]
    nw = 1 + 0.3 * torch.randn(C)
    d = {k: getattr(a, k).data.double() for k in ("w_in", "w_out", "mix")}
    e = {k: getattr(b, k).data.double() for k in ("w_in", "w_out", "mix")}
    x1 = oracle.hyper_write(xs.double().view(6, n, C), y.double().view(6, C), d["mix"], d["w_out"])
    h1 = oracle.layer_norm(oracle.hyper_read(x1, e["w_in"]), nw.double(), 1e-3)
    total = oracle.hyper_write(x1, y2.double().view(6, C), e["mix"], e["w_out"]).sum(1)
    a, b = a.to(device), b.to(device)
    norm = StreamLayerNorm(C, eps=1e-3, bias=False)
    norm.weight.data = nw
    norm = norm.to(device)
    s, h = a.write(xs.clone().to(device), y.to(device), (b.w_in, norm.weight), 1e-3, F32)
    assert s.shape == xs.shape and h.shape == y.shape
    close(s.cpu().view(6, n, C), x1, 2e-5)
    close(h.cpu().view(6, C), h1, 5e-5)
    close(b.read(s, norm, F32).cpu().view(6, C), h1, 5e-5)
    _, u = b.write(s, y2.to(device), None, 1e-3, F32)
    assert u.dtype == F32
    close(u.cpu().view(6, C), total, 1e-4)
    close(norm(u).cpu().view(6, C), oracle.layer_norm(total, nw.double(), 1e-3), 1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n,C", [(3, 24), (6, 10)])
def test_streams_start_as_one_row(device, n, C):
    """The first write spreads one shared row; the row itself stays as it is."""
    torch.manual_seed(2)
    x, y = torch.randn(1, 4, C), torch.randn(1, 4, C)
    hc, norm = HyperConnection(n), StreamLayerNorm(C, eps=EPS, bias=False)
    hc.w_in.data, hc.w_out.data, hc.mix.data = torch.randn(n), torch.randn(n), torch.randn(n, n)
    spread = x[0].double().unsqueeze(1).repeat(1, n, 1)
    want_h = oracle.layer_norm(oracle.hyper_read(spread, hc.w_in.double()), norm.weight.double(), EPS)
    want = oracle.hyper_write(spread, y[0].double(), hc.mix.double(), hc.w_out.double())
    hc, norm = hc.to(device), norm.to(device)
    row = x.clone().to(device)
    close(hc.read(row, norm, F32).cpu()[0], want_h, 2e-5)
    s, _ = hc.write(row, y.to(device), (hc.w_in, norm.weight), EPS, F32)
    close(s.cpu()[0], want, 2e-5)
    assert torch.equal(row.cpu(), x)
    _, u = hc.write(row, y.to(device), None, EPS, F32)      # a model of one sublayer
    close(u.cpu()[0], want.sum(1), 2e-5)


@pytest.mark.gpu
def test_streams_bf16_terms_gpu():
    torch.manual_seed(3)
    for n, C in ((3, 520), (4, 96), (6, 50)):
        xs, y = torch.randn(1, 5, n, C), torch.randn(1, 5, C).bfloat16()
        hc = HyperConnection(n)
        hc.w_in.data, hc.w_out.data, hc.mix.data = torch.randn(n), torch.randn(n), torch.randn(n, n)
        nw = 1 + 0.3 * torch.randn(C)
        want = oracle.hyper_write(xs[0].double(), y[0].double(), hc.mix.double(), hc.w_out.double())
        wh = oracle.layer_norm(oracle.hyper_read(want, hc.w_in.double()), nw.double(), EPS)
        hc = hc.cuda()
        s, h = hc.write(xs.cuda(), y.cuda(), (hc.w_in, nw.cuda()), EPS, BF16)
        assert h.dtype == BF16 and s.dtype == F32
        close(s.cpu()[0], want, 2e-5)
        close(h.cpu()[0], wh, 1e-3, 0.005)


# ------------------------------------------------------------ attention rows
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("H,G,D,Dv,dims", [(3, 1, 8, 6, 4), (4, 2, 16, 8, 16), (6, 3, 24, 16, 16),
                                           (2, 2, 5, 3, 4), (5, 1, 128, 64, 64), (2, 1, 72, 40, 48),
                                           (2, 1, 16, 8, 0)])
def test_query_key_value_rows(device, dtype, H, G, D, Dv, dims):
    """Rotation, unit norms, value blend and page scatter of column slices, at
    far positions, beside pad tokens and over stale pages."""
    torch.manual_seed(4)
    wide = torch.randn(2, 5, H * D + G * D + G * Dv + 8).to(dtype)
    first = torch.randn(2, 5, G * Dv + 8).to(dtype)
    q, k, v = torch.split(wide[..., :-8], [H * D, G * D, G * Dv], dim=-1)
    pos = torch.tensor([[700, 701, 702, 703, 704], [0, 1, 2, -1, -1]])
    page, nblk = 4, 6
    slots = torch.tensor([[17, 18, 19, 8, 9], [0, 1, 2, -1, -1]])
    lam = torch.tensor([0.3])
    inv = half_split_inv_freq(70.0, dims)[0] if dims else None
    mc = {"rot": {"base": 70.0, "dims": dims} if dims else None}
    for blend in (False, True):
        kc, vc = torch.randn(nblk, page, G, D).to(dtype), torch.randn(nblk, page, G, Dv).to(dtype)
        gk, gv = kc.clone().to(device), vc.clone().to(device)
        st = step_of(pos, [0, 1], device)
        dev = [t.to(device) for t in (wide, first)]
        qd, kd, vd = torch.split(dev[0][..., :-8], [H * D, G * D, G * Dv], dim=-1)
        got = seqmix.attention_rows(
            qd, kd, vd, st, None if inv is None else inv.to(device), True, EPS, gk, gv,
            slots.flatten().to(device), dev[1][..., :G * Dv] if blend else None,
            lam.to(device) if blend else None).cpu()
        tol = (3e-4, 0.0) if dtype == F32 else (2e-3, 0.006)
        flat_k, flat_v = gk.view(-1, G, D).cpu(), gv.view(-1, G, Dv).cpu()
        for b, n in ((0, 5), (1, 3)):
            def unit(x, heads):
                x = x[b, :n].double().view(n, heads, D)
                if dims:
                    x = oracle.rotate_halves(x, pos[b, :n], mc["rot"]["base"], dims)
                return oracle.rms(x, EPS)
            close(got[b, :n].view(n, H, D), unit(q, H), *tol)
            close(flat_k[slots[b, :n]], unit(k, G), *tol)
            wv = v[b, :n].double()
            if blend:
                wv = oracle.mix_values(wv, first[b, :n, :G * Dv].double(), lam.double())
            close(flat_v[slots[b, :n]], wv.view(n, G, Dv), *tol)
        untouched = torch.ones(nblk * page, dtype=torch.bool)
        untouched[slots[slots >= 0]] = False
        assert torch.equal(flat_k[untouched], kc.view(-1, G, D)[untouched])
        assert torch.equal(flat_v[untouched], vc.view(-1, G, Dv)[untouched])


# ------------------------------------------------------------ attention
def _attention_alone(device, L, T, cuts=None, page=4, dtype=F32, tol=5e-5, spikes=(), blend=True):
    """An attention core against the oracle over a paged cache. ``spikes``
    (i, j): query i lines up with key j after both rotations, so one score
    stands out wherever it is seen."""
    torch.manual_seed(5)
    H, G, D, Dv = (L[k] for k in ("heads", "kv_heads", "dim", "vdim"))
    rot = L["rot"]
    q, k, v, first = (torch.randn(T, n).double() for n in (H * D, G * D, G * Dv, G * Dv))
    gate = torch.randn(T, H).double()
    if dtype != F32:
        q, k, v, first, gate = (t.to(dtype).double() for t in (q, k, v, first, gate))
    for i, j in spikes:
        kj = k[j].view(1, G, D).repeat_interleave(H // G, dim=1)
        q[i] = oracle.rotate_halves(kj, torch.tensor([j - i]), rot["base"], rot["dims"]).reshape(-1)
    lam = 0.35
    vm = oracle.mix_values(v, first, lam) if blend else v
    want = oracle.block_attend(oracle.unit_heads(q, H, L, EPS), oracle.unit_heads(k, G, L, EPS),
                               vm.view(T, G, Dv), L["scale"], L["mask"]["size"], gate)
    att = ChunkedRotaryAttention(H, G, D, Dv, L["scale"], EPS, chunk=L["mask"]["size"], rot=rot,
                                 mixes_values=blend)
    if blend:
        att.v_lambda.data.fill_(lam)
    att = att.to(device)
    nblk = (T + page - 1) // page
    mgr = BlockKVCacheManager(1, 1, 1, num_blocks=nblk + 2, block_size=page, dtype=dtype,
                              tp_degree=1, layer_kv_shapes=[att.kv_shape()]).to(device)
    mgr.k_caches[0].data.normal_()                      # stale pages
    mgr.v_caches[0].data.normal_()
    bt = torch.randperm(nblk + 2)[:nblk].view(1, nblk).to(device)
    got, at = [], 0
    for n in cuts or [T]:
        pos = torch.arange(at, at + n).view(1, n).to(device)
        mgr.set_step_context(bt, generate_slot_mapping(bt, pos, page))
        st = seqmix.StepLayout(pos, torch.zeros(1, dtype=torch.long, device=device))
        part = [t[at:at + n].view(1, n, -1).to(device, dtype) for t in (q, k, v, gate, first)]
        got.append(att(*part[:3], mgr, 0, st, gate=part[3],
                       v_first=part[4] if blend else None)[0].float().cpu())
        at += n
    got = torch.cat(got)
    if dtype == F32:
        close(got, want, tol)
    else:
        assert (got.double() - want).std().item() < tol * want.std().item()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("L", [att_cfg(size=10, scale=1.5), att_cfg(4, 4, 6, 6, size=10, dims=6),
                               att_cfg(5, 1, 10, 3, size=10, dims=2, base=5.0, scale=1.1)])
def test_chunked_attention_in_portions(device, L):
    # a block's first key, the last key of the block before (unseen), queries that
    # open or end a block, page borders inside blocks, the first token
    spikes = [(9, 0), (19, 10), (20, 19), (21, 19), (10, 9), (25, 20), (28, 23), (15, 9), (30, 30)]
    _attention_alone(device, L, 33, spikes=spikes)
    _attention_alone(device, L, 33, spikes=spikes, cuts=[1, 2, 7, 1, 1, 1, 20])
    _attention_alone(device, L, 33, spikes=spikes, cuts=[3] + [1] * 30, page=8)
    _attention_alone(device, L, 33, spikes=spikes, cuts=[2] * 16 + [1])
    _attention_alone(device, L, 33, spikes=spikes, cuts=[10, 10, 11, 2], blend=False)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size", [1, 2, 4, 7, 500, 0])
def test_block_sizes_from_one_to_longer_than_the_sequence(device, size):
    L = att_cfg(2, 1, 8, 4, size=size, scale=1.2)
    for cuts in (None, [5, 2, 1, 1, 1, 12], [1] * 22):
        _attention_alone(device, L, 22, cuts=cuts,
                         spikes=[(21, 0), (14, 13), (8, 7), (7, 4), (3, 2), (20, 15)])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [None, [250] + [1] * 30, [100, 100, 60, 20]])
def test_attention_far_key_among_hundreds(device, cuts):
    """Blocks of 140: keys of one's own block more than a hundred positions
    back decide, the neighbouring block's do not."""
    L = att_cfg(2, 1, 12, 6, size=140, scale=1.4, base=10000.0, dims=8)
    _attention_alone(device, L, 280, cuts=cuts, page=16, tol=2e-4,
                     spikes=[(279, 140), (278, 139), (270, 144), (139, 0), (140, 139), (265, 159),
                             (266, 160), (100, 1)])


@pytest.mark.gpu
@pytest.mark.parametrize("L,cuts", [
    (att_cfg(4, 2, 32, 32, size=50, scale=0.5, dims=32), None),
    (att_cfg(6, 2, 24, 40, size=64, scale=0.5, dims=16), [3, 60, 1, 66]),
    (att_cfg(8, 8, 64, 64, size=100, scale=0.25, dims=32), [64, 66]),
    (att_cfg(8, 2, 128, 128, size=120, scale=0.2, dims=128), [70, 50] + [1] * 10),
    (att_cfg(3, 1, 12, 10, size=33, scale=0.8, dims=4), [100, 29, 1]),             # vector kernel
])
def test_attention_bf16_matrix_path_gpu(L, cuts):
    spikes = [(129, 128), (129, 100), (110, 101), (99, 50), (128, 127), (60, 51), (49, 0)]
    _attention_alone("cuda", L, 130, spikes=spikes, cuts=cuts, page=16, dtype=BF16, tol=0.03)


# ------------------------------------------------------------ matrix memory
def _memory_alone(device, H, D, Dv, T, cuts, cap=4.0, dtype=F32, tol=3e-5, ib=0.0, fb=2.0,
                  gain=2.0, rows=1):
    """The recurrence with its gates and read-out from given projections,
    carried over ``cuts``; other state slots are left alone."""
    torch.manual_seed(12)
    q, k = torch.randn(rows, T, H * D), torch.randn(rows, T, H * D)
    v, gate = torch.randn(rows, T, H * Dv), torch.randn(rows, T, H * Dv)
    zi, zf = torch.randn(rows, T, H) * gain, torch.randn(rows, T, H) * gain
    bi, bf = torch.randn(H) + ib, torch.randn(H) + fb
    nw = 1 + 0.3 * torch.randn(H * Dv)
    if dtype != F32:
        q, k, v, gate, zi, zf = (t.to(dtype).float() for t in (q, k, v, gate, zi, zf))
    want, ends = [], []
    for b in range(rows):
        i, f = oracle.mlstm_gates(zi[b].double() + bi, zf[b].double() + bf, cap)
        o, end = oracle.mlstm_scan(q[b].double().view(T, H, D) * D ** -0.5,
                                   k[b].double().view(T, H, D), v[b].double().view(T, H, Dv), i, f)
        want.append(oracle.rms(o, EPS).reshape(T, H * Dv) * nw.double()
                    * torch.sigmoid(gate[b].double()))
        ends.append(end)
    want = torch.stack(want)
    m = ExponentialGateMemory(H, D, Dv, cap, EPS)
    m.i_bias.data, m.f_bias.data, m.norm_weight.data = bi, bf, nw
    m = m.to(device)
    states = RecurrentStateManager(rows + 2)
    for name, shape in m.state_shapes().items():
        states.register("x." + name, shape)
    states = states.to(device)
    for t in states.tensors.values():
        t.data.normal_()                                 # stale state
    keep = {n: t.data[:2].clone() for n, t in states.tensors.items()}
    # column slices of one wide row, as the fused projection leaves them
    splits = [H * D, H * D, H * Dv, H * Dv, H, H]
    wide = torch.cat([q, k, v, gate, zi, zf, torch.zeros(rows, T, -sum(splits) % 8)], dim=-1)
    got, at = [], 0
    for n in cuts:
        st = step_of(torch.arange(at, at + n).view(1, n).expand(rows, n),
                     torch.arange(2, 2 + rows), device)
        parts = torch.split(wide[:, at:at + n].to(device, dtype), splits + [-sum(splits) % 8], -1)
        got.append(m(*parts[:6], states, "x", st).float().cpu())
        at += n
    assert at == T
    for n, t in states.tensors.items():
        assert torch.equal(t.data[:2], keep[n])
    got = torch.cat(got, dim=1)
    if dtype == F32:
        # a read-out whose products cancel magnifies their rounding: few, and not by much
        close(got, want, 100 * tol, 10 * tol)
        assert (got.double() - want).std().item() < tol
    else:                                                # one rounding of the result
        close(got, want, 4e-3, 6e-3)
    mem, mx = states.get("x.mem")[2:].cpu(), states.get("x.max")[2:].cpu()
    for b, (S, nv, mm) in enumerate(ends):               # carried for the next step, exact
        close(mem[b, :, :Dv].transpose(-1, -2) / D ** -0.5, S, tol * max(S.abs().max().item(), 1.0))
        close(mem[b, :, Dv] / D ** -0.5, nv, tol * max(nv.abs().max().item(), 1.0))
        close(mx[b], mm, tol * 10)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,Dv,cap", [(3, 5, 8, 4.0), (1, 12, 20, 15.0), (2, 33, 3, 1.0),
                                        (2, 64, 17, 8.0), (1, 1, 1, 2.0), (4, 16, 16, 0.5)])
def test_matrix_memory_in_portions(device, H, D, Dv, cap):
    for cuts in ([40], [1] * 40, [2, 15, 1, 16, 6], [2] * 20, [17, 2, 21]):
        _memory_alone(device, H, D, Dv, 40, cuts, cap)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cap,ib,fb,gain", [
    (15.0, 0.0, 8.0, 1.0),        # nothing is forgotten: the maximum keeps an early peak
    (15.0, 0.0, -8.0, 1.0),       # everything is: the memory is the last token
    (15.0, -12.0, 8.0, 0.5),      # tiny inputs: the denominator's floor exp(-m) rules, m from zero
    (60.0, 20.0, 0.0, 20.0),      # gates that swing over tens of orders of magnitude
    (0.3, 5.0, -5.0, 9.0)])       # gates at their caps
def test_matrix_memory_gate_extremes(device, cap, ib, fb, gain):
    kw = dict(cap=cap, ib=ib, fb=fb, gain=gain)
    _memory_alone(device, 2, 16, 8, 90, [90], **kw)
    _memory_alone(device, 2, 16, 8, 90, [50, 2, 1, 37], **kw)
    _memory_alone(device, 2, 16, 8, 90, [3] + [1] * 87, **kw)


@pytest.mark.parametrize("device", DEVICES)
def test_the_running_maximum_starts_at_zero(device):
    """One token with a very small input gate: with m from zero the floor of
    the denominator is one and the read-out is (nearly) nothing next to eps."""
    m = ExponentialGateMemory(1, 4, 4, 15.0, 1e-2).to(device)
    st = RecurrentStateManager(1)
    for name, shape in m.state_shapes().items():
        st.register("x." + name, shape)
    st = st.to(device)
    one = torch.ones(1, 1, 4, device=device)
    z = torch.full((1, 1, 1), -7.0, device=device)
    out = m(one, one, one, one * 50, z, torch.zeros_like(z), st, "x", step_of([[0]], [0], device))
    i, f = oracle.mlstm_gates(torch.full((1, 1), -7.0).double(), torch.zeros(1, 1).double(), 15.0)
    o, (_, _, mx) = oracle.mlstm_scan(torch.ones(1, 1, 4).double() / 2, torch.ones(1, 1, 4).double(),
                                      torch.ones(1, 1, 4).double(), i, f)
    close(out.cpu()[0], oracle.rms(o, 1e-2).view(1, 4), 1e-6)
    assert out.abs().max() < 0.1
    close(st.get("x.max").cpu()[0], mx, 1e-6)
    assert abs(mx.item() + 0.6931) < 1e-3                # f of the first token, not its i


@pytest.mark.parametrize("device,dtype", [
    ("cpu", F32), pytest.param("cuda", F32, marks=pytest.mark.gpu),
    pytest.param("cuda", BF16, marks=pytest.mark.gpu)])
def test_the_denominators_constant(device, dtype):
    """Large gates (exp(-m) far below 1e-6) and a query orthogonal to the
    normalizer: the constant 1e-6 is what divides, and with values this small
    next to the norm's eps it shows. The first two tokens write, the rest read."""
    H, D, Dv, T, eps, cap = 1, 8, 16, 128, 1e-4, 16.0
    torch.manual_seed(14)
    k = torch.zeros(T, D)
    k[0, 0] = k[1, 1] = 1.0
    q = torch.zeros(T, D)
    q[:, 0], q[:, 1] = 1.0, -1.0
    v = (torch.randn(T, Dv) * 3e-8).to(dtype).float()
    z = torch.full((T, H), 64.0)
    i, f = oracle.mlstm_gates(z.double(), z.double(), cap)
    o, (_, _, m) = oracle.mlstm_scan(q.double().view(T, H, D) * D ** -0.5, k.double().view(T, H, D),
                                     v.double().view(T, H, Dv), i, f)
    assert torch.exp(-m).item() < 2e-7
    want = oracle.rms(o, eps).view(T, Dv) * 0.5
    for cuts in ([T], [64, 62, 1, 1], [2] * 3 + [T - 6], [1] * 6 + [T - 6]):
        mem, mx = torch.zeros(1, H, Dv + 1, D, device=device), torch.zeros(1, H, device=device)
        got, at = [], 0
        zero, one = torch.zeros(H, device=device), torch.ones(H * Dv, device=device)
        for n in cuts:
            st = step_of(torch.arange(at, at + n).view(1, n), [0], device)
            part = [t[None, at:at + n].to(device, dtype) for t in (q, k, v, z, z, torch.zeros(T, Dv))]
            got.append(seqmix.mlstm(*part, zero, zero, cap, one, eps, mem, mx, st, D, Dv)[0].cpu())
            at += n
        assert want[1:].abs().mean() > 0.05
        close(torch.cat(got), want, 2e-3, 0.05)


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,Dv,T,cuts", [
    (2, 64, 48, 300, [300]), (3, 128, 128, 700, [700]), (2, 32, 64, 520, [257, 1, 262]),
    (1, 256, 40, 530, [530]), (2, 20, 24, 400, [398, 2]), (4, 128, 64, 193, [97, 96]),
    (2, 96, 80, 333, [64, 128, 141]), (2, 8, 8, 230, [113, 117]), (3, 40, 104, 200, [100, 100]),
    (1, 72, 72, 1100, [1100]), (2, 64, 136, 150, [150]), (2, 16, 128, 129, [64, 65]),
    (1, 24, 16, 4300, [4300])])
def test_matrix_memory_long_rows_gpu(H, D, Dv, T, cuts):
    """Rows that are scanned in segments side by side or, in bf16, in chunks on
    the matrix cores; memory that reaches across all of them, gates that swing;
    the state is exact either way."""
    for dtype in (F32, BF16):
        _memory_alone("cuda", H, D, Dv, T, cuts, 15.0, fb=7.0, gain=1.0, dtype=dtype)
        if T < 1000:
            _memory_alone("cuda", H, D, Dv, T, cuts, 6.0, gain=4.0, dtype=dtype)
            _memory_alone("cuda", H, D, Dv, T, cuts, 30.0, fb=0.0, ib=-3.0, gain=15.0, dtype=dtype)
    if T < 1000:
        _memory_alone("cuda", H, D, Dv, T, cuts, 15.0, fb=4.0, dtype=BF16, rows=3)


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,Dv", [(3, 128, 128), (2, 64, 40), (1, 256, 300), (2, 6, 9), (5, 30, 64)])
def test_matrix_memory_decoding_gpu(H, D, Dv):
    """Single-token steps (one launch) behind a prompt and from the start."""
    for dtype in (F32, BF16):
        _memory_alone("cuda", H, D, Dv, 90, [70] + [1] * 20, 15.0, fb=6.0, dtype=dtype, rows=2)
        _memory_alone("cuda", H, D, Dv, 30, [1] * 30, 5.0, gain=4.0, dtype=dtype)


@pytest.mark.parametrize("device,lens,chunked", [
    ("cpu", [9, 1, 0, 70], False),
    pytest.param("cuda", [9, 1, 0, 70], False, marks=pytest.mark.gpu),
    pytest.param("cuda", [64, 1, 0, 130], True, marks=pytest.mark.gpu),   # bf16, matrix cores
    pytest.param("cuda", [1, 1, 0, 1], False, marks=pytest.mark.gpu)])    # single-token form
def test_memory_of_unequal_rows_and_pads(device, lens, chunked):
    torch.manual_seed(13)
    H, D, Dv = (2, 16, 24) if chunked else (2, 6, 5)
    S, cap, dt = max(lens), 5.0, BF16 if chunked else F32
    shape = {"q": D, "k": D, "v": Dv, "g": Dv, "i": 1, "f": 1}
    x = {n: torch.randn(4, S, H * c).to(dt) for n, c in shape.items()}
    pos = torch.full((4, S), -1)
    for b, n in enumerate(lens):
        pos[b, :n] = torch.arange(n)
    mem, mx = torch.randn(4, H, Dv + 1, D, device=device), torch.randn(4, H, device=device)
    keep = mem[3].clone(), mx[3].clone()
    zero, nw = torch.zeros(H, device=device), torch.ones(H * Dv, device=device)
    got = seqmix.mlstm(*(x[n].to(device) for n in ("q", "k", "v", "i", "f", "g")), zero, zero, cap,
                       nw, EPS, mem, mx, step_of(pos, [2, 0, -1, 1], device), D, Dv).float().cpu()
    for b, n in enumerate(lens):
        if not n:
            continue
        r = {k: t[b, :n].double() for k, t in x.items()}
        o, end = oracle.mlstm_scan(r["q"].view(n, H, D) * D ** -0.5, r["k"].view(n, H, D),
                                   r["v"].view(n, H, Dv), *oracle.mlstm_gates(r["i"], r["f"], cap))
        want = oracle.rms(o, EPS).reshape(n, H * Dv) * torch.sigmoid(r["g"])
        close(got[b, :n], want, *((4e-3, 6e-3) if chunked else (2e-4, 0.0)))
        close(mx[[2, 0, -1, 1][b]].cpu(), end[2], 1e-4)
    assert torch.equal(mem[3], keep[0]) and torch.equal(mx[3], keep[1])


# ------------------------------------------------------------ router, experts
def _dense(picks, T, E):
    want = torch.zeros(T, E, dtype=torch.float64)
    for t, row in enumerate(picks):
        for e, w in row:
            want[t, e] = w
    return want


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T,W,E,top,count,keep", [
    (5, 24, 8, 2, 4, 2), (64, 64, 16, 4, 4, 1), (9, 136, 3, 3, 1, 1), (6, 10, 1, 1, 1, 1),
    (33, 20, 6, 3, 6, 4),                                # groups of one expert
    (7, 32, 130, 5, 2, 1), (600, 32, 9, 3, 3, 2)])       # many experts; many tokens
def test_sigmoid_router_with_groups_and_correction(device, T, W, E, top, count, keep):
    """Choice (groups too) by the corrected score, which may be negative;
    weights from the scores as they are, renormalised, times the scale."""
    torch.manual_seed(18)
    w, corr = torch.randn(E, W) * 0.4, torch.randn(E) - 1.0
    x = torch.randn(T, W)
    rc = {"experts": E, "top": top, "scale": 2.2, "groups": {"count": count, "keep": keep}}
    want = _dense(oracle.route(x.double() @ w.double().T, corr.double(), rc), T, E)
    dense_w, idx, wts = seqmix.route_tokens(
        x.to(device), w.to(device), E, top, count, keep, 2.2, True, correction=corr.to(device),
        score="sigmoid", group_top=2, norm_eps=1e-20)
    close(dense_w.cpu(), want, 1e-5)
    close(wts.sum(-1).cpu(), torch.full((T,), 2.2), 1e-5)
    assert (torch.gather(dense_w, 1, idx.long()) - wts).abs().max() == 0
    if E > top:
        plain = _dense(oracle.route(x.double() @ w.double().T, torch.zeros(E).double(), rc), T, E)
        assert ((plain > 0) != (want > 0)).any()


@pytest.mark.parametrize("device", DEVICES)
def test_a_group_scores_as_its_two_best_and_sums_stay_finite(device):
    """The group with the single best expert loses against one with two good
    ones; scores so small that the sum is next to nothing are divided by the
    sum plus 1e-20."""
    E = 6
    logit = torch.tensor([[2.0, -4.0, -4.0, 1.0, 1.0, -9.0],
                          [-48.0, -90.0, -90.0, -47.0, -47.5, -90.0]])
    rc = {"experts": E, "top": 2, "scale": 1.0, "groups": {"count": 2, "keep": 1}}
    want = _dense(oracle.route(logit.double(), torch.zeros(E).double(), rc), 2, E)
    assert (want[0] > 0).tolist() == [False, False, False, True, True, False]
    assert want[1].sum() < 0.9
    for route in ("fused", "split"):
        if route == "fused":
            got = seqmix.route_tokens(logit.to(device), torch.eye(E, device=device), E, 2, 2, 1, 1.0,
                                      True, score="sigmoid", group_top=2, norm_eps=1e-20)[0]
        else:
            got = seqmix.group_limited_router(logit.to(device), E, 2, 2, 1, 1.0, True,
                                              score="sigmoid", group_top=2, norm_eps=1e-20)[0]
        close(got.cpu(), want, 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("E,ff,rest", [(3, 5, 7), (4, 8, 16), (2, 16, 0), (1, 8, 8)])
def test_silu_units_times_routing_weight(device, dtype, E, ff, rest):
    torch.manual_seed(17)
    T, C = 9, E * ff + rest
    hid = (torch.randn(T, 2 * C) * 2).to(dtype)
    gates = torch.rand(T, E)
    gates[:, 0] = 0.0
    got = seqmix.silu_glu_scale(hid.to(device), gates.to(device), ff, E).cpu()
    full = torch.cat([gates, torch.ones(T, 1)], dim=1).double()
    g, u = hid.double()[:, :C], hid.double()[:, C:]
    want = g * torch.sigmoid(g) * u * full[:, (torch.arange(C) // ff).clamp(max=E)]
    close(got, want, *((2e-5, 0.0) if dtype == F32 else (1e-3, 0.005)))
    assert (got[:, :ff] == 0).all()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("fc", [moe(), moe(3, 3, ff=6, shared_ff=0, count=1, keep=1),
                                moe(1, 1, ff=10, shared_ff=4, count=1, keep=1),
                                moe(8, 2, ff=16, shared_ff=24, count=2, keep=1, scale=0.5)])
def test_feed_forward_alone(device, fc, T=19, Wd=16):
    torch.manual_seed(6)
    W = make_weights(model_cfg(layers=[layer("mlstm", mem_cfg(), fc)], width=Wd), seed=6)
    h = torch.randn(T, Wd)
    p = "l0.mlp."
    want = oracle.moe_ff(h.double(), W, p, fc)
    rc, sh = fc["router"], bool(fc.get("shared"))
    E = rc["experts"]
    m = GroupRoutedFeedForward(Wd, E, rc["top"], fc["expert"]["ff"], F32,
                               n_groups=rc["groups"]["count"], keep_groups=rc["groups"]["keep"],
                               scale=rc["scale"], normalize=True,
                               shared_ff=fc["shared"]["ff"] if sh else 0, shared_gate=False,
                               act="silu_glu", router=ROUTER)
    m.router.weight.data, m.router.correction.data = W[p + "router"], W[p + "correction"]
    m.experts.gate_up.weight.data = FusedGatedExperts.stack_gate_up(
        [W[p + f"e{e}.gate"] for e in range(E)], [W[p + f"e{e}.up"] for e in range(E)],
        W[p + "shared.gate"] if sh else None, W[p + "shared.up"] if sh else None)
    m.experts.down.weight.data = FusedGatedExperts.stack_down(
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
def test_long_decoding_across_many_blocks_and_pages(device):
    cfg = model_cfg()
    W = make_weights(cfg, seed=21)
    toks = tokens_for(cfg, 90, seed=22)
    eng = make_engine(cfg, W, device, pages=30, max_len=96)
    close(feed(eng, toks, [3] + [1] * 87), oracle.forward(cfg, W, toks), 3e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_a_far_token_decides_through_each_mechanism(device):
    """Changing only the FIRST token of a sequence moves the last logits, as
    much as the oracle says: through a state that forgets little, or through
    a key of the same block; with the block one shorter it does not at all."""
    def run(cfg, W, T, moves):
        toks = tokens_for(cfg, T, seed=34)
        other = [(toks[0] + 11) % cfg["vocab"]] + toks[1:]
        a, b = oracle.forward(cfg, W, toks), oracle.forward(cfg, W, other)
        assert ((a[-1] - b[-1]).abs().max() > 3e-3) == moves
        eng = make_engine(cfg, W, device, pages=24, max_len=96)
        for cuts in ([T], [T - 20, 2] + [1] * 18):
            close(feed(eng, toks, cuts)[-1], a[-1], 3e-4)
            close(feed(eng, other, cuts)[-1], b[-1], 3e-4)

    cfg = model_cfg(layers=[layer("mlstm", mem_cfg(2, 8, 8, gate_cap=15.0), None)])
    W = make_weights(cfg, seed=33)
    W["l0.mix.f.b"] += 8.0
    run(cfg, W, 80, True)
    for size, moves in ((80, True), (79, False)):
        cfg = model_cfg(layers=[layer("attention", att_cfg(2, 1, 8, 6, size=size, scale=0.3), None)])
        run(cfg, make_weights(cfg, seed=35), 80, moves)


@pytest.mark.parametrize("device", DEVICES)
def test_first_layers_values_reach_the_later_ones(device):
    """lambda of one replaces a layer's own values altogether; of the first
    value-mixing layer it changes nothing."""
    L = att_cfg(4, 2, 6, 5, size=9)
    cfg = model_cfg(layers=[layer("mlstm", mem_cfg(), None), layer("attention", L, None),
                            layer("attention", dict(L, v_mix=False), None),
                            layer("attention", L, None)])
    W = make_weights(cfg, seed=40)
    toks = tokens_for(cfg, 21, seed=41)
    W["l3.mix.vmix"] = torch.tensor(1.0)
    want = oracle.forward(cfg, W, toks)
    close(feed(make_engine(cfg, W, device), toks, [9, 2, 1, 9]), want, 3e-4)
    for name, same in (("l1.mix.vmix", True), ("l2.mix.vmix", True), ("l3.mix.v", True),
                       ("l1.mix.v", False)):
        W2 = dict(W)
        W2[name] = W[name] + 1.5
        got = feed(make_engine(cfg, W2, device), toks, [9, 2, 1, 9])
        close(got, oracle.forward(cfg, W2, toks), 3e-4)
        assert ((got - want.float()).abs().max() < 1e-3) == same, name


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("make", [model_cfg, varied_cfg])
def test_residual_stream_per_layer(device, make):
    cfg = make()
    W = make_weights(cfg, seed=7)
    toks = tokens_for(cfg, 9, seed=8)
    sums = []
    oracle.forward(cfg, W, toks, sums)
    eng = make_engine(cfg, W, device)
    seen = []
    hooks = [l.register_forward_hook(lambda m, a, out: seen.append(out.detach().clone().cpu()))
             for l in eng.model.model.layers]
    feed(eng, toks, [9])
    for hk in hooks:
        hk.remove()
    assert len(seen) == len(sums) == len(cfg["layers"])
    for r, s in enumerate(seen):                     # the last layer leaves the sum itself
        assert (s.dim() == 3) == (r == len(seen) - 1)
        close(s[0] if s.dim() == 3 else s[0].sum(1), sums[r], 4e-5 * sums[r].abs().max().item())


def test_attention_holds_pages_and_memory_holds_state():
    cfg = varied_cfg()
    eng = make_engine(cfg, make_weights(cfg, seed=16))
    mgr = eng.kv_mgr
    for i, lc in enumerate(cfg["layers"]):
        assert (mgr.k_caches[i].numel() > 0) == (lc["type"] == "attention")
        assert (mgr.v_caches[i].numel() > 0) == (lc["type"] == "attention")
    assert set(mgr.state.tensors.keys()) == {"run0_mem", "run0_max", "run3_mem", "run3_max"}
    assert all(t.dtype == F32 for t in mgr.state.tensors.values())
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
    for t in list(eng.kv_mgr.k_caches) + list(eng.kv_mgr.v_caches) + \
            list(eng.kv_mgr.state.tensors.values()):
        t.data.normal_()
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
    replayed many times beside eager prefills; the recurrent state survives
    the capture's warm-up runs."""
    cfg = model_cfg()
    W = make_weights(cfg, seed=11)
    prompts = [tokens_for(cfg, n, seed=20 + n) for n in (9, 5, 14, 6)]
    want = [_oracle_greedy(cfg, W, p, 12) for p in prompts]
    eng = make_engine(cfg, W, "cuda", slots=2, page=4, pages=14, max_len=28,
                      capture_decode=True, async_depth=2)
    rids = [eng.add_request(torch.tensor(p), max_new_tokens=12) for p in prompts]
    out = eng.run()
    assert [out[r] for r in rids] == want


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


@pytest.mark.gpu
def test_bfloat16_serving_precision_gpu():
    """bf16 projections, fp32 streams/scores/norms/router/recurrence: close to
    the oracle and independent of how the prompt is cut, beyond rounding."""
    att = dict(heads=8, kv_heads=2, dim=32, vdim=40, size=45, dims=16, scale=0.2)
    ff = moe(6, 6, ff=64, shared_ff=48, count=1, keep=1)
    cfg = model_cfg(layers=[
        layer("attention", att_cfg(**att), ff),
        layer("mlstm", mem_cfg(4, 32, 48, gate_cap=15.0), ff),
        layer("attention", att_cfg(**att), ff),
        layer("mlstm", mem_cfg(4, 32, 48, gate_cap=15.0), None),
    ], width=128, vocab=96, streams=4)
    W = make_weights(cfg, seed=12)
    toks = tokens_for(cfg, 160, seed=13)
    want = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, "cuda", dtype="bfloat16", page=16, pages=12, max_len=192)
    a = feed(eng, toks, [160])
    b = feed(eng, toks, [7, 80, 2, 1, 1, 69])
    scale = want.std().item()
    assert (a.double() - want).std().item() < 0.04 * scale
    assert (b.double() - want).std().item() < 0.04 * scale
    assert (a - b).double().std().item() < 0.04 * scale


@pytest.mark.gpu
def test_float32_kernels_at_larger_sizes_gpu():
    cfg = model_cfg(layers=[
        layer("mlstm", mem_cfg(5, 64, 72, gate_cap=12.0), moe(8, 3, ff=32, shared_ff=48, count=4,
                                                              keep=2)),
        layer("attention", att_cfg(6, 3, 48, 40, size=150, dims=32, base=10000.0, scale=0.3),
              moe(8, 3, ff=40, shared_ff=0, count=2, keep=1)),
        layer("attention", att_cfg(6, 3, 40, 40, size=99, dims=40, base=10000.0, scale=0.3), None),
    ], width=160, vocab=101, streams=3)
    W = make_weights(cfg, seed=30)
    toks = tokens_for(cfg, 310, seed=31)
    want = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, "cuda", page=16, pages=24, max_len=320, slots=2)
    close(feed(eng, toks, [310]), want, 5e-4)
    close(feed(eng, toks, [100, 7, 2, 160] + [1] * 41), want, 5e-4)


# ------------------------------------------------------------ checkpoint, CLI, config
def _write_checkpoint(path, cfg, W):
    from safetensors.torch import save_file

    path.mkdir()
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.bfloat16().contiguous() for k, v in W.items()}, str(path / "model.safetensors"))


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
    _write_checkpoint(mdir, cfg, W)
    disk = copy.deepcopy(cfg)
    del disk["vocab"], disk["width"], disk["streams"], disk["logit_softcap"]
    for lc in disk["layers"]:
        mc, fc = lc["mixer"], lc["mlp"]
        for key in ("heads", "dim", "vdim") + (("kv_heads",) if lc["type"] == "attention" else ()):
            del mc[key]
        if fc:
            del fc["expert"]["ff"], fc["router"]["experts"]
            if fc.get("shared"):
                del fc["shared"]["ff"]
    (mdir / "config.json").write_text(json.dumps(disk))
    assert model_type_from_config(str(mdir)) == "sitidra"
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
    wa, wb = (oracle.forward(cfg, W, t) for t in (a, b))
    g = [torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
         for i in range(3)]
    close(g[0], wa[[0, 7]], 3e-4)
    close(g[1], wb[[0]], 3e-4)
    close(g[2], torch.stack([wb[8], wa[20]]), 3e-4)


def test_command_line_generation(tmp_path, capsys):
    """inference_demo --model-type sitidra: checkpoint folder -> compile ->
    load -> greedy generation, the same path as every other family."""
    from neuronx_distributed_inference_amd.inference_demo import main

    cfg = model_cfg()
    W = make_weights(cfg, seed=3)
    mdir = tmp_path / "model"
    _write_checkpoint(mdir, cfg, W)
    prompt = tokens_for(cfg, 9, seed=1)
    rc = main(["--model-type", "sitidra", "run", "--model-path", str(mdir),
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
                   lambda c: c["layers"][0]["mlp"].update(kind="dense"),
                   lambda c: c["layers"][0]["mixer"].update(kv_heads=4),       # 6 heads
                   lambda c: c["layers"][2]["mixer"].update(vdim=9),           # not the first's
                   lambda c: c["layers"][1]["mlp"]["router"].update(top=5),    # 2 groups of 2 stay
                   lambda c: c["layers"][1]["mlp"]["router"].update(experts=7),
                   lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=4),
                   lambda c: c.update(streams=0)):
        bad = copy.deepcopy(cfg)
        change(bad)
        with pytest.raises(ValueError):
            SitidraInferenceConfig(neuron_config=EngineConfig(tp_degree=1), **bad)
