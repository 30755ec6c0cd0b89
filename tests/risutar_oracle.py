"""Plain, slow, whole-sequence Risutar in float64, one function per mechanism,
written from the equations. Shares no code with the package: it is the
yardstick the engine, its cache and state handling and its kernels are
compared with.

A model is ``(cfg, weights)``: ``cfg`` the checkpoint's config dictionary,
``weights`` a dict of tensors under the checkpoint's names. Every function
takes the full token sequence of ONE request; nothing is cached, recurrences
start from zero and walk token by token.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def _w(weights, name):
    return weights[name].to(F64)


# ------------------------------------------------------------------- norms
def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, b, eps):
    mean = x.mean(-1, keepdim=True)
    dev = x - mean
    return dev / torch.sqrt((dev * dev).mean(-1, keepdim=True) + eps) * w + b


def post_norm(x, y, alpha, w, b, eps):
    """The residual step: the norm follows the sum."""
    return layer_norm(alpha * x + y, w, b, eps)


# -------------------------------------------------------------- embeddings
def bigram_rows(tokens, bg):
    """Row of the bigram table for every token of a sequence."""
    rows = []
    for t, tok in enumerate(tokens):
        if t == 0:
            rows.append(bg["buckets"])
        else:
            rows.append((int(tokens[t - 1]) * bg["mul_prev"] + int(tok) * bg["mul_cur"])
                        % bg["buckets"])
    return rows


def embed(tokens, weights, bg):
    tokens = [int(t) for t in tokens]
    return _w(weights, "embed")[tokens] + _w(weights, "bigram")[bigram_rows(tokens, bg)]


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def token_side(x, tokens, weights, i, dim, eps):
    """x plus layer i's share of the per-layer token input."""
    tokens = [int(t) for t in tokens]
    e = _w(weights, "side.embed")[tokens][:, i * dim:(i + 1) * dim]
    p = f"l{i}.side."
    g = gelu_tanh(x @ _w(weights, p + "gate").T) * e
    y = g @ _w(weights, p + "proj").T
    return x + rms(y, eps) * _w(weights, p + "norm")


# ---------------------------------------------------------- latent attention
def rotate_halves(x, positions, base, dims):
    """x (T, N, C): channel i < dims/2 and channel i + dims/2 turn together
    by the angle p * base^(-2i/dims); channels from ``dims`` on pass."""
    out = x.clone()
    p = positions.to(F64).view(-1, 1)
    half = dims // 2
    for i in range(half):
        a = p * float(base) ** (-2.0 * i / dims)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def latent_rows(dkv, norm_w, mc, eps):
    """What a latent layer's cache holds for every token: (normed latent c
    (T, kv_rank), rotated shared key part (T, rot_dim)) from the
    down-projection dkv (T, kv_rank + rot_dim)."""
    C, R = mc["kv_rank"], mc["rot_dim"]
    c = rms(dkv[:, :C], eps) * norm_w
    pos = torch.arange(dkv.shape[0])
    kr = rotate_halves(dkv[:, C:].reshape(-1, 1, R), pos, mc["rot"]["base"], mc["rot"]["dims"])
    return c, kr[:, 0]


def latent_attend(q, c, k_rot, uk, uv, mc, head_gate=None):
    """Causal softmax attention over latent rows. q (T, H * (dim + rot_dim))
    after the query up-projection; head_gate (T, H) logits or None. Returns
    the concatenated heads."""
    T = q.shape[0]
    H, D, R, Dv = mc["heads"], mc["dim"], mc["rot_dim"], mc["vdim"]
    q = q.view(T, H, D + R)
    pos = torch.arange(T)
    q_rot = rotate_halves(q[..., D:], pos, mc["rot"]["base"], mc["rot"]["dims"])
    k_plain = (c @ uk.T).view(T, H, D)
    v = (c @ uv.T).view(T, H, Dv)
    future = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = torch.zeros(T, H, Dv, dtype=F64)
    for hd in range(H):
        s = (q[:, hd, :D] @ k_plain[:, hd].T + q_rot[:, hd] @ k_rot.T) * mc["scale"]
        p = torch.softmax(s.masked_fill(future, float("-inf")), dim=-1)
        out[:, hd] = p @ v[:, hd]
    if head_gate is not None:
        out = out * torch.sigmoid(head_gate).view(T, H, 1)
    return out.reshape(T, H * Dv)


def latent_mixer(h, weights, pre, mc, eps, rows):
    """h (T, W); ``rows`` = latent_rows of the layer whose cache is read."""
    cq = rms(h @ _w(weights, pre + "dq").T, eps) * _w(weights, pre + "dq.norm")
    q = cq @ _w(weights, pre + "uq").T
    gate = h @ _w(weights, pre + "g").T
    heads = latent_attend(q, rows[0], rows[1], _w(weights, pre + "uk"), _w(weights, pre + "uv"),
                          mc, gate)
    return heads @ _w(weights, pre + "o").T


# ------------------------------------------------------ gated linear attention
def gla_decay(z, tau):
    """Per-channel decay from its logits."""
    return torch.sigmoid(z) ** (1.0 / tau)


def gla_scan(q, k, v, decay):
    """q, k, decay (T, H, D), v (T, H, Dv) -> o (T, H, Dv), final state."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for t in range(T):
        S = decay[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out, S


def gla_mixer(h, weights, pre, mc, eps):
    T = h.shape[0]
    H, D, Dv = mc["heads"], mc["dim"], mc["vdim"]
    q = (h @ _w(weights, pre + "q").T).view(T, H, D) * D ** -0.5
    k = (h @ _w(weights, pre + "k").T).view(T, H, D)
    v = (h @ _w(weights, pre + "v").T).view(T, H, Dv)
    z = (h @ _w(weights, pre + "a1").T) @ _w(weights, pre + "a2").T + _w(weights, pre + "a2.b")
    o, _ = gla_scan(q, k, v, gla_decay(z.view(T, H, D), mc["tau"]))
    o = (rms(o, eps) * _w(weights, pre + "norm")).reshape(T, H * Dv)
    g = h @ _w(weights, pre + "g").T
    return (o * g * torch.sigmoid(g)) @ _w(weights, pre + "o").T


# --------------------------------------------------------------- feed-forward
def dense_ff(h, weights, pre):
    g = h @ _w(weights, pre + "gate").T
    return (g * torch.sigmoid(g) * (h @ _w(weights, pre + "up").T)) @ _w(weights, pre + "down").T


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def expert(h, weights, pre):
    return gelu_erf(h @ _w(weights, pre + "up").T) @ _w(weights, pre + "down").T


def route(h, weights, pre, top):
    """(chosen (T, top), weights (T, top)): the largest biased logits, and a
    softmax over the chosen ones only."""
    z = h @ _w(weights, pre + "router").T + _w(weights, pre + "router.b")
    idx = torch.topk(z, top, dim=-1).indices
    return idx, torch.softmax(torch.gather(z, 1, idx), dim=-1)


def moe_ff(h, weights, pre, fc):
    idx, wts = route(h, weights, pre, fc["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, wt in zip(idx[t].tolist(), wts[t]):
            out[t] += wt * expert(h[t:t + 1], weights, pre + f"e{e}.")[0]
    if fc.get("shared"):
        out = out + expert(h, weights, pre + "shared.")
    return out


# ---------------------------------------------------------------------- model
def layer(x, tokens, cfg, weights, i, rows):
    """``rows``: dict of latent rows by layer index, filled by owners."""
    lc = cfg["layers"][i]
    mc = lc["mixer"]
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    p = f"l{i}."
    if lc["type"] == "latent_attention":
        src = mc.get("kv_from")
        if src is None:
            src = i
            rows[i] = latent_rows(x @ _w(weights, p + "mix.dkv").T,
                                  _w(weights, p + "mix.dkv.norm"), mc, eps)
        y = latent_mixer(x, weights, p + "mix.", mc, eps, rows[src])
    elif lc["type"] == "gla":
        y = gla_mixer(x, weights, p + "mix.", mc, eps)
    else:
        raise ValueError(lc["type"])
    x = post_norm(x, y, alpha, _w(weights, p + "norm1"), _w(weights, p + "norm1.b"), eps)
    fc = lc.get("mlp")
    if fc:
        y = dense_ff(x, weights, p + "mlp.") if fc["kind"] == "dense" \
            else moe_ff(x, weights, p + "mlp.", fc)
        x = post_norm(x, y, alpha, _w(weights, p + "norm2"), _w(weights, p + "norm2.b"), eps)
    return token_side(x, tokens, weights, i, cfg["token_side"]["dim"], eps)


def forward(cfg, weights, tokens, collect=None):
    """Logits (T, vocab) in float64; ``collect`` (a list) receives the
    stream after every layer."""
    x = embed(tokens, weights, cfg["embedding"]["bigram"])
    rows = {}
    for i in range(len(cfg["layers"])):
        x = layer(x, tokens, cfg, weights, i, rows)
        if collect is not None:
            collect.append(x.clone())
    x = layer_norm(x, _w(weights, "final.norm"), _w(weights, "final.norm.b"), cfg["norm"]["eps"])
    return x @ _w(weights, "head").T
