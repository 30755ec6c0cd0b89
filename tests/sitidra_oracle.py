"""Plain, slow, whole-sequence Sitidra in float64, one function per mechanism,
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


def layer_norm(x, w, eps):
    dev = x - x.mean(-1, keepdim=True)
    return dev / torch.sqrt((dev * dev).mean(-1, keepdim=True) + eps) * w


# -------------------------------------------------------- parallel streams
def hyper_read(xs, w_in):
    """xs (T, s, W), w_in (s,) -> the sublayer's view of the streams."""
    u = torch.zeros_like(xs[:, 0])
    for s in range(xs.shape[1]):
        u = u + w_in[s] * xs[:, s]
    return u


def hyper_write(xs, y, mix, w_out):
    """All streams anew from the old ones: stream t is sum_s mix[s, t] x_s
    plus out[t] times the sublayer's result."""
    new = torch.zeros_like(xs)
    n = xs.shape[1]
    for t in range(n):
        for s in range(n):
            new[:, t] += mix[s, t] * xs[:, s]
        new[:, t] += w_out[t] * y
    return new


# ------------------------------------------------------------------ attention
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


def unit_heads(x, n, mc, eps):
    """(T, n * dim) -> (T, n, dim): rotated, then divided by the head's own
    root mean square."""
    T = x.shape[0]
    x = x.view(T, n, -1)
    rot = mc.get("rot")
    if rot:
        x = rotate_halves(x, torch.arange(T), rot["base"], rot["dims"])
    return rms(x, eps)


def block_attend(q, k, v, scale, size, head_gate=None):
    """q (T, H, D), k (T, G, D), v (T, G, Dv), head_gate (T, H) logits or
    None: softmax over the keys of the query's own block of ``size``
    positions. Returns the concatenated heads (T, H * Dv)."""
    T, H = q.shape[:2]
    G = k.shape[1]
    i = torch.arange(T)
    seen = (i.view(1, T) <= i.view(T, 1))
    if size:
        seen &= (i // size).view(1, T) == (i // size).view(T, 1)
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        out[:, h] = torch.softmax(s.masked_fill(~seen, float("-inf")), dim=-1) @ v[:, g]
    if head_gate is not None:
        out = out * torch.sigmoid(head_gate).view(T, H, 1)
    return out.reshape(T, -1)


def mix_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attention_mixer(h, weights, pre, mc, eps, first):
    """``first``: the values of the first value-mixing layer, or None in a
    layer that does not mix (that first one included). Returns (output, this
    layer's values as projected)."""
    T = h.shape[0]
    H, G = mc["heads"], mc["kv_heads"]
    q = unit_heads(h @ _w(weights, pre + "q").T, H, mc, eps)
    k = unit_heads(h @ _w(weights, pre + "k").T, G, mc, eps)
    v = h @ _w(weights, pre + "v").T
    vm = v if first is None else mix_values(v, first, _w(weights, pre + "vmix").reshape(()))
    heads = block_attend(q, k, vm.view(T, G, -1), mc["scale"], mc["mask"]["size"],
                         h @ _w(weights, pre + "g").T)
    return heads @ _w(weights, pre + "o").T, v


# --------------------------------------------------- matrix memory (mLSTM)
def mlstm_gates(zi, zf, cap):
    """Gate logits (T, H), biases included -> (log input gate, log forget
    gate)."""
    return cap * torch.tanh(zi / cap), torch.nn.functional.logsigmoid(cap * torch.tanh(zf / cap))


def mlstm_scan(q, k, v, i, f):
    """q, k (T, H, D), v (T, H, Dv), i, f (T, H) log gates -> (o (T, H, Dv),
    (S, n, m))."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    n = torch.zeros(H, D, dtype=F64)
    m = torch.zeros(H, dtype=F64)
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep = torch.exp(f[t] + m - m_new).view(H, 1)
        add = torch.exp(i[t] - m_new).view(H, 1)
        S = keep.unsqueeze(-1) * S + (add * k[t]).unsqueeze(-1) * v[t].unsqueeze(1)
        n = keep * n + add * k[t]
        m = m_new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t].unsqueeze(-1)).sum(1) / den.view(H, 1)
    return out, (S, n, m)


def mlstm_mixer(h, weights, pre, mc, eps):
    T = h.shape[0]
    H, D, Dv = mc["heads"], mc["dim"], mc["vdim"]
    q = (h @ _w(weights, pre + "q").T).view(T, H, D) * D ** -0.5
    k = (h @ _w(weights, pre + "k").T).view(T, H, D)
    v = (h @ _w(weights, pre + "v").T).view(T, H, Dv)
    i, f = mlstm_gates(h @ _w(weights, pre + "i").T + _w(weights, pre + "i.b"),
                       h @ _w(weights, pre + "f").T + _w(weights, pre + "f.b"), mc["gate_cap"])
    o, _ = mlstm_scan(q, k, v, i, f)
    o = rms(o, eps).reshape(T, H * Dv) * _w(weights, pre + "norm")
    return (o * torch.sigmoid(h @ _w(weights, pre + "g").T)) @ _w(weights, pre + "o").T


# --------------------------------------------------------------- feed-forward
def expert(h, weights, pre):
    g = h @ _w(weights, pre + "gate").T
    return (g * torch.sigmoid(g) * (h @ _w(weights, pre + "up").T)) @ _w(weights, pre + "down").T


def route(z, corr, rc):
    """Router logits (T, E) -> per token the list of (expert, weight)."""
    E, top = rc["experts"], rc["top"]
    gc = rc.get("groups") or {"count": 1, "keep": 1}
    per = E // gc["count"]
    out = []
    for row in z:
        s = torch.sigmoid(row)
        choice = (s + corr).tolist()
        groups = []
        for g in range(gc["count"]):
            members = sorted(choice[g * per:(g + 1) * per], reverse=True)
            groups.append((sum(members[:2]), g))
        best = [g for _, g in sorted(groups, reverse=True)[:gc["keep"]]]
        open_ = [e for e in range(E) if e // per in best]
        chosen = sorted(open_, key=lambda e: -choice[e])[:top]
        total = sum(s[e] for e in chosen) + 1e-20
        out.append([(e, s[e] / total * rc["scale"]) for e in chosen])
    return out


def moe_ff(h, weights, pre, fc):
    picks = route(h @ _w(weights, pre + "router").T, _w(weights, pre + "correction"), fc["router"])
    out = torch.zeros_like(h)
    for t, row in enumerate(picks):
        for e, wt in row:
            out[t] += wt * expert(h[t:t + 1], weights, pre + f"e{e}.")[0]
    if fc.get("shared"):
        out = out + expert(h, weights, pre + "shared.")
    return out


# ---------------------------------------------------------------------- model
def layer(xs, cfg, weights, i, firsts):
    """``firsts``: a list that holds the first value-mixing layer's values
    once that layer has run."""
    lc = cfg["layers"][i]
    mc = lc["mixer"]
    eps = cfg["norm"]["eps"]
    p = f"l{i}."

    def sub(xs, q, f):
        u = hyper_read(xs, _w(weights, p + f"hc{q}.in"))
        y = f(layer_norm(u, _w(weights, p + f"norm{q}"), eps))
        return hyper_write(xs, y, _w(weights, p + f"hc{q}.mix"), _w(weights, p + f"hc{q}.out"))

    def mixer(h):
        if lc["type"] == "attention":
            mixes = bool(mc.get("v_mix"))
            y, v = attention_mixer(h, weights, p + "mix.", mc, eps,
                                   firsts[0] if mixes and firsts else None)
            if mixes and not firsts:
                firsts.append(v)
            return y
        if lc["type"] == "mlstm":
            return mlstm_mixer(h, weights, p + "mix.", mc, eps)
        raise ValueError(lc["type"])

    xs = sub(xs, 1, mixer)
    if lc.get("mlp"):
        xs = sub(xs, 2, lambda h: moe_ff(h, weights, p + "mlp.", lc["mlp"]))
    return xs


def forward(cfg, weights, tokens, collect=None):
    """Logits (T, vocab) in float64; ``collect`` (a list) receives the sum of
    the streams after every layer."""
    x = _w(weights, "embed")[[int(t) for t in tokens]]
    xs = x.unsqueeze(1).repeat(1, cfg["streams"], 1)
    firsts = []
    for i in range(len(cfg["layers"])):
        xs = layer(xs, cfg, weights, i, firsts)
        if collect is not None:
            collect.append(xs.sum(1))
    x = layer_norm(xs.sum(1), _w(weights, "final.norm"), cfg["norm"]["eps"])
    logits = x @ _w(weights, "head").T
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits
