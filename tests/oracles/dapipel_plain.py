"""A plain float64 implementation of the Dapipel design over whole sequences, one function per mechanism.

It shares no code with ``llmctl``: full score matrices with explicit masks, a token loop for the recurrence, a tap
loop for the convolutions, a per-token loop over the chosen experts.  ``W`` maps checkpoint tensor names to tensors,
``cfg`` is the parsed ``config.json``.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def embed(cfg, W, tokens):
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    return x + W["pos"][:len(tokens)]


def group_norm(x, w, groups, eps):
    """Every one of ``groups`` consecutive parts of a row over its own root mean square, the whole times w."""
    n = x.shape[-1] // groups
    parts = [x[..., g * n:(g + 1) * n] for g in range(groups)]
    return torch.cat([p / torch.sqrt((p * p).mean(-1, keepdim=True) + eps) for p in parts], -1) * w


def add_conv(h, w):
    """h_t + sum_j w[:, j] h_(t - taps + 1 + j), zeros before the first row."""
    T, taps = h.shape[0], w.shape[1]
    out = h.clone()
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * h[s]
    return out


def window_mask(T, size):
    i = torch.arange(T)
    d = i[:, None] - i[None, :]
    return (d >= 0) & (d < size)


def attend(q, k, v, scale, visible):
    """One softmax attention of one head: q, k [T, dim], v [T, vdim]."""
    s = (q @ k.T) * scale
    s = s.masked_fill(~visible, float("-inf"))
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return (e / e.sum(-1, keepdim=True)) @ v


def diff_lambda(W, p, diff):
    return (torch.exp((W[p + "lq1"] * W[p + "lk1"]).sum()) - torch.exp((W[p + "lq2"] * W[p + "lk2"]).sum())) + diff


def diff_attention(h, W, p, m, eps):
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m["vdim"])
    diff = float(m["diff"])
    q = (h @ W[p + "q"].T).view(T, H, 2, d)
    k = (h @ W[p + "k"].T).view(T, G, 2, d)
    v = (h @ W[p + "v"].T).view(T, G, dv)
    size = int((m.get("mask") or {}).get("size", T))
    vis = window_mask(T, size)
    lam = diff_lambda(W, p, diff)
    heads = []
    for n in range(H):
        g = n // (H // G)
        a1 = attend(q[:, n, 0], k[:, g, 0], v[:, g], float(m["scale"]), vis)
        a2 = attend(q[:, n, 1], k[:, g, 1], v[:, g], float(m["scale"]), vis)
        o = a1 - lam * a2
        heads.append(o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps) * (1.0 - diff))
    return torch.cat(heads, -1) @ W[p + "o"].T


def mingru(h, W, p, m, eps):
    z = sigmoid(h @ W[p + "z"].T + W[p + "z.b"])
    u = h @ W[p + "x"].T + W[p + "x.b"]
    cand = torch.where(u >= 0, u + 0.5, sigmoid(u))
    S = torch.zeros(u.shape[1], dtype=F64)
    rows = []
    for t in range(h.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * cand[t]
        rows.append(S)
    return (torch.stack(rows) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


MIXERS = {"attention": diff_attention, "mingru": mingru}


def dense(h, W, p):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def expert(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(h, W, p, r):
    """Per token: (chosen expert ids, their weights = the softmax over the chosen logits)."""
    z = h @ W[p + "router"].T
    picks = []
    for t in range(h.shape[0]):
        ids = torch.argsort(z[t], descending=True, stable=True)[:int(r["top"])].tolist()
        c = torch.exp(z[t, ids] - z[t, ids].max())
        picks.append((ids, (c / c.sum()).tolist()))
    return picks


def moe(h, W, p, mlp):
    out = torch.zeros_like(h)
    for t, (ids, ws) in enumerate(route(h, W, p, mlp["router"])):
        for e, w in zip(ids, ws):
            out[t] += w * expert(h[t:t + 1], W, f"{p}e{e}.")[0]
    return out


def feed_forward(h, W, p, mlp):
    return moe(h, W, p, mlp) if mlp["kind"] == "moe" else dense(h, W, p)


def forward(cfg, W, tokens):
    """Returns (logits [T, vocab], [the residual stream after every layer])."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps, groups = float(cfg["norm"]["eps"]), int(cfg["norm"].get("groups", 1))
    x = embed(cfg, W, tokens)
    trail = []
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = add_conv(group_norm(x, W[p + "norm1"], groups, eps), W[p + "canon1"])
        x = x + MIXERS[spec["type"]](h, W, p + "mix.", spec["mixer"], eps)
        if spec.get("mlp") is not None:
            h = add_conv(group_norm(x, W[p + "norm2"], groups, eps), W[p + "canon2"])
            x = x + feed_forward(h, W, p + "mlp.", spec["mlp"])
        trail.append(x)
    return group_norm(x, W["final.norm"], groups, eps) @ W["embed"].T, trail
