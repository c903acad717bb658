"""A plain float64 implementation of the Dumazen design over whole sequences, one function per mechanism.

It shares no code with ``llmctl``: full score matrices with explicit masks, token loops for the three recurrences, a
tap loop for the convolutions.  ``W`` maps checkpoint tensor names to tensors, ``cfg`` is the parsed ``config.json``.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def rms(x, eps):
    """x over its own root mean square (last axis)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_one_plus(x, w, eps):
    """An RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1.0 + w)


def conv(u, w, bias=None):
    """sum_j w[:, j] u_(t - taps + 1 + j) (+ bias) per channel, zeros before the first row."""
    T, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * u[s]
    return out if bias is None else out + bias


def frequencies(rot):
    """Rotary frequencies of ``rot`` = {base, dims[, scaling]}: wavelengths below original / high keep theirs, those above
    original / low are divided by factor, a ramp in original / wavelength lies between."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    sc = rot.get("scaling")
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            wl = 2.0 * math.pi / f
            factor, low, high, orig = (float(sc[k]) for k in ("factor", "low", "high", "original"))
            if wl > orig / low:
                f = f / factor
            elif wl >= orig / high:
                s = (orig / wl - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return out


def rotate(x, rot):
    """x [T, n]: entry i of the first ``dims`` is turned with entry i + dims/2 by position * f_i."""
    half = int(rot["dims"]) // 2
    y = x.clone()
    for t in range(x.shape[0]):
        for i, f in enumerate(frequencies(rot)):
            c, s = math.cos(t * f), math.sin(t * f)
            u, v = x[t, i], x[t, i + half]
            y[t, i], y[t, i + half] = u * c - v * s, v * c + u * s
    return y


def window_mask(T, size):
    i = torch.arange(T)
    d = i[:, None] - i[None, :]
    return (d >= 0) & (d < size)


def attention(h, W, p, m, eps):
    """Windowed grouped-query softmax attention: biases on q, k, v; q and k normed as whole rows, then rotated."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m["vdim"])
    q = rms(h @ W[p + "q"].T + W[p + "q.b"], eps) * W[p + "q.norm"]
    k = rms(h @ W[p + "k"].T + W[p + "k.b"], eps) * W[p + "k.norm"]
    v = h @ W[p + "v"].T + W[p + "v.b"]
    vis = window_mask(T, int(m["mask"]["size"]))
    ks = [rotate(k[:, g * d:(g + 1) * d], m["rot"]) for g in range(G)]
    heads = []
    for n in range(H):
        g = n // (H // G)
        s = (rotate(q[:, n * d:(n + 1) * d], m["rot"]) @ ks[g].T) * float(m["scale"])
        s = s.masked_fill(~vis, float("-inf"))
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        heads.append((e / e.sum(-1, keepdim=True)) @ v[:, g * dv:(g + 1) * dv])
    return torch.cat(heads, -1) @ W[p + "o"].T


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(h, W, p, m, eps):
    """The gated delta rule: decay the memory, write the part of v that it does not give for k, read with q."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m["vdim"])
    q, k, v = (silu(conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in ("q", "k", "v"))
    beta = sigmoid(h @ W[p + "b"].T)
    decay = torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    heads = []
    for n in range(H):
        g = n // (H // G)
        qn, kn = unit(q[:, g * d:(g + 1) * d]) * d ** -0.5, unit(k[:, g * d:(g + 1) * d])
        S, rows = torch.zeros(d, dv, dtype=F64), []
        for t in range(T):
            S = decay[t, n] * S
            u = beta[t, n] * (v[t, n * dv:(n + 1) * dv] - S.T @ kn[t])
            S = S + torch.outer(kn[t], u)
            rows.append(S.T @ qn[t])
        heads.append(rms(torch.stack(rows), eps) * W[p + "norm"])
    return (torch.cat(heads, -1) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel(h, W, p, m, eps):
    left, right = attention(h, W, p + "left.", m["left"], eps), delta_rule(h, W, p + "right.", m["right"], eps)
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


def mamba2(h, W, p, m, eps):
    T = h.shape[0]
    H, dv, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    inner = H * dv
    z, xbc, dt = torch.split(h @ W[p + "in"].T, [inner, inner + 2 * G * N, H], -1)
    xbc = silu(conv(xbc, W[p + "conv"], W[p + "conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], -1)
    dt = softplus(dt + W[p + "dt_bias"])
    heads = []
    for n in range(H):
        g = n // (H // G)
        S, rows = torch.zeros(N, dv, dtype=F64), []
        for t in range(T):
            xt = x[t, n * dv:(n + 1) * dv]
            S = torch.exp(-torch.exp(W[p + "A_log"][n]) * dt[t, n]) * S + dt[t, n] * torch.outer(B[t, g * N:(g + 1) * N], xt)
            rows.append(S.T @ C[t, g * N:(g + 1) * N] + W[p + "D"][n] * xt)
        heads.append(torch.stack(rows))
    y = torch.cat(heads, -1) * silu(z)
    part = inner // int(m["norm_groups"])
    y = torch.cat([rms(y[:, i:i + part], eps) for i in range(0, inner, part)], -1) * W[p + "norm"]
    return y @ W[p + "o"].T


def retention(h, W, p, m, eps):
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = h @ W[p + "q"].T, h @ W[p + "k"].T, h @ W[p + "v"].T
    heads = []
    for n in range(H):
        qn, kn = rotate(q[:, n * d:(n + 1) * d], m["rot"]), rotate(k[:, n * d:(n + 1) * d], m["rot"]) * d ** -0.5
        S, rows = torch.zeros(d, dv, dtype=F64), []
        for t in range(T):
            S = float(m["decay"][n]) * S + torch.outer(kn[t], v[t, n * dv:(n + 1) * dv])
            rows.append(S.T @ qn[t])
        heads.append(rms(torch.stack(rows), eps))
    return (torch.cat(heads, -1) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


MIXERS = {"parallel": parallel, "mamba2": mamba2, "retention": retention}


def dense(h, W, p):
    return gelu_erf(h @ W[p + "up"].T + W[p + "up.b"]) @ W[p + "down"].T + W[p + "down.b"]


def forward(cfg, W, tokens):
    """Returns (logits [T, vocab], [the residual stream after every layer])."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    trail = []
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + mult * norm_one_plus(MIXERS[spec["type"]](x, W, p + "mix.", spec["mixer"], eps), W[p + "norm1"], eps)
        if spec.get("mlp") is not None:
            x = x + mult * norm_one_plus(dense(x, W, p + "mlp."), W[p + "norm2"], eps)
        trail.append(x)
    return norm_one_plus(x, W["final.norm"], eps) @ W["embed"].T, trail
