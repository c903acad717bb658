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
    for j in range(taps):
        back = taps - 1 - j
        for t in range(back, T):
            out[t] += w[:, j] * u[t - back]
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
    t = torch.arange(x.shape[0], dtype=F64)
    y = x.clone()
    for i, f in enumerate(frequencies(rot)):
        c, s = torch.cos(t * f), torch.sin(t * f)
        u, v = x[:, i], x[:, i + half]
        y[:, i], y[:, i + half] = u * c - v * s, v * c + u * s
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


def delta_memory(q, k, v, decay, beta, S):
    """One head over T tokens from memory S [dim, vdim]: (outputs [T, vdim], the memory after the last token)."""
    rows = []
    for t in range(v.shape[0]):
        S = decay[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        rows.append(S.T @ q[t])
    return torch.stack(rows), S


def decayed_memory(q, k, v, decay, write, S):
    """The same without the subtraction: every token adds ``write`` times k v^T."""
    rows = []
    for t in range(v.shape[0]):
        S = decay[t] * S + write[t] * torch.outer(k[t], v[t])
        rows.append(S.T @ q[t])
    return torch.stack(rows), S


def delta_rule(h, W, p, m, eps):
    """The gated delta rule: decay the memory, write the part of v that it does not give for k, read with q."""
    H, G, d, dv = int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m["vdim"])
    q, k, v = (silu(conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in ("q", "k", "v"))
    beta = sigmoid(h @ W[p + "b"].T)
    decay = torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    heads = []
    for n in range(H):
        g = n // (H // G)
        qn, kn = unit(q[:, g * d:(g + 1) * d]) * d ** -0.5, unit(k[:, g * d:(g + 1) * d])
        o, _ = delta_memory(qn, kn, v[:, n * dv:(n + 1) * dv], decay[:, n], beta[:, n], torch.zeros(d, dv, dtype=F64))
        heads.append(rms(o, eps) * W[p + "norm"])
    return (torch.cat(heads, -1) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel(h, W, p, m, eps):
    left, right = attention(h, W, p + "left.", m["left"], eps), delta_rule(h, W, p + "right.", m["right"], eps)
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


def mamba2(h, W, p, m, eps):
    H, dv, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    inner = H * dv
    z, xbc, dt = torch.split(h @ W[p + "in"].T, [inner, inner + 2 * G * N, H], -1)
    xbc = silu(conv(xbc, W[p + "conv"], W[p + "conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], -1)
    dt = softplus(dt + W[p + "dt_bias"])
    heads = []
    for n in range(H):
        g = n // (H // G)
        xn, cols = x[:, n * dv:(n + 1) * dv], slice(g * N, (g + 1) * N)
        decay = torch.exp(-torch.exp(W[p + "A_log"][n]) * dt[:, n])
        o, _ = decayed_memory(C[:, cols], B[:, cols], xn, decay, dt[:, n], torch.zeros(N, dv, dtype=F64))
        heads.append(o + W[p + "D"][n] * xn)
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
        one = torch.ones(T, dtype=F64)
        o, _ = decayed_memory(qn, kn, v[:, n * dv:(n + 1) * dv], float(m["decay"][n]) * one, one, torch.zeros(d, dv, dtype=F64))
        heads.append(rms(o, eps))
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
