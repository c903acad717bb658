"""Helpers of the Dumazen tests: small configurations and random checkpoints written from the naming rules of
the checkpoint layout (not from the model class).  The engine, the schedule driver and the error measures are
those of the Lenitar and Malinex tests."""

from __future__ import annotations

import copy
import math
from typing import Dict, List, Optional, Tuple

import torch

from tests.models.lenitar_util import engine, rel_err, run_schedule, write_checkpoint  # noqa: F401
from tests.models.malinex_util import rel_errs  # noqa: F401

SCALING = {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 48}


def left(heads=4, kv_heads=2, dim=8, vdim=6, window=7, base=300.0, dims=None, scaling=SCALING, scale=None):
    rot = {"base": base, "dims": dims if dims is not None else dim // 2 * 2}
    if scaling:
        rot["scaling"] = dict(scaling)
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "rot": rot,
            "scale": scale if scale is not None else 1.3 * dim ** -0.5}


def right(heads=3, kv_heads=3, dim=6, vdim=5, conv=4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def par(l=None, r=None, left_scale=0.7, right_scale=0.45):
    return {"type": "parallel", "mixer": {"left": l or left(), "right": r or right(), "left_scale": left_scale, "right_scale": right_scale}}


def ssm(heads=4, vdim=6, state=7, groups=2, conv=3, norm_groups=3):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": norm_groups}}


def ret(heads=3, dim=8, vdim=5, base=500.0, dims=None, decay=None):
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay or [0.9, 0.97, 0.995, 0.8, 1.0, 0.5][:heads],
                                           "rot": {"base": base, "dims": dims if dims is not None else dim // 2 * 2}}}


def dense(ff=18):
    return {"kind": "dense", "ff": ff}


def config(layers: List[Tuple[dict, Optional[dict]]], width=24, vocab=50, eps=1e-6, mult=0.6) -> dict:
    return {"architecture": "Dumazen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "layers": [dict(copy.deepcopy(m), mlp=copy.deepcopy(f)) for m, f in layers]}


def random_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def lin(o, i, gain=1.0):
        return (torch.randn(o, i, generator=g) * gain / math.sqrt(i)).bfloat16().float()

    def vec(n, mean=0.0, std=1.0):
        return (mean + std * torch.randn(n, generator=g)).bfloat16().float()

    def delta(q, m):
        H, G, d, dv, t = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
        out = {q + "q": lin(G * d, W), q + "k": lin(G * d, W), q + "v": lin(H * dv, W), q + "g": lin(H * dv, W, 1.5), q + "a": lin(H, W),
               q + "b": lin(H, W, 1.5), q + "o": lin(W, H * dv), q + "norm": vec(dv, 1.0, 0.2), q + "A_log": vec(H, -1.0, 0.7),
               q + "dt_bias": vec(H, -2.0, 1.0)}
        for n, c in (("q", G * d), ("k", G * d), ("v", H * dv)):
            out[f"{q}{n}.conv"] = vec(c * t, 0.2, 0.5).view(c, t)
        return out

    out = {"embed": vec(cfg["vocab"] * W).view(cfg["vocab"], W), "final.norm": vec(W, 0.0, 0.2)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        q = p + "mix."
        out[p + "norm1"] = vec(W, 0.0, 0.2)
        if layer["type"] == "parallel":
            l, ql = m["left"], q + "left."
            H, G, d, dv = l["heads"], l["kv_heads"], l["dim"], l["vdim"]
            for n, rows, gain in (("q", H * d, 1.5), ("k", G * d, 1.5), ("v", G * dv, 1.0)):
                out[ql + n], out[ql + n + ".b"] = lin(rows, W, gain), vec(rows, 0.0, 0.4)
            out.update({ql + "q.norm": vec(H * d, 1.0, 0.3), ql + "k.norm": vec(G * d, 1.0, 0.3), ql + "o": lin(W, H * dv)})
            out.update(delta(q + "right.", m["right"]))
        elif layer["type"] == "mamba2":
            H, dv, N, G, t = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
            c = H * dv + 2 * G * N
            out.update({q + "in": lin(H * dv + c + H, W, 1.3), q + "conv": vec(c * t, 0.2, 0.5).view(c, t), q + "conv.b": vec(c, 0.0, 0.3),
                        q + "dt_bias": vec(H, -2.0, 1.0), q + "A_log": vec(H, -0.5, 0.7), q + "D": vec(H, 0.5, 0.5),
                        q + "norm": vec(H * dv, 1.0, 0.2), q + "o": lin(W, H * dv)})
        else:
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            out.update({q + "q": lin(H * d, W), q + "k": lin(H * d, W), q + "v": lin(H * dv, W), q + "g": lin(H * dv, W, 1.5),
                        q + "o": lin(W, H * dv)})
        if f is not None:
            out[p + "norm2"] = vec(W, 0.0, 0.2)
            out.update({p + "mlp.up": lin(f["ff"], W, 1.5), p + "mlp.up.b": vec(f["ff"], 0.0, 0.4), p + "mlp.down": lin(W, f["ff"]),
                        p + "mlp.down.b": vec(W, 0.0, 0.4)})
    return out
