"""Helpers of the Dapipel tests: small configurations and random checkpoints written from the naming rules of
the checkpoint layout (not from the model class).  The engine, the schedule driver and the error measures are
those of the Lenitar and Malinex tests."""

from __future__ import annotations

import copy
import math
from typing import Dict, List, Optional, Tuple

import torch

from tests.models.lenitar_util import engine, rel_err, run_schedule, write_checkpoint  # noqa: F401
from tests.models.malinex_util import rel_errs  # noqa: F401


def att(heads=4, kv_heads=2, dim=8, vdim=6, window=7, diff=0.35, scale=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff,
                                           "scale": scale if scale is not None else 1.5 * dim ** -0.5, "mask": {"size": window}}}


def gru(width=22):
    return {"type": "mingru", "mixer": {"width": width}}


def dense(ff=18):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=10):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(layers: List[Tuple[dict, Optional[dict]]], width=24, vocab=50, eps=1e-5, groups=3, taps=3, scale=1.7,
           positions=160) -> dict:
    return {"architecture": "Dapipel", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups}, "canon": {"taps": taps},
            "embedding": {"scale": scale}, "max_positions": positions,
            "layers": [dict(copy.deepcopy(m), mlp=copy.deepcopy(f)) for m, f in layers]}


def without_choice(cfg: dict) -> dict:
    """The configuration with routers that choose every expert: nothing can flip under bf16 rounding.  Tensor shapes stay."""
    out = copy.deepcopy(cfg)
    for s in out["layers"]:
        if (s.get("mlp") or {}).get("kind") == "moe":
            s["mlp"]["router"]["top"] = s["mlp"]["router"]["experts"]
    return out


def random_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    g = torch.Generator().manual_seed(seed)
    W, taps = cfg["width"], cfg["canon"]["taps"]

    def lin(o, i, gain=1.0):
        return (torch.randn(o, i, generator=g) * gain / math.sqrt(i)).bfloat16().float()

    def vec(n, mean=0.0, std=1.0):
        return (mean + std * torch.randn(n, generator=g)).bfloat16().float()

    out = {"embed": vec(cfg["vocab"] * W).view(cfg["vocab"], W), "pos": vec(cfg["max_positions"] * W, 0.0, 0.5).view(-1, W),
           "final.norm": vec(W, 1.0, 0.2)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        for n in (1, 2) if f is not None else (1,):
            out[f"{p}norm{n}"], out[f"{p}canon{n}"] = vec(W, 1.0, 0.2), vec(W * taps, 0.0, 0.5).view(W, taps)
        q = p + "mix."
        if layer["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            out.update({q + "q": lin(H * 2 * d, W, 1.5), q + "k": lin(G * 2 * d, W, 1.5), q + "v": lin(G * dv, W), q + "o": lin(W, H * dv)})
            for n, s in (("lq1", -0.3), ("lk1", 0.3), ("lq2", 0.1), ("lk2", 0.1)):
                out[q + n] = vec(d, s, 0.1)
        else:
            n = m["width"]
            out.update({q + "z": lin(n, W, 1.5), q + "z.b": vec(n, -1.0, 1.5), q + "x": lin(n, W, 1.5), q + "x.b": vec(n, 0.0, 0.7),
                        q + "g": lin(n, W, 1.5), q + "o": lin(W, n)})
        if f is None:
            continue
        if f["kind"] == "dense":
            out.update({p + "mlp.gate": lin(f["ff"], W, 2.0), p + "mlp.up": lin(f["ff"], W), p + "mlp.down": lin(W, f["ff"])})
        else:
            E, ff = f["router"]["experts"], f["expert"]["ff"]
            out[p + "mlp.router"] = lin(E, W, 3.0)
            for e in range(E):
                out[f"{p}mlp.e{e}.gate"], out[f"{p}mlp.e{e}.up"], out[f"{p}mlp.e{e}.down"] = lin(ff, W, 2.0), lin(ff, W), lin(W, ff)
    return out
