"""Dumazen: a decoder-only design whose sublayers read the residual stream as it is and are normed on their way out.

* ``x = embed[token]`` (fp32 residual stream).
* A layer: ``x += residual_mult * norm1(mixer(x))``, then ``x += residual_mult * norm2(ff(x))`` (or only the first); the norms are
  RMS norms with weights stored around zero (``x / rms(x) * (1 + w)``).  The pass that ends a sublayer norms its result, adds
  it to the stream and hands the stream on in the activation dtype.
* Mixers, chosen per layer: ``parallel`` = :class:`~llmctl.models.mixers.ParallelMixers` of a windowed
  :class:`~llmctl.models.mixers.GroupedAttention` (biases, norms over all of q and all of k, rotary on half pairs with
  frequencies scaled by wavelength) and a :class:`~llmctl.models.mixers.GatedDeltaRule`, with fixed factors;
  ``mamba2`` = :class:`~llmctl.models.mixers.Mamba2`; ``retention`` = :class:`~llmctl.models.mixers.Retention`.
* Feed-forward: :class:`~llmctl.models.mixers.DenseFF` with biases and the erf GELU, or none.
* Final norm (the same kind), then ``logits = embed x``.

Checkpoint layout: ``config.json`` (``architecture``, ``vocab``, ``width``, ``norm.eps``, ``residual_mult``, ``layers`` = one entry per
layer with ``type``, ``mixer``, ``mlp`` or null) and ``model.safetensors`` with ``embed``, ``l<i>.norm1|norm2``, ``l<i>.mix.*`` (the
parallel pair: ``l<i>.mix.left.*`` and ``l<i>.mix.right.*``), ``l<i>.mlp.*``, ``final.norm``; linear weights ``[out, in]``, biases
under the weight's name with ``.b``, convolutions ``[channels, taps]`` under ``.conv``.
"""

from __future__ import annotations

import copy
import json
from dataclasses import dataclass, field
from pathlib import Path
from typing import Any, Dict, List, Optional

import torch
import torch.nn as nn

from llmctl.ops import hybrid as hops

from .mixers import DenseFF, GatedDeltaRule, GroupedAttention, Mamba2, ParallelMixers, Retention, StepBatch, _mm_f32

ARCHITECTURE = "Dumazen"


@dataclass
class DumazenConfig:
    name: str = "dumazen"
    architecture: str = ARCHITECTURE
    vocab_size: int = 512
    hidden: int = 256
    layer_specs: List[Dict[str, Any]] = field(default_factory=list)
    layer_norm_eps: float = 1e-6
    residual_mult: float = 1.0
    max_position_embeddings: int = 1 << 20
    extra: Dict[str, Any] = field(default_factory=dict)

    tie_word_embeddings = True
    is_moe = False

    @property
    def layers(self) -> int:
        return len(self.layer_specs)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "DumazenConfig":
        d = copy.deepcopy(dict(d))
        kw = dict(architecture=d.pop("architecture", ARCHITECTURE), vocab_size=int(d.pop("vocab")),
                  hidden=int(d.pop("width")), layer_specs=list(d.pop("layers")),
                  layer_norm_eps=float(d.pop("norm")["eps"]), residual_mult=float(d.pop("residual_mult", 1.0)))
        if "name" in d:
            kw["name"] = d.pop("name")
        for spec in kw["layer_specs"]:
            if spec["type"] not in MIXER_TYPES:
                raise ValueError(f"unknown mixer type {spec['type']!r} (known: {sorted(MIXER_TYPES)})")
            mlp = spec.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
        return cls(extra=d, **kw)

    @classmethod
    def from_file(cls, path) -> "DumazenConfig":
        return cls.from_dict(json.loads(Path(path).read_text()))

    def to_dict(self) -> Dict[str, Any]:
        d = {"architecture": self.architecture, "name": self.name, "vocab": self.vocab_size, "width": self.hidden,
             "norm": {"eps": self.layer_norm_eps}, "residual_mult": self.residual_mult, "layers": copy.deepcopy(self.layer_specs)}
        d.update(self.extra)
        return d

    def num_parameters(self, include_embedding: bool = True) -> int:
        with torch.device("meta"):
            m = DumazenLM(self, dtype=torch.bfloat16)
        n = sum(p.numel() for p in m.parameters())
        return n if include_embedding else n - self.vocab_size * self.hidden


def _parallel(width, m, eps, **kw):
    l, r = m["left"], m["right"]
    rot = l.get("rot") or {}
    left = GroupedAttention(width, heads=int(l["heads"]), kv_heads=int(l.get("kv_heads", l["heads"])), dim=int(l["dim"]),
                            vdim=int(l.get("vdim", l["dim"])), rot_base=float(rot.get("base", 10000.0)), rot_dims=int(rot.get("dims", 0)),
                            rot_scaling=rot.get("scaling"), interleaved=False, scale=float(l["scale"]), eps=eps,
                            window=(l.get("mask") or {}).get("size"), qk_norm="whole", bias=True, **kw)
    right = GatedDeltaRule(width, heads=int(r["heads"]), kv_heads=int(r.get("kv_heads", r["heads"])), dim=int(r["dim"]),
                           vdim=int(r.get("vdim", r["dim"])), taps=int(r["conv"]), eps=eps, **kw)
    return ParallelMixers(left, right, float(m.get("left_scale", 1.0)), float(m.get("right_scale", 1.0)))


def _mamba2(width, m, eps, **kw):
    return Mamba2(width, heads=int(m["heads"]), vdim=int(m["vdim"]), state=int(m["state"]), groups=int(m.get("groups", 1)),
                  taps=int(m["conv"]), norm_groups=int(m.get("norm_groups", 1)), eps=eps, **kw)


def _retention(width, m, eps, **kw):
    rot = m.get("rot") or {}
    return Retention(width, heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), decay=m["decay"],
                     rot_base=float(rot.get("base", 10000.0)), rot_dims=int(rot.get("dims", 0)), rot_scaling=rot.get("scaling"),
                     eps=eps, **kw)


MIXER_TYPES = {"parallel": _parallel, "mamba2": _mamba2, "retention": _retention}


class DumazenLayer(nn.Module):
    def __init__(self, cfg: DumazenConfig, spec: Dict[str, Any], device=None, dtype=None):
        super().__init__()
        W = cfg.hidden
        f32 = dict(device=device, dtype=torch.float32)
        kw = dict(device=device, dtype=dtype)
        self.mixer = MIXER_TYPES[spec["type"]](W, spec["mixer"], cfg.layer_norm_eps, **kw)
        self.norm1 = nn.Parameter(torch.zeros(W, **f32))
        mlp = spec.get("mlp")
        self.ff = None
        if mlp is not None:
            self.ff = DenseFF(W, int(mlp["ff"]), "gelu", bias=True, **kw)
            self.norm2 = nn.Parameter(torch.zeros(W, **f32))


class DumazenLM(nn.Module):
    is_hybrid = True
    has_recurrent_state = True

    def __init__(self, cfg: DumazenConfig, device=None, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.cfg = cfg
        W = cfg.hidden
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, W, device=device, dtype=dtype))
        self.layers = nn.ModuleList([DumazenLayer(cfg, s, device=device, dtype=dtype) for s in cfg.layer_specs])
        self.final_norm = nn.Parameter(torch.zeros(W, device=device, dtype=torch.float32))
        with torch.no_grad():
            self.embed.normal_(0.0, 0.02)

    @property
    def dtype(self):
        return self.embed.dtype

    def head_weight(self):
        return self.embed

    def cache_kinds(self):
        """One cache entry per layer: state pools, and the paged rows of a pair that attends."""
        out = []
        for l in self.layers:
            m = l.mixer
            if m.cache_kind == "rows+state":
                out.append(("rows+state", (m.cache_row, m.state_shapes())))
            else:
                out.append(("state", m.state_shapes()))
        return out

    # ------------------------------------------------------------------ serving step
    def step(self, b: StepBatch, cache, rows: Optional[torch.Tensor] = None, trail: Optional[list] = None):
        """Run the step's packed tokens through all layers against the engine's cache (``cache.layer(i)``).  Returns the
        fp32 residual stream of ``rows`` (all rows if None) after the last layer; ``trail`` collects it after every layer."""
        mult, eps, dt = self.cfg.residual_mult, self.cfg.layer_norm_eps, self.dtype
        x, h = hops.embed_f32(b.ids, self.embed)
        for i, layer in enumerate(self.layers):
            y = layer.mixer.step(h, b, cache.layer(i))
            (y1, s1), (y2, s2) = y if isinstance(y, tuple) else ((y, 1.0), (None, 0.0))
            h = hops.norm_add_f32_(x, y1, s1, y2, s2, layer.norm1, mult, eps, True, dt)
            if layer.ff is not None:
                h = hops.norm_add_f32_(x, layer.ff(h), 1.0, None, 0.0, layer.norm2, mult, eps, True, dt)
            if trail is not None:
                trail.append(x.clone())
        return x if rows is None else x.index_select(0, rows)

    def logits(self, x: torch.Tensor) -> torch.Tensor:
        xn, _ = hops.add_rmsnorm2_f32_(x.contiguous(), None, None, self.final_norm, None, self.cfg.layer_norm_eps, True, self.dtype)
        return _mm_f32(xn, self.embed)

    # ------------------------------------------------------------------ checkpoint names
    def _named(self):
        """(tensors of the checkpoint, stacked in order, parameter or its filled rows) for every parameter."""
        def recurrent(m, q):
            n = m.cols
            if isinstance(m, Mamba2):
                yield [q + "in"], m.w_in[:n]
                yield from (([q + "conv"], m.conv.weight), ([q + "conv.b"], m.conv_bias), ([q + "D"], m.skip), ([q + "norm"], m.norm))
            elif isinstance(m, Retention):
                yield [q + s for s in ("q", "k", "v", "g")], m.w_in[:n]
            else:
                yield [q + s for s in ("q", "k", "v", "g", "a", "b")], m.w_in[:n]
                yield [q + s + ".conv" for s in ("q", "k", "v")], m.conv.weight
                yield [q + "norm"], m.norm
            if not isinstance(m, Retention):
                yield [q + "A_log"], m.a_log
                yield [q + "dt_bias"], m.dt_bias
            yield [q + "o"], m.w_o

        yield ["embed"], self.embed
        yield ["final.norm"], self.final_norm
        for i, layer in enumerate(self.layers):
            p, m = f"l{i}.", layer.mixer
            yield [p + "norm1"], layer.norm1
            if isinstance(m, ParallelMixers):
                a, q = m.left, p + "mix.left."
                yield [q + s for s in ("q", "k", "v")], a.w_qkv
                yield [q + s + ".b" for s in ("q", "k", "v")], a.b_qkv
                yield [q + "q.norm"], a.q_norm
                yield [q + "k.norm"], a.k_norm
                yield [q + "o"], a.w_o
                yield from recurrent(m.right, p + "mix.right.")
            else:
                yield from recurrent(m, p + "mix.")
            if layer.ff is not None:
                yield [p + "norm2"], layer.norm2
                for s in ("up", "down"):
                    yield [f"{p}mlp.{s}"], getattr(layer.ff, "w_" + s)
                    yield [f"{p}mlp.{s}.b"], getattr(layer.ff, "b_" + s)

    def _split_rows(self, names: List[str]) -> List[int]:
        """Rows of every checkpoint tensor that a stacked parameter holds."""
        layer = self.layers[int(names[0].split(".")[0][1:])].mixer
        m = (layer.left if ".left." in names[0] else layer.right) if isinstance(layer, ParallelMixers) else layer
        H, dk, dv = m.H, m.dk, m.dv
        G = getattr(m, "G", H)
        v = G * dv if isinstance(m, GroupedAttention) else H * dv
        q = G * dk if isinstance(m, GatedDeltaRule) else H * dk
        return [q, G * dk, v, H * dv, H, H][:len(names)]

    @torch.no_grad()
    def load_named(self, W: Dict[str, torch.Tensor]) -> None:
        """Copy a checkpoint's tensors (its names, see the module docstring) into the fused parameters."""
        for names, dst in self._named():
            if len(names) > 1:
                for n, rows in zip(names, self._split_rows(names)):
                    if W[n].shape[0] != rows:
                        raise ValueError(f"{n}: {W[n].shape[0]} rows, the configuration has {rows}")
            src = torch.cat([W[n] for n in names], 0) if len(names) > 1 else W[names[0]]
            if tuple(dst.shape) != tuple(src.shape):
                raise ValueError(f"{names[0]}: shape {tuple(src.shape)} does not fit {tuple(dst.shape)}")
            dst.copy_(src.to(dst.dtype))

    @torch.no_grad()
    def export_named(self) -> Dict[str, torch.Tensor]:
        """The inverse of :meth:`load_named`: tensors under the checkpoint's names."""
        out = {}
        for names, src in self._named():
            parts = [src] if len(names) == 1 else src.split(self._split_rows(names), 0)
            out.update(zip(names, parts))
        return {k: v.detach().clone().contiguous() for k, v in out.items()}


def load_dumazen(ck: Path, cfg: DumazenConfig, device=None, dtype=torch.bfloat16) -> DumazenLM:
    from safetensors import safe_open

    with safe_open(str(ck / "model.safetensors"), framework="pt", device="cpu") as f:
        W = {k: f.get_tensor(k) for k in f.keys()}
    model = DumazenLM(cfg, device=device, dtype=dtype)
    model.load_named(W)
    return model


def dumazen_template(width: int = 256, layers: int = 4, heads: int = 4, kv_heads: int = 2, vocab: int = 512, every: int = 3,
                     ff: Optional[int] = None, head_dim: Optional[int] = None, window: int = 1024, taps: int = 4) -> DumazenConfig:
    """A random-init configuration for benchmarks and smoke runs: every ``every``-th layer is the parallel pair of windowed
    attention (heads of ``head_dim``) and gated delta rule, the others are Mamba-2 and retention by turns; the memories
    have ``heads`` heads with keys of half of ``head_dim`` and values of ``head_dim``.  A dense feed-forward in every layer."""
    d = head_dim or width // heads
    dk = max(d // 2 // 2 * 2, 2)
    par = {"left": {"heads": heads, "kv_heads": kv_heads, "dim": d, "vdim": d, "scale": d ** -0.5, "mask": {"size": window},
                    "rot": {"base": 100000.0, "dims": d // 2 * 2, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 8192}}},
           "right": {"heads": heads, "kv_heads": heads, "dim": dk, "vdim": d, "conv": taps}, "left_scale": 0.5, "right_scale": 0.5}
    ssm = {"heads": heads, "vdim": d, "state": dk, "groups": 1, "conv": taps, "norm_groups": 1}
    ret = {"heads": heads, "dim": dk, "vdim": d, "rot": {"base": 10000.0, "dims": dk},
           "decay": [1.0 - 2.0 ** -(5.0 + 5.0 * i / max(heads - 1, 1)) for i in range(heads)]}
    mlp = {"kind": "dense", "ff": ff or 4 * width}
    specs, turn = [], 0
    for i in range(layers):
        if (i + 1) % every == 0:
            t, m = "parallel", par
        else:
            t, m = (("mamba2", ssm), ("retention", ret))[turn % 2]
            turn += 1
        specs.append({"type": t, "mixer": copy.deepcopy(m), "mlp": copy.deepcopy(mlp)})
    return DumazenConfig(name=f"dumazen-w{width}-l{layers}", vocab_size=vocab, hidden=width, layer_specs=specs,
                         layer_norm_eps=1e-6, residual_mult=0.5)
