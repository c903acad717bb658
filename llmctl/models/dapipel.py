"""Dapipel: a decoder-only design of pre-norm layers whose sublayers read a causally convolved input, elementwise
recurrences among windowed differential attentions.

* ``x = embed[token] * embedding_scale + pos[position]`` (fp32 residual stream).
* A layer: ``x += mixer(in1(x))``, then ``x += ff(in2(x))``, where ``in(x) = h + conv(h)``, ``h`` = an RMS norm of x in
  ``norm_groups`` equal consecutive parts (each over its own root mean square, the whole times a weight) and ``conv`` a
  causal convolution over time per channel.  The last ``taps - 1`` rows of h of both sublayers are part of a sequence's
  state in every layer.  The update of the stream, the norm and the convolution are one pass over the rows.
* Mixers, chosen per layer: ``mingru`` = :class:`~llmctl.models.mixers.MinGRU` (an fp32 vector per state slot) and
  ``attention`` = :class:`~llmctl.models.mixers.DifferentialAttention` (paged rows ``[v | k_1 | k_2]``).
* Feed-forward: ``dense`` = :class:`~llmctl.models.mixers.GatedFF` with the tanh GELU, or ``moe`` =
  :class:`~llmctl.models.moe.BiasedSoftmaxMoE` with gated SiLU experts weighted by the softmax over the chosen logits
  (no selection bias, no shared expert), or none.
* Final norm (the same grouped one), then ``logits = embed x`` (the unscaled embedding table).

Checkpoint layout: ``config.json`` (``architecture``, ``vocab``, ``width``, ``embedding.scale``, ``norm.eps``,
``norm.groups``, ``canon.taps``, ``max_positions``, ``layers`` = one entry per layer with ``type``, ``mixer``, ``mlp`` or
null) and ``model.safetensors`` with ``embed``, ``pos``, ``l<i>.norm1|norm2``, ``l<i>.canon1|canon2`` (``[width, taps]``),
``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``; linear weights ``[out, in]``.
"""

from __future__ import annotations

import copy
import json
from dataclasses import dataclass, field
from pathlib import Path
from typing import Any, Dict, List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from llmctl.ops import hybrid as hops

from .mixers import CausalConv, DifferentialAttention, GatedFF, MinGRU, StepBatch, _mm_f32
from .moe import BiasedSoftmaxMoE

ARCHITECTURE = "Dapipel"


@dataclass
class DapipelConfig:
    name: str = "dapipel"
    architecture: str = ARCHITECTURE
    vocab_size: int = 512
    hidden: int = 256
    layer_specs: List[Dict[str, Any]] = field(default_factory=list)
    layer_norm_eps: float = 1e-5
    norm_groups: int = 1
    taps: int = 4
    embedding_scale: float = 1.0
    max_position_embeddings: int = 8192
    extra: Dict[str, Any] = field(default_factory=dict)

    tie_word_embeddings = True

    @property
    def is_moe(self) -> bool:
        return any((s.get("mlp") or {}).get("kind") == "moe" for s in self.layer_specs)

    @property
    def layers(self) -> int:
        return len(self.layer_specs)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "DapipelConfig":
        d = copy.deepcopy(dict(d))
        norm = d.pop("norm")
        kw = dict(architecture=d.pop("architecture", ARCHITECTURE), vocab_size=int(d.pop("vocab")),
                  hidden=int(d.pop("width")), layer_specs=list(d.pop("layers")), layer_norm_eps=float(norm["eps"]),
                  norm_groups=int(norm.get("groups", 1)), taps=int(d.pop("canon")["taps"]),
                  embedding_scale=float((d.pop("embedding", None) or {}).get("scale", 1.0)),
                  max_position_embeddings=int(d.pop("max_positions", d.pop("max_position_embeddings", 8192))))
        if "name" in d:
            kw["name"] = d.pop("name")
        if kw["hidden"] % kw["norm_groups"]:
            raise ValueError("the norm's groups must divide the width")
        if kw["taps"] < 1:
            raise ValueError("the input convolutions need at least one tap")
        for spec in kw["layer_specs"]:
            if spec["type"] not in MIXER_TYPES:
                raise ValueError(f"unknown mixer type {spec['type']!r} (known: {sorted(MIXER_TYPES)})")
            mlp = spec.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") not in ("dense", "moe"):
                raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
        return cls(extra=d, **kw)

    @classmethod
    def from_file(cls, path) -> "DapipelConfig":
        return cls.from_dict(json.loads(Path(path).read_text()))

    def to_dict(self) -> Dict[str, Any]:
        d = {"architecture": self.architecture, "name": self.name, "vocab": self.vocab_size, "width": self.hidden,
             "norm": {"eps": self.layer_norm_eps, "groups": self.norm_groups}, "canon": {"taps": self.taps},
             "embedding": {"scale": self.embedding_scale}, "max_positions": self.max_position_embeddings,
             "layers": copy.deepcopy(self.layer_specs)}
        d.update(self.extra)
        return d

    def num_parameters(self, include_embedding: bool = True) -> int:
        with torch.device("meta"):
            m = DapipelLM(self, dtype=torch.bfloat16)
        n = sum(p.numel() for p in m.parameters())
        return n if include_embedding else n - self.vocab_size * self.hidden


def _mingru(width, m, eps, **kw):
    return MinGRU(width, state_width=int(m["width"]), **kw)


def _attention(width, m, eps, **kw):
    return DifferentialAttention(width, heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])), dim=int(m["dim"]),
                                 vdim=int(m["vdim"]), scale=float(m["scale"]), diff=float(m["diff"]), eps=eps,
                                 window=(m.get("mask") or {}).get("size"), **kw)


MIXER_TYPES = {"mingru": _mingru, "attention": _attention}


class DapipelLayer(nn.Module):
    def __init__(self, cfg: DapipelConfig, spec: Dict[str, Any], device=None, dtype=None):
        super().__init__()
        W = cfg.hidden
        f32 = dict(device=device, dtype=torch.float32)
        kw = dict(device=device, dtype=dtype)
        self.norm1 = nn.Parameter(torch.ones(W, **f32))
        self.canon1 = CausalConv(W, cfg.taps, residual=True, device=device)
        self.mixer = MIXER_TYPES[spec["type"]](W, spec["mixer"], cfg.layer_norm_eps, **kw)
        mlp = spec.get("mlp")
        self.ff = None
        if mlp is not None:
            if mlp.get("kind", "dense") == "dense":
                self.ff = GatedFF(W, int(mlp["ff"]), "gelu_tanh", **kw)
            else:
                r = mlp["router"]
                self.ff = BiasedSoftmaxMoE(W, int(mlp["expert"]["ff"]), int(r["experts"]), int(r["top"]), "swiglu",
                                           select_bias=False, **kw)
            self.norm2 = nn.Parameter(torch.ones(W, **f32))
            self.canon2 = CausalConv(W, cfg.taps, residual=True, device=device)

    def sublayers(self):
        """(norm weight, input convolution) per sublayer, in order."""
        return [(self.norm1, self.canon1)] + ([(self.norm2, self.canon2)] if self.ff is not None else [])

    def state_shapes(self):
        """The mixer's own state, then the carried rows of the input convolutions."""
        return list(self.mixer.state_shapes()) + [c.state_shape() for _, c in self.sublayers()]


class DapipelLM(nn.Module):
    is_hybrid = True
    has_recurrent_state = True  # the input convolutions of every layer

    def __init__(self, cfg: DapipelConfig, device=None, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.cfg = cfg
        kw = dict(device=device, dtype=dtype)
        W = cfg.hidden
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, W, **kw))
        self.pos = nn.Parameter(torch.empty(cfg.max_position_embeddings, W, **kw))
        self.layers = nn.ModuleList([DapipelLayer(cfg, s, **kw) for s in cfg.layer_specs])
        self.final_norm = nn.Parameter(torch.ones(W, device=device, dtype=torch.float32))
        with torch.no_grad():
            self.embed.normal_(0.0, 0.02)
            self.pos.normal_(0.0, 0.02)

    @property
    def dtype(self):
        return self.embed.dtype

    @property
    def position_limit(self) -> int:
        """Positions the engine may ask for (rows of the learned position table)."""
        return self.pos.shape[0]

    def head_weight(self):
        return self.embed

    def cache_kinds(self):
        """One cache entry per layer: the layer's state pools, and the mixer's paged rows where it attends."""
        out = []
        for l in self.layers:
            if l.mixer.cache_kind == "latent":
                out.append(("rows+state", (l.mixer.cache_row, l.state_shapes())))
            else:
                out.append(("state", l.state_shapes()))
        return out

    # ------------------------------------------------------------------ serving step
    def step(self, b: StepBatch, cache, rows: Optional[torch.Tensor] = None, trail: Optional[list] = None):
        """Run the step's packed tokens through all layers against the engine's cache (``cache.layer(i)``: the rows and
        the state pools of layer i).  Returns the fp32 residual stream of ``rows`` (all rows if None) after the last
        layer; ``trail`` collects it after every layer."""
        cfg, eps, dt = self.cfg, self.cfg.layer_norm_eps, self.dtype
        x = y = None
        for i, layer in enumerate(self.layers):
            entry = cache.layer(i)
            states = entry[1] if layer.mixer.cache_kind == "latent" else entry
            own = len(layer.mixer.state_shapes())
            for q, (norm, conv) in enumerate(layer.sublayers()):
                carried = states[own + q]
                if x is None:
                    x, h = hops.embed_norm_conv(self.embed, self.pos, cfg.embedding_scale, norm, cfg.norm_groups, eps,
                                                conv.tap_major(), carried, b)
                else:
                    x, h = hops.add_norm_conv(x, y, norm, cfg.norm_groups, eps, conv.tap_major(), carried, b, dt)
                y = layer.mixer.step(h, b, entry) if q == 0 else layer.ff(h)
            if trail is not None:
                trail.append(x + y.float())
        if x is None:
            x = self.embed[b.ids].float() * cfg.embedding_scale + self.pos[b.pos.long()].float()
        if rows is not None:
            x, y = x.index_select(0, rows), (y.index_select(0, rows) if y is not None else None)
        return x if y is None else x + y.float()

    def logits(self, x: torch.Tensor) -> torch.Tensor:
        _, xn = hops.group_norm_f32(x.contiguous(), None, self.final_norm, self.cfg.norm_groups, self.cfg.layer_norm_eps, self.dtype)
        return _mm_f32(xn, self.embed)

    # ------------------------------------------------------------------ checkpoint names
    @torch.no_grad()
    def load_named(self, W: Dict[str, torch.Tensor]) -> None:
        """Copy a checkpoint's tensors (its names, see the module docstring) into the fused parameters."""
        def put(dst, src):
            if tuple(dst.shape) != tuple(src.shape):
                raise ValueError(f"shape {tuple(src.shape)} does not fit {tuple(dst.shape)}")
            dst.copy_(src.to(dst.dtype))

        put(self.embed, W["embed"])
        put(self.pos, W["pos"])
        put(self.final_norm, W["final.norm"])
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            for n, (norm, conv) in enumerate(layer.sublayers(), 1):
                put(norm, W[f"{p}norm{n}"])
                put(conv.weight, W[f"{p}canon{n}"])
            m, q = layer.mixer, p + "mix."
            if isinstance(m, MinGRU):
                put(m.w_in, torch.cat([W[q + "z"], W[q + "x"], W[q + "g"]], 0))
                put(m.b_z, W[q + "z.b"])
                put(m.b_x, W[q + "x.b"])
            else:
                put(m.w_qkv, torch.cat([W[q + "q"], W[q + "k"], W[q + "v"]], 0))
                for n in ("lq1", "lk1", "lq2", "lk2"):
                    put(getattr(m, n), W[q + n])
            put(m.w_o, W[q + "o"])
            ff, f = layer.ff, p + "mlp."
            if ff is None:
                continue
            if isinstance(ff, GatedFF):
                put(ff.w_gu, torch.cat([W[f + "gate"], W[f + "up"]], 0))
                put(ff.w_down, W[f + "down"])
            else:
                put(ff.w_router, W[f + "router"])
                for e in range(ff.E):
                    put(ff.experts_up[e], torch.cat([W[f"{f}e{e}.gate"], W[f"{f}e{e}.up"]], 0))
                    put(ff.experts_down[e], W[f"{f}e{e}.down"])

    @torch.no_grad()
    def export_named(self) -> Dict[str, torch.Tensor]:
        """The inverse of :meth:`load_named`: tensors under the checkpoint's names."""
        out = {"embed": self.embed, "pos": self.pos, "final.norm": self.final_norm}
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            for n, (norm, conv) in enumerate(layer.sublayers(), 1):
                out[f"{p}norm{n}"], out[f"{p}canon{n}"] = norm, conv.weight
            m, q = layer.mixer, p + "mix."
            if isinstance(m, MinGRU):
                out[q + "z"], out[q + "x"], out[q + "g"] = m.w_in.split(m.n, 0)
                out.update({q + "z.b": m.b_z, q + "x.b": m.b_x})
            else:
                out[q + "q"], out[q + "k"], out[q + "v"] = m.w_qkv.split([2 * m.H * m.dk, 2 * m.G * m.dk, m.G * m.dv], 0)
                out.update({q + n: getattr(m, n) for n in ("lq1", "lk1", "lq2", "lk2")})
            out[q + "o"] = m.w_o
            ff, f = layer.ff, p + "mlp."
            if ff is None:
                continue
            if isinstance(ff, GatedFF):
                out[f + "gate"], out[f + "up"], out[f + "down"] = ff.w_gu[:ff.ff], ff.w_gu[ff.ff:], ff.w_down
            else:
                out[f + "router"] = ff.w_router
                for e in range(ff.E):
                    out[f"{f}e{e}.gate"], out[f"{f}e{e}.up"] = ff.w_up[e, :ff.ff], ff.w_up[e, ff.ff:]
                    out[f"{f}e{e}.down"] = ff.experts_down[e]
        return {k: v.detach().clone().contiguous() for k, v in out.items()}


def load_dapipel(ck: Path, cfg: DapipelConfig, device=None, dtype=torch.bfloat16) -> DapipelLM:
    from safetensors import safe_open

    with safe_open(str(ck / "model.safetensors"), framework="pt", device="cpu") as f:
        W = {k: f.get_tensor(k) for k in f.keys()}
    cfg.max_position_embeddings = int(W["pos"].shape[0])
    model = DapipelLM(cfg, device=device, dtype=dtype)
    model.load_named(W)
    return model


def dapipel_template(width: int = 256, layers: int = 4, heads: int = 4, kv_heads: int = 2, vocab: int = 512, every: int = 3,
                     ff: Optional[int] = None, experts: int = 0, top: int = 2, expert_ff: Optional[int] = None,
                     head_dim: Optional[int] = None, state_width: Optional[int] = None, window: int = 1024, groups: int = 4,
                     taps: int = 4, max_positions: int = 8192) -> DapipelConfig:
    """A random-init configuration for benchmarks and smoke runs: minGRU in every layer but each ``every``-th, which is
    a windowed differential attention (values of ``head_dim``, two maps of half that); dense feed-forwards, or routed
    experts when ``experts`` > 0."""
    d = head_dim or width // heads
    att = {"heads": heads, "kv_heads": kv_heads, "dim": max(d // 2, 1), "vdim": d, "scale": max(d // 2, 1) ** -0.5, "diff": 0.5,
           "mask": {"size": window}}
    rec = {"width": state_width or width}
    if experts:
        mlp = {"kind": "moe", "expert": {"ff": expert_ff or width // 2}, "router": {"experts": experts, "top": top}}
    else:
        mlp = {"kind": "dense", "ff": ff or 2 * width}
    specs = [{"type": "attention" if (i + 1) % every == 0 else "mingru",
              "mixer": copy.deepcopy(att if (i + 1) % every == 0 else rec), "mlp": copy.deepcopy(mlp)} for i in range(layers)]
    return DapipelConfig(name=f"dapipel-w{width}-l{layers}", vocab_size=vocab, hidden=width, layer_specs=specs,
                         layer_norm_eps=1e-5, norm_groups=groups, taps=taps, embedding_scale=float(width) ** 0.5,
                         max_position_embeddings=max_positions)
