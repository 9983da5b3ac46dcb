"""Fanotar: a layered decoder whose norms are elementwise (dynamic tanh) and stand on both sides of each sublayer.

Every norm of the model is D(v) = tanh(alpha v) * w + b with a scalar alpha (tensors ``<name>``, ``<name>.b``,
``<name>.alpha``); it has no statistics.  ``config.json`` lists the layers; each has one sequence mixer and
optionally one feed-forward:

    x <- x + D1b(mixer(D1(x)));      x <- x + D2b(ff(D2(x)))

from x = D_embed(embed[token] * embedding.scale); the model ends with D_final and the ``head`` projection.

The mixer type ``attention`` is :class:`.mixers.ConvAttentionMixer`: short convolutions on q, k and v, normed q
and k, a query temperature, a distance bias, a sliding window, a softmax sink, an elementwise output gate; a
layer with ``kv_from`` uses an earlier layer's cached keys and values.  Feed-forwards: the clamped gated unit,
dense, or as a mixture of experts (sigmoid scores, choice by score + correction, weights renormalised over the
chosen and scaled) with a shared expert.

The residual stream is f32 whatever the activation dtype; one kernel norms a sublayer's output into the
stream and the stream into the next sublayer's input (:func:`..ops.mixers.dyn_tanh_residual`), the embedding
gather does the same for the first layer, and a mixer's projections (q | k | v | gate) are one stacked GEMM.

Checkpoint tensors: ``embed``, ``embed.norm``, ``l<i>.norm1``, ``l<i>.norm1b``, ``l<i>.norm2``, ``l<i>.norm2b``,
``l<i>.mix.<name>``, ``l<i>.mlp.<name>``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from typing import Dict

import torch
import torch.nn.functional as F

from ..ops import mixers as mx
from .common import AttentionMetadata, HybridCache
from .configs import ModelConfig
from .layered import Layer, LayeredDecoder
from .mixers import DenseFF, RoutedFF


def example_config(width: int = 160, vocab: int = 704, pattern: str = "AEkK", scale_up: bool = False,
                   heads: int = 0) -> Dict:
    """A config.json-shaped dict for random-weight models (tests, benchmarks).  ``pattern``: one letter per layer --
    a/A attention without a feed-forward / with a dense one, e/E with a routed one without / with a shared expert, k/K
    like A / E but on the keys and values of the last layer before it that has its own.  ``scale_up``: sizes
    in the range of a real model's layers."""
    if scale_up:
        H = heads or width // 128
        att = {"conv": 4, "dim": 128, "heads": H, "kv_heads": max(H // 4, 1), "mask": {"size": 1024},
               "q_temp": {"coef": 0.1, "every": 1024}, "scale": 128 ** -0.5, "vdim": 128}
        dense = {"ff": 3 * width, "kind": "dense", "limit": 7.0}
        moe = {"expert": {"ff": width // 2, "limit": 7.0}, "kind": "moe", "router": {"experts": 32, "scale": 2.5, "top": 4}}
        shared = {"ff": width, "limit": 7.0}
    else:
        att = {"conv": 3, "dim": 24, "heads": 6, "kv_heads": 2, "mask": {"size": 37},
               "q_temp": {"coef": 0.4, "every": 11}, "scale": 0.3, "vdim": 20}
        dense = {"ff": 224, "kind": "dense", "limit": 1.7}
        moe = {"expert": {"ff": 56, "limit": 1.2}, "kind": "moe", "router": {"experts": 7, "scale": 1.8, "top": 3}}
        shared = {"ff": 40, "limit": 0.9}
    layers, own = [], None
    for i, ch in enumerate(pattern):
        m = {k: (dict(v) if isinstance(v, dict) else v) for k, v in att.items()}
        if ch in "kK":
            m["kv_from"] = own
        else:
            own = i
        if ch == "a":
            mlp = None
        elif ch in "Ak":
            mlp = dict(dense)
        else:
            mlp = {k: (dict(v) if isinstance(v, dict) else v) for k, v in moe.items()}
            if ch in "EK":
                mlp["shared"] = dict(shared)
        layers.append({"type": "attention", "mixer": m, "mlp": mlp})
    return {"architecture": "Fanotar", "embedding": {"scale": 3.0}, "layers": layers, "norm": {"eps": 1e-5}, "vocab": vocab,
            "width": width}


class _Layer(Layer):
    def __init__(self, i: int, spec: Dict, width: int, eps: float):
        super().__init__(i, spec, width, eps, FanotarModel.mixer_types)
        mlp = spec.get("mlp")
        if mlp is None:
            self.ff = None
        elif mlp["kind"] == "dense":
            self.ff = DenseFF(mlp, width, act="clamped", gated=True)
        elif mlp["kind"] == "moe":
            self.ff = RoutedFF(mlp, width, score="sigmoid", renorm=True)
        else:
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
        self.width = width
        self.w_ff = None
        self.dt = {}             # norm name -> mx.DynTanh

    def norms(self):
        return ("norm1", "norm1b", "norm2", "norm2b") if self.ff is not None else ("norm1", "norm1b")

    def extra_shapes(self) -> Dict[str, tuple]:
        s = {}
        for n in self.norms():
            s.update({f"{n}.b": (self.width,), f"{n}.alpha": ()})
        return s


class FanotarModel(LayeredDecoder):
    arch = "fanotar"
    mixer_types = {"attention": "conv_attention"}

    def __init__(self, cfg: ModelConfig, device="cuda", dtype=torch.bfloat16):
        super().__init__(cfg, device, dtype)
        self.has_state = any(l.mixer.taps > 1 for l in self.layers)
        self.embed_scale = float((cfg.embedding or {}).get("scale", 1.0))
        for i, l in enumerate(self.layers):
            m, j = l.mixer, l.mixer.kv_from
            if j is None:
                continue
            src = self.layers[j].mixer if 0 <= j < i else None
            if src is None or src.kv_from is not None or (src.H, src.G, src.D, src.P) != (m.H, m.G, m.D, m.P):
                raise ValueError(f"{cfg.name}: layer {i}: kv_from must name an earlier layer with keys and values of "
                                 "its own and the same head counts and sizes")

    def make_layer(self, i: int, spec: Dict) -> Layer:
        return _Layer(i, spec, self.cfg.hidden_size, self.cfg.norm_eps)

    def extra_shapes(self) -> Dict[str, tuple]:
        W = self.cfg.hidden_size
        return {"embed.norm": (W,), "embed.norm.b": (W,), "embed.norm.alpha": (), "final.norm.b": (W,), "final.norm.alpha": ()}

    @staticmethod
    def _dyn_tanh(get, name: str) -> mx.DynTanh:
        return mx.DynTanh(float(get(name + ".alpha").float().item()), get(name).float().contiguous(),
                          get(name + ".b").float().contiguous())

    def load_layer(self, l: Layer, get) -> None:
        dt = self.dtype
        l.dt = {n: self._dyn_tanh(get, f"{l.prefix}.{n}") for n in l.norms()}
        l.w_in = l.mixer.load(lambda k, p=l.prefix: get(f"{p}.mix.{k}"), dt).contiguous()
        if l.ff is not None:
            w = l.ff.load(lambda k, p=l.prefix: get(f"{p}.mlp.{k}"), dt)
            l.w_ff = w.contiguous() if w is not None else None

    def load_extra(self, get) -> None:
        self.embed_dt = self._dyn_tanh(get, "embed.norm")
        self.final_dt = self._dyn_tanh(get, "final.norm")

    # -- forward -----------------------------------------------------------------------------------
    def forward(self, ids: torch.Tensor, positions: torch.Tensor, meta: AttentionMetadata, kv: HybridCache) -> torch.Tensor:
        """Final-normed hidden states [T, width] of every row of the step."""
        dt = self.dtype
        if meta.seg_cu is None:
            raise ValueError("this model needs the segment view of the step (AttentionMetadata.seg_*)")
        n = len(self.layers)
        x, h = mx.dyn_tanh_embed(ids, self.embed, self.embed_scale, self.embed_dt, self.layers[0].dt["norm1"], dt)
        for i, l in enumerate(self.layers):
            m = l.mixer
            y = m.forward(F.linear(h, l.w_in), positions, meta, kv.layers[i],
                          kv_cache=kv.layers[m.kv_from] if m.kv_from is not None else None)
            nxt = self.layers[i + 1].dt["norm1"] if i + 1 < n else self.final_dt
            # the norm of this sublayer's output, the residual sum and the norm of what comes next: one pass
            h = mx.dyn_tanh_residual(x, y, l.dt["norm1b"], l.dt["norm2"] if l.ff is not None else nxt, dt)
            if l.ff is not None:
                y = l.ff.forward(h, F.linear(h, l.w_ff) if l.w_ff is not None else None)
                h = mx.dyn_tanh_residual(x, y, l.dt["norm2b"], nxt, dt)
            if self.capture is not None:
                self.capture.append(x.clone())
        return h
