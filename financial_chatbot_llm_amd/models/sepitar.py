"""Sepitar: a looped layered decoder of parallel blocks with three kinds of attention.

``config.json`` lists the layers; each has one sequence mixer and optionally one routed feed-forward, both reading the
SAME normed input:

    h = RMSnorm(x) * (1 + w_norm1);   x <- x + (mixer(h) + ff(h))

With a ``loop`` entry {start, stop, times} the layers start .. stop - 1 run ``times`` times in a row with the same
weights, each pass with its own cache; before every pass but the first the embedding output is added to x once more.
The model ends with RMSnorm * (1 + ``final.norm``) and the ``head`` projection.

Mixer types: ``attention`` is :class:`.mixers.RelBiasAttentionMixer` (biased projections, logarithmic distance bias,
sliding window, elementwise gate), ``attention_2`` :class:`.mixers.CappedAttentionMixer` (whole-projection norms,
rotation scaled by wavelength, soft cap, sink, gate per head), ``latent_attention``
:class:`.mixers.SinkLatentAttentionMixer` (interleaved rotation with a ramped scaling, sliding window, sink).
Feed-forward: clamped gated experts, the softmax over the chosen biased logits as weights, a shared expert.

The residual stream is f32 whatever the activation dtype; each block's update, the embedding output that enters before
a repeated pass and the next block's norm are one pass over x (:func:`..ops.mixers.residual_norm`), and the mixer's and
the shared expert's input projections are one stacked GEMM.

Checkpoint tensors: ``embed``, ``l<i>.norm1``, ``l<i>.mix.<name>``, ``l<i>.mlp.<name>``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from typing import Dict

import torch
import torch.nn.functional as F

from ..ops import mixers as mx
from .common import AttentionMetadata, HybridCache
from .configs import ModelConfig
from .layered import Layer, LayeredDecoder
from .mixers import RoutedFF


def example_config(width: int = 160, vocab: int = 736, pattern: str = "LRC", scale_up: bool = False, heads: int = 0,
                   loop=(0, 2, 2)) -> Dict:
    """A config.json-shaped dict for random-weight models (tests, benchmarks).  ``pattern``: one letter per layer --
    l/L latent attention, r/R attention with the distance bias, c/C soft-capped attention; upper case with a routed
    feed-forward and a shared expert, lower case without a feed-forward.  ``loop``: (start, stop, times) or None.
    ``scale_up``: sizes in the range of a real model's layers."""
    if scale_up:
        H = heads or width // 128
        G = max(H // 4, 1)
        lat = {"dim": 96, "heads": H, "kv_rank": 256, "mask": {"size": 1024}, "q_rank": 768,
               "rot": {"base": 10000.0, "dims": 32, "scaling": {"factor": 4.0, "fast": 32.0, "original": 4096, "slow": 1.0}},
               "rot_dim": 32, "scale": 128 ** -0.5, "vdim": 96}
        rel = {"bias_max": 1024, "buckets": 32, "dim": 128, "heads": H, "kv_heads": G, "mask": {"size": 1024}, "scale": 128 ** -0.5,
               "vdim": 128}
        cap = {"dim": 128, "heads": H, "kv_heads": G, "rot": {"base": 500000.0, "dims": 128, "scaling": {
            "factor": 8.0, "high": 4.0, "low": 1.0, "original": 8192}}, "scale": 128 ** -0.5, "softcap": 30.0, "vdim": 128}
        moe = {"expert": {"ff": width // 2, "limit": 7.0}, "kind": "moe", "router": {"experts": 32, "top": 4},
               "shared": {"ff": width, "limit": 7.0}}
    else:
        lat = {"dim": 24, "heads": 3, "kv_rank": 40, "mask": {"size": 21}, "q_rank": 56,
               "rot": {"base": 10000.0, "dims": 8, "scaling": {"factor": 3.0, "fast": 8.0, "original": 128, "slow": 0.5}},
               "rot_dim": 8, "scale": 0.2, "vdim": 20}
        rel = {"bias_max": 30, "buckets": 12, "dim": 24, "heads": 6, "kv_heads": 2, "mask": {"size": 37}, "scale": 0.25, "vdim": 20}
        cap = {"dim": 32, "heads": 4, "kv_heads": 2, "rot": {"base": 1000.0, "dims": 24, "scaling": {
            "factor": 5.0, "high": 6.0, "low": 1.5, "original": 96}}, "scale": 0.3, "softcap": 4.0, "vdim": 28}
        moe = {"expert": {"ff": 40, "limit": 1.2}, "kind": "moe", "router": {"experts": 7, "top": 3},
               "shared": {"ff": 56, "limit": 0.8}}
    copy = lambda d: {k: (copy(v) if isinstance(v, dict) else v) for k, v in d.items()}  # noqa: E731
    kinds = {"l": ("latent_attention", lat), "r": ("attention", rel), "c": ("attention_2", cap)}
    layers = [{"type": kinds[ch.lower()][0], "mixer": copy(kinds[ch.lower()][1]), "mlp": copy(moe) if ch.isupper() else None}
              for ch in pattern]
    c = {"architecture": "Sepitar", "layers": layers, "norm": {"eps": 1e-5}, "vocab": vocab, "width": width}
    if loop:
        c["loop"] = {"start": loop[0], "stop": min(loop[1], len(layers)), "times": loop[2]}
    return c


class _Layer(Layer):
    def __init__(self, i: int, spec: Dict, width: int, eps: float):
        super().__init__(i, spec, width, eps, SepitarModel.mixer_types)
        mlp = spec.get("mlp")
        if mlp is not None and mlp["kind"] != "moe":
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
        self.ff = RoutedFF(mlp, width, score="softmax_top") if mlp is not None else None
        self.in_bias = None


class SepitarModel(LayeredDecoder):
    arch = "sepitar"
    mixer_types = {"attention": "rel_bias_attention", "attention_2": "capped_attention",
                   "latent_attention": "sink_latent_attention"}
    has_state = False            # every mixer's memory is paged rows
    loops = True
    norm_offset = 1.0            # norm weights are stored around zero

    def make_layer(self, i: int, spec: Dict) -> Layer:
        return _Layer(i, spec, self.cfg.hidden_size, self.cfg.norm_eps)

    def load_layer(self, l: Layer, get) -> None:
        dt = self.dtype
        l.norm1 = (get(l.prefix + ".norm1").float() + self.norm_offset).contiguous()
        parts = [l.mixer.load(lambda k, p=l.prefix: get(f"{p}.mix.{k}"), dt)]
        if l.ff is not None:
            w = l.ff.load(lambda k, p=l.prefix: get(f"{p}.mlp.{k}"), dt)
            if w is not None:
                parts.append(w)
        l.w_in = torch.cat(parts, 0).contiguous()         # ONE in-projection per block
        bias = l.mixer.in_bias
        l.in_bias = F.pad(bias, (0, l.w_in.shape[0] - bias.shape[0])).contiguous() if bias is not None else None

    # -- forward -----------------------------------------------------------------------------------
    def forward(self, ids: torch.Tensor, positions: torch.Tensor, meta: AttentionMetadata, kv: HybridCache) -> torch.Tensor:
        """Final-normed hidden states [T, width] of every row of the step."""
        eps, dt = self.cfg.norm_eps, self.dtype
        if meta.seg_cu is None:
            raise ValueError("this model needs the segment view of the step (AttentionMetadata.seg_*)")
        runs = self.runs
        x, h = mx.embed_norm(ids, self.embed, self.layers[runs[0].layer].norm1, eps, dt)
        for r, run in enumerate(runs):
            l = self.layers[run.layer]
            proj = F.linear(h, l.w_in, l.in_bias)
            nm = l.mixer.in_rows
            a = l.mixer.forward(proj[:, :nm], positions, meta, kv.layers[r])
            b = l.ff.forward(h, proj[:, nm:]) if l.ff is not None else None
            nxt = runs[r + 1] if r + 1 < len(runs) else None
            w = self.layers[nxt.layer].norm1 if nxt is not None else self.final_norm
            again = nxt is not None and nxt.again         # the embedding output enters before a repeated pass
            if self.capture is not None:
                mx.residual_norm(x, None, eps, a, b)
                self.capture.append(x.clone())
                a = b = None
            h = mx.residual_norm(x, w, eps, a, b, out_dtype=dt, ids=ids if again else None, table=self.embed if again else None)
        return h
