"""Labirax: a sandwich-normed stack of unlike mixers served by the paged
engine.

Every sub-layer f (a mixer, then a feed-forward where the layer has one) has
a layer norm with weight and bias on both sides:

    x ← x + ln_b(f(ln_a(x)))

The stream x is f32; sub-layers see their normed input rounded to the
activation dtype. Mixers (models/mixers.py): GLAMixer (gated linear
attention with a decay per key channel), LatentAttention (low-rank queries,
a sliding window, an output gate per value dimension) and
RotaryWindowAttention without a rotation (a learned bias per head and
distance, a query temperature, biases on q/k/v). The feed-forward is the
engine's MoEMLP: softmax routing over all experts, renormalised weights, an
always-on shared expert.

A layer may run on an earlier layer's weights; every run keeps caches and
states of its own. Output: the model's layer norm, a head of its own, then
the logits scaled and soft-capped.

The norm behind a sub-layer, the residual sum and the norm ahead of the next
one are one step (ops.sandwich_norm_residual), so a layer receives its
normed input and is told which norm comes next; the embedding and the first
norm are one step too (ops.embed_layer_norm).
"""
from __future__ import annotations

import math
from typing import Dict, Optional

import torch
import torch.nn as nn

from .. import ops
from ..engine.config import ModelConfig
from .hybrid_base import HybridStackBase, MixerLayerBase, f32_vector
from .hybrid_config import LayerSpec, layer_moe_config
from .mixers import GLAMixer, LatentAttention, RotaryWindowAttention
from .moe import MoEMLP


class LayerNormWeights(nn.Module):
    def __init__(self, width: int):
        super().__init__()
        self.weight = f32_vector(width)
        self.bias = f32_vector(width)


class LabiraxLayer(MixerLayerBase):
    def __init__(self, cfg: ModelConfig, spec: LayerSpec):
        super().__init__()
        self.cfg, self.spec = cfg, spec
        h, eps, dt = cfg.hidden_size, cfg.rms_eps, cfg.dtype
        if spec.kind == "gla":
            self.mixer = GLAMixer(h, spec.gla, dt, eps)
        elif spec.kind == "latent_attention":
            self.mixer = LatentAttention(h, spec.latent, dt, eps)
        elif spec.kind == "attention":
            self.mixer = RotaryWindowAttention(h, spec.rattn, dt, eps)
        else:
            raise ValueError(spec.kind)
        self.norm1, self.norm1b = LayerNormWeights(h), LayerNormWeights(h)
        self.mlp = self.norm2 = self.norm2b = None
        if spec.moe is not None:
            self.mlp = MoEMLP(layer_moe_config(cfg, spec.moe))
            self.norm2, self.norm2b = LayerNormWeights(h), LayerNormWeights(h)

    def mixers(self):
        return [self.mixer]

    def norms(self) -> Dict[str, LayerNormWeights]:
        return {n: getattr(self, n)
                for n in ("norm1", "norm1b", "norm2", "norm2b")
                if getattr(self, n) is not None}

    def _close(self, x32, y, norm: LayerNormWeights,
               nxt: Optional[LayerNormWeights], y2=None):
        """Sub-layer output y (+ y2) normed into the stream; the next
        sub-layer's input (None after the last)."""
        return ops.sandwich_norm_residual(
            x32, y, norm.weight, norm.bias,
            nxt.weight if nxt is not None else None,
            nxt.bias if nxt is not None else None, self.cfg.rms_eps,
            self.cfg.dtype, y2=y2)

    def forward(self, x32, h, positions, cache, meta, next_norm):
        y = self.mixer(h, positions, self._view(cache, self.mixer), meta)
        if self.mlp is None:
            return self._close(x32, y, self.norm1b, next_norm)
        h = self._close(x32, y, self.norm1b, self.norm2)
        y, shared = self.mlp(h, keep_f32=True, split_shared=True)
        return self._close(x32, y, self.norm2b, next_norm, shared)


class LabiraxForCausalLM(HybridStackBase):
    kernel_groups = ("lnorm", "mix", "latent", "diag", "route", "moe", "core")

    def __init__(self, cfg: ModelConfig):
        super().__init__(cfg)
        self.embed_tokens = nn.Embedding(cfg.vocab_size, cfg.hidden_size,
                                         dtype=cfg.dtype)
        self.embed_tokens.weight.requires_grad_(False)
        specs = cfg.layer_specs
        # the layers that have weights, and for every run the one it uses
        self.layer_ids = [i for i, s in enumerate(specs)
                          if s.weights_of is None]
        self.layers = nn.ModuleList(
            [LabiraxLayer(cfg, specs[i]) for i in self.layer_ids])
        self.runs = [self.layer_ids.index(
            i if s.weights_of is None else s.weights_of)
            for i, s in enumerate(specs)]
        self.norm = LayerNormWeights(cfg.hidden_size)
        self.lm_head = nn.Parameter(
            torch.empty(cfg.vocab_size, cfg.hidden_size, dtype=cfg.dtype),
            requires_grad=False)

    def run_layers(self):
        return [self.layers[r] for r in self.runs]

    def decode_graph_capturable(self) -> bool:
        """True when no decode-step op reads device data on the host: the
        routed layers must take the fused grouped-GEMM path."""
        return all(
            layer.mlp is None or (
                self.cfg.dtype == torch.bfloat16
                and self.cfg.hidden_size % 64 == 0
                and layer.mlp.ie_local % 64 == 0)
            for layer in self.layers)

    def forward(self, input_ids, positions, kv_caches, meta,
                hidden_in=None) -> torch.Tensor:
        cfg, order = self.cfg, self.run_layers()
        first = order[0].norm1
        x32, h = ops.embed_layer_norm(
            input_ids, self.embed_tokens.weight, cfg.embed_scale,
            first.weight, first.bias, cfg.rms_eps)
        for j, layer in enumerate(order):
            nxt = order[j + 1].norm1 if j + 1 < len(order) else None
            h = layer(x32, h, positions, kv_caches[j], meta, nxt)
            if self.layer_hook is not None:
                self.layer_hook(j, x32)
        return x32

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        cfg = self.cfg
        h = ops.layer_norm_cast(hidden.contiguous(), self.norm.weight,
                                self.norm.bias, cfg.rms_eps, cfg.dtype)
        return ops.scaled_softcap(ops.linear_f32(h, self.lm_head),
                                  cfg.logit_scale, cfg.final_logit_softcap)

    # ---- weights ----------------------------------------------------------
    @torch.no_grad()
    def random_init(self, seed: int = 0):
        """Random weights of the right shapes with magnitudes that keep
        every mechanism active (decays away from 0 and 1, gates open)."""
        dev = self.lm_head.device
        gen = torch.Generator(device=dev).manual_seed(seed)

        def normal(p, std, mean=0.0):
            t = torch.empty(p.shape, dtype=torch.float32, device=dev)
            t.normal_(mean, std, generator=gen)
            p.copy_(t.to(p.dtype))

        def uniform(p, lo, hi):
            t = torch.empty(p.shape, dtype=torch.float32, device=dev)
            t.uniform_(lo, hi, generator=gen)
            p.copy_(t.to(p.dtype))

        for name, p in self.named_parameters():
            last = name.split(".")[-1]
            if last in ("weight", "out_norm", "kv_norm", "q_norm") \
                    and "embed" not in name:
                uniform(p, 0.8, 1.2)
            elif last == "bias":
                normal(p, 0.1)
            elif last in ("qkv_bias", "dist_bias"):
                normal(p, 0.5)
            elif last == "a_bias":
                normal(p, 1.0, 2.0)
            elif last == "a2":                       # [in, out]
                normal(p, 1.0 / math.sqrt(p.shape[0]))
            elif "embed" in name:
                normal(p, 0.5 / max(self.cfg.embed_scale, 1.0))
            else:
                normal(p, 1.0 / math.sqrt(p.shape[-1]))
        return self
