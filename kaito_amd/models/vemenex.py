"""Vemenex: a stack of hyper-connected layers served by the paged engine.

The stack carries S copies ("streams") of the residual row, equal to the
RMS-normed token embedding at the start. Every sub-layer f (a mixer, then a
feed-forward where the layer has one) reads one weighted sum of the streams
and writes back through a matrix:

    u = Σ_s in_s·x_s;   y = f(rms(u)·g);   x_t ← Σ_s mix_{s,t}·x_s + m·out_t·y

with a single number g as the norm's weight and m the model's residual
factor (folded into `out` at load). Streams are f32, [tokens, S, width];
sub-layers see their input rounded to the activation dtype. Mixers
(models/mixers.py RotaryWindowAttention, q and k plainly normed behind the
rotation): "attention" weighs keys by sigmoid(score + a per-head bias) and
rotates neighbouring dimensions; "attention_2" is a softmax with a unit
sink, a rotation of halves and a gate per head. The feed-forward is a relu
GatedFF or the engine's MoEMLP (clamped-GLU experts beside identity
experts, group-limited softmax routing with a choice correction).

Output: the sum of the streams, the model's norm, a head of its own.

A sub-layer's write is fused with the next one's read and norm
(ops.stream_mix_norm), so a layer receives its normed input and is told
which connection reads next; the embedding, its norm, the copies and the
first read are one step (ops.stream_embed).
"""
from __future__ import annotations

import math
from typing import List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..engine.config import ModelConfig
from .hybrid_base import HybridStackBase, MixerLayerBase, f32_vector
from .hybrid_config import LayerSpec, layer_moe_config
from .mixers import GatedFF, RotaryWindowAttention
from .moe import MoEMLP


class StreamConnection(nn.Module):
    """How one sub-layer reads from and writes to the streams."""

    def __init__(self, streams: int):
        super().__init__()
        self.norm = f32_vector(1)
        self.w_in = f32_vector(streams)
        self.w_out = f32_vector(streams)          # times the residual factor
        self.mix = nn.Parameter(torch.empty(streams, streams,
                                            dtype=torch.float32),
                                requires_grad=False)      # [from, to]


class VemenexLayer(MixerLayerBase):
    def __init__(self, cfg: ModelConfig, spec: LayerSpec):
        super().__init__()
        self.cfg, self.spec = cfg, spec
        h, dt = cfg.hidden_size, cfg.dtype
        if spec.kind not in ("attention", "attention_2"):
            raise ValueError(spec.kind)
        self.attn = RotaryWindowAttention(h, spec.rattn, dt, cfg.rms_eps)
        self.hc1 = StreamConnection(cfg.residual_streams)
        self.mlp = self.hc2 = None
        if spec.glu is not None:
            self.mlp = GatedFF(h, spec.glu, dt)
        elif spec.moe is not None:
            self.mlp = MoEMLP(layer_moe_config(cfg, spec.moe))
        if self.mlp is not None:
            self.hc2 = StreamConnection(cfg.residual_streams)

    def mixers(self):
        return [self.attn]

    def connections(self) -> List[StreamConnection]:
        return [c for c in (self.hc1, self.hc2) if c is not None]

    def feed_forward(self, h):
        if isinstance(self.mlp, MoEMLP):
            return self.mlp(h, keep_f32=True)
        return self.mlp(h)


class VemenexForCausalLM(HybridStackBase):
    def __init__(self, cfg: ModelConfig):
        super().__init__(cfg)
        assert cfg.residual_streams >= 1
        self.embed_tokens = nn.Embedding(cfg.vocab_size, cfg.hidden_size,
                                         dtype=cfg.dtype)
        self.embed_tokens.weight.requires_grad_(False)
        self.embed_norm = f32_vector(1)
        self.layers = nn.ModuleList(
            [VemenexLayer(cfg, s) for s in cfg.layer_specs])
        self.norm = f32_vector(cfg.hidden_size)   # one number, repeated
        self.lm_head = nn.Parameter(
            torch.empty(cfg.vocab_size, cfg.hidden_size, dtype=cfg.dtype),
            requires_grad=False)
        # the stack's output reads every stream with weight one
        self.register_buffer("ones", torch.ones(
            cfg.residual_streams, dtype=torch.float32), persistent=False)

    def decode_graph_capturable(self) -> bool:
        """True when no decode-step op reads device data on the host: the
        routed layers must take the fused grouped-GEMM path."""
        return all(
            not isinstance(layer.mlp, MoEMLP) or (
                self.cfg.dtype == torch.bfloat16
                and self.cfg.hidden_size % 64 == 0
                and layer.mlp.ie_local % 64 == 0)
            for layer in self.layers)

    def _connect(self, x, y, c: StreamConnection,
                 nxt: Optional[StreamConnection]):
        """Sub-layer output y into the streams; the next sub-layer's input,
        or after the last one the sum of the streams (f32)."""
        eps = self.cfg.rms_eps
        if nxt is None:
            return ops.stream_mix_norm(
                x, y, c.mix, c.w_out, self.ones, None, eps, torch.float32,
                write_x=self.layer_hook is not None)
        return ops.stream_mix_norm(x, y, c.mix, c.w_out, nxt.w_in, nxt.norm,
                                   eps, self.cfg.dtype)

    def forward(self, input_ids, positions, kv_caches, meta,
                hidden_in=None) -> torch.Tensor:
        layers = list(self.layers)
        first = layers[0].hc1
        x, h = ops.stream_embed(input_ids, self.embed_tokens.weight,
                                self.embed_norm, first.w_in, first.norm,
                                self.cfg.rms_eps)
        for i, layer in enumerate(layers):
            after = layers[i + 1].hc1 if i + 1 < len(layers) else None
            y = layer.attn(h, positions, layer._view(kv_caches[i],
                                                     layer.attn), meta)
            h = self._connect(x, y, layer.hc1, layer.hc2 or after)
            if layer.mlp is not None:
                h = self._connect(x, layer.feed_forward(h), layer.hc2, after)
            if self.layer_hook is not None:
                self.layer_hook(i, x.sum(1))
        return h

    # ---- weights ----------------------------------------------------------
    @torch.no_grad()
    def random_init(self, seed: int = 0):
        """Random weights of the right shapes with magnitudes that keep
        every mechanism active."""
        dev = self.norm.device
        gen = torch.Generator(device=dev).manual_seed(seed)

        def normal(p, std, mean=0.0):
            t = torch.empty(p.shape, dtype=torch.float32, device=dev)
            t.normal_(mean, std, generator=gen)
            p.copy_(t.to(p.dtype))

        def uniform(p, lo, hi):
            t = torch.empty(p.shape, dtype=torch.float32, device=dev)
            t.uniform_(lo, hi, generator=gen)
            p.copy_(t.to(p.dtype))

        S, m = self.cfg.residual_streams, self.cfg.residual_mult
        for name, p in self.named_parameters():
            last = name.split(".")[-1]
            if last in ("norm", "embed_norm"):
                uniform(p, 0.8, 1.2)
            elif last == "w_in":
                uniform(p, 0.5 / S, 1.5 / S)
            elif last == "w_out":
                uniform(p, 0.5 * m, 1.5 * m)
            elif last == "mix":
                normal(p, 0.1 / S)
                p.add_(torch.eye(S, device=dev) * 0.9)
            elif last == "score_bias":
                normal(p, 0.5, -3.0)
            elif last == "e_score_correction_bias":
                normal(p, 0.05)
            else:
                normal(p, 1.0 / math.sqrt(p.shape[-1]))
        return self
