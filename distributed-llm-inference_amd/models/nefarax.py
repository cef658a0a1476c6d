"""Nefarax: a decoder-only stack of single-norm layers (``models/mixers.py``: ``SingleNormLayer``).

Every layer reads one norm of the fp32 stream — ``tanh(α x) · w + b``, no statistics — with its mixer and its feed-forward
side by side; ``residual_mult`` times their sum is added back.  Mixers: ``delta`` (gated delta rule), ``mlstm`` (matrix memory
with exponential gating) and ``parallel`` (causal attention with convolved q / k, keys as values and a sink, beside a Mamba-2
recurrence; both outputs RMS-normed and averaged).  The feed-forward is a plain tanh-GELU one or absent.  The same kind of
norm and the embedding table as LM head close the stack.

The configuration comes from the checkpoint's ``config.json`` (``config.nefarax_config``).  Checkpoint tensors: ``embed``,
``final.norm{,.b,.alpha}``, and per layer ``l<i>.norm1{,.b,.alpha}``, ``l<i>.mix.*`` (``parallel``: ``l<i>.mix.left.*`` and
``l<i>.mix.right.*``), ``l<i>.mlp.{up,down}``.  All projections that read the norm are fused into one GEMM, the output
projections of mixer and feed-forward into one over their concatenated inputs.
"""
from __future__ import annotations

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops
from ..config import KV_BLOCK_SIZE, ModelConfig
from ..parallel.state import ParallelContext
from .layers import Weight
from .mixers import SingleNormLayer, TanhNorm


class NefaraxForCausalLM(nn.Module):
    def __init__(self, cfg: ModelConfig, ctx: ParallelContext, dtype, device):
        super().__init__()
        if ctx.tp_size != 1:
            raise NotImplementedError("Nefarax stacks run on one GPU per replica (no tensor-parallel sharding of the mixers)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise TypeError(f"Nefarax runs in bfloat16 or float32, not {dtype}")
        self.cfg, self.ctx, self.dtype = cfg, ctx, dtype
        W = cfg.hidden_size
        self.embed = Weight((cfg.vocab_size, W), None, ctx, dtype, device)          # also the LM head
        self.layers = nn.ModuleList(SingleNormLayer(s, W, cfg.rms_eps, ctx, dtype, device) for s in cfg.layer_specs)
        self.final_norm = TanhNorm(W, ctx, device)
        self.layer_outputs = None          # a list: the stream after every layer is appended (tests, debugging)

    # ---- cache: pages of the attention halves; recurrent state, convolution inputs and running maxima per state slot
    def allocate_caches(self, num_blocks: int, num_slots: int, device):
        return [l.cache(num_blocks, num_slots, self.dtype, device) for l in self.layers]

    def bytes_per_block(self) -> int:
        item = torch.empty((), dtype=self.dtype).element_size()
        return max(sum(sum(s.cache_row) for s in self.cfg.layer_specs) * KV_BLOCK_SIZE * item, 1)      # 1: no attention layer

    def bytes_per_slot(self) -> int:
        return sum(t.numel() * t.element_size() for l in self.layers for t in l.cache(0, 1, self.dtype, "meta").state_tensors())

    def forward(self, input_ids: torch.Tensor, meta, caches) -> torch.Tensor:
        cfg = self.cfg
        x = F.embedding(input_ids, self.embed.data).float()
        pending = None                     # the previous layer's output, added by the next norm's pass over the stream
        for layer, cache in zip(self.layers, caches):
            h = layer.norm1.read(x, pending, cfg.residual_mult, cfg.rms_eps, self.dtype)
            if self.layer_outputs is not None and pending is not None:
                self.layer_outputs.append(x.clone())
            pending = layer(h, meta, cache)
        h = self.final_norm.read(x, pending, cfg.residual_mult, cfg.rms_eps, self.dtype)
        if self.layer_outputs is not None:
            self.layer_outputs.append(x.clone())
        return h

    def compute_logits(self, h: torch.Tensor) -> torch.Tensor:
        return ops.linear(h, self.embed.data).float()

    # ---- parameters: (name, holder, init kind, checkpoint tensors: concatenated along dim 0, or — behind "@cols" — along dim 1)
    def named_weight_sources(self):
        yield "embed", self.embed, "normal", None
        for i, l in enumerate(self.layers):
            yield from l.weights(f"l{i}.")
        yield from self.final_norm.weights("final.norm")

    def named_weights(self):
        for name, w, kind, _src in self.named_weight_sources():
            yield name, w, kind

    def checkpoint_sources(self) -> dict:
        return {name: src for name, _w, _k, src in self.named_weight_sources() if src}
