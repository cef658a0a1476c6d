"""Mozalix: a decoder-only stack of post-norm layers (``models/mixers.py``: ``PostNormLayer``).

Mixer and feed-forward read the fp32 stream itself and add an RMS norm (``1 + w``) of their output.  Mixers: ``attention`` (chunked,
per-head q / k norm, partial rotation, a sink), ``attention_2`` (differential attention over a sliding window) and ``parallel``
(soft-capped window attention with kept first tokens and without positions, beside a gated delta rule with a decay per key
channel).  The feed-forward is clamped, with biases, or absent.  A layer with ``weights_of`` runs on another layer's parameters with
a cache and state of its own.  The norm of the stream and an LM head close the stack; embedding rows are scaled.

The configuration comes from the checkpoint's ``config.json`` (``config.mozalix_config``).  Checkpoint tensors: ``embed``, ``head``,
``final.norm``, and per layer with parameters of its own ``l<i>.norm{1,2}``, ``l<i>.mix.*`` (``parallel``: ``l<i>.mix.left.*`` and
``l<i>.mix.right.*``), ``l<i>.mlp.{gate,up,down}(.b)``.
"""
from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from ..config import KV_BLOCK_SIZE, ModelConfig
from ..ops import seqmix
from ..parallel.state import ParallelContext
from .layers import Weight
from .mixers import PostNormLayer, _param


class MozalixForCausalLM(nn.Module):
    def __init__(self, cfg: ModelConfig, ctx: ParallelContext, dtype, device):
        super().__init__()
        if ctx.tp_size != 1:
            raise NotImplementedError("Mozalix stacks run on one GPU per replica (no tensor-parallel sharding of the mixers)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise TypeError(f"Mozalix runs in bfloat16 or float32, not {dtype}")
        self.cfg, self.ctx, self.dtype = cfg, ctx, dtype
        W = cfg.hidden_size
        self.embed = Weight((cfg.vocab_size, W), None, ctx, dtype, device)
        # modules of the layers that own parameters, by layer index; owner of every layer run
        self.layers = nn.ModuleDict({str(i): PostNormLayer(s, W, cfg.rms_eps, ctx, dtype, device)
                                     for i, s in enumerate(cfg.layer_specs) if s.weights_of < 0})
        self.runs = tuple(str(i if s.weights_of < 0 else s.weights_of) for i, s in enumerate(cfg.layer_specs))
        self.final_norm = _param((W,), ctx, device)
        self.head = Weight((cfg.vocab_size, W), None, ctx, dtype, device)
        self.layer_outputs = None          # a list: the stream after every layer is appended (tests, debugging)

    # ---- cache: pages of the attention mixers, recurrent state and convolution inputs per state slot — of every layer run
    def allocate_caches(self, num_blocks: int, num_slots: int, device):
        return [self.layers[r].cache(num_blocks, num_slots, self.dtype, device) for r in self.runs]

    def bytes_per_block(self) -> int:
        item = torch.empty((), dtype=self.dtype).element_size()
        return sum(sum(s.cache_row) for s in self.cfg.layer_specs) * KV_BLOCK_SIZE * item

    def bytes_per_slot(self) -> int:
        return sum(t.numel() * t.element_size() for r in self.runs for t in self.layers[r].cache(0, 1, self.dtype, "meta").state_tensors())

    def forward(self, input_ids: torch.Tensor, meta, caches) -> torch.Tensor:
        x, h = seqmix.embed_rows(input_ids, self.embed.data, self.cfg.embed_scale, self.dtype)
        last = len(self.runs) - 1
        for i, (run, cache) in enumerate(zip(self.runs, caches)):
            h = self.layers[run](x, h, meta, cache, self.final_norm.data if i == last else None)
            if self.layer_outputs is not None:
                self.layer_outputs.append(x.clone())
        return h

    def compute_logits(self, h: torch.Tensor) -> torch.Tensor:
        return ops.linear(h, self.head.data).float()

    # ---- parameters: (name, holder, init kind, checkpoint tensors: concatenated along dim 0, stacked (a list of lists), side by side
    # (behind "@cols") or along the diagonal (behind "@diag"))
    def named_weight_sources(self):
        yield "embed", self.embed, "normal", None
        for i, l in self.layers.items():
            yield from l.weights(f"l{i}.")
        yield "final.norm", self.final_norm, "zeros", None
        yield "head", self.head, "normal", None

    def named_weights(self):
        for name, w, kind, _src in self.named_weight_sources():
            yield name, w, kind

    def checkpoint_sources(self) -> dict:
        return {name: src for name, _w, _k, src in self.named_weight_sources() if src}
