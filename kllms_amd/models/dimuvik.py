"""Dimuvik: a decoder over an fp32 stream x whose sublayers are normed before
and after by dynamic tanh, dyt(v) = tanh(alpha v) w + b:
    x <- x + dyt_1b(mixer(dyt_1(x)));   x <- x + dyt_2b(ff(dyt_2(x)))
Mixers, listed layer by layer in the config: differential attention with short
convolutions on q, k and v (optionally on the keys and values of an earlier
layer), and latent attention with a query latent and a sink; the feed-forward
is a squared-relu layer, routed silu experts with a shared expert, or absent.
The LM head is a matrix of its own.

Kernel plan: embed_dyt (the stream and the first norm), then per layer: mixer
on h -> dyt_residual (post-norm, residual add, the next reader's norm, cast)
-> feed-forward -> dyt_residual.
"""

from __future__ import annotations

import hashlib
import math
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..engine.config import DimuvikArchConfig, DimuvikLayerSpec
from ..engine.kvcache import LayerCacheSpec, LayerState
from ..parallel.tp import ParallelContext
from .listed import ListedLayerLM
from .llama import ForwardBatch
from .mixers import ActFF, DiffAttention, DynamicTanh, LatentAttention, RoutedExperts


class DimuvikLayer(nn.Module):
    def __init__(self, spec: DimuvikLayerSpec, hidden: int, eps: float, dtype):
        super().__init__()
        self.kind = spec.type
        self.norm1, self.norm1b = DynamicTanh(hidden), DynamicTanh(hidden)
        self.mix = (DiffAttention(spec.attention, hidden, eps, dtype) if spec.type == "attention"
                    else LatentAttention(spec.latent, hidden, eps, dtype))
        self.mlp = None
        if spec.mlp is not None:
            self.norm2, self.norm2b = DynamicTanh(hidden), DynamicTanh(hidden)
            self.mlp = (ActFF(spec.mlp, hidden, dtype) if spec.mlp.kind == "dense"
                        else RoutedExperts(spec.mlp, hidden, dtype))

    def checkpoint_map(self, pre: str) -> Dict[str, torch.Tensor]:
        m = {**self.norm1.checkpoint_map(pre + "norm1"), **self.norm1b.checkpoint_map(pre + "norm1b"),
             **self.mix.checkpoint_map(pre + "mix.")}
        if self.mlp is not None:
            m.update(self.norm2.checkpoint_map(pre + "norm2"))
            m.update(self.norm2b.checkpoint_map(pre + "norm2b"))
            m.update(self.mlp.checkpoint_map(pre + "mlp."))
        return m


class DimuvikForCausalLM(ListedLayerLM):
    def __init__(self, cfg: DimuvikArchConfig, ctx: Optional[ParallelContext] = None, dtype=torch.bfloat16):
        super().__init__()
        self.cfg = cfg
        self.ctx = ctx or ParallelContext()
        assert self.ctx.world_size == 1, "the Dimuvik family runs unsharded (tp_size must be 1)"
        self.dtype = dtype
        W = cfg.hidden_size
        self.embed_tokens = nn.Embedding(cfg.vocab_size, W, dtype=dtype)
        self.embed_tokens.weight.requires_grad_(False)
        self.layers = nn.ModuleList([DimuvikLayer(sp, W, cfg.rms_norm_eps, dtype) for sp in cfg.layers])
        self.final_norm = DynamicTanh(W)
        self.lm_head = nn.Linear(W, cfg.vocab_size, bias=False, dtype=dtype)
        self.lm_head.weight.requires_grad_(False)

    # --- cache layout ---------------------------------------------------------
    def cache_layout(self) -> List[LayerCacheSpec]:
        return [layer.mix.cache_spec() for layer in self.layers]

    # --- weights ----------------------------------------------------------------
    def checkpoint_map(self) -> Dict[str, torch.Tensor]:
        m = {"embed": self.embed_tokens.weight, "head": self.lm_head.weight,
             **self.final_norm.checkpoint_map("final.norm")}
        for i, layer in enumerate(self.layers):
            m.update(layer.checkpoint_map(f"l{i}."))
        return m

    def _after_load(self) -> None:
        for layer in self.layers:
            if layer.kind == "attention":
                layer.mix.fold()

    @torch.no_grad()
    def random_init_(self, seed: int = 0) -> None:
        """Deterministic random init, one generator per checkpoint name:
        matrices ~ N(0, 1/in), norm weights 1 and biases 0, the tanh slopes
        below one, small lambda vectors, corrections and projection biases."""
        for name, dst in self.checkpoint_map().items():
            g = torch.Generator(device="cpu")
            g.manual_seed(int(hashlib.md5(f"{seed}/{name}".encode()).hexdigest()[:15], 16))
            parts = name.split(".")
            normed = parts[-2] if parts[-1] in ("b", "alpha") else parts[-1]
            for part in dst if isinstance(dst, (list, tuple)) else [dst]:
                if parts[-1] == "alpha":
                    t = torch.full(part.shape, 0.6)
                elif normed in ("norm", "norm1", "norm2", "norm1b", "norm2b"):
                    t = torch.full(part.shape, 0.0 if parts[-1] == "b" else 1.0)
                elif parts[-1] in ("b", "correction", "lq1", "lk1", "lq2", "lk2"):
                    t = torch.randn(part.shape, generator=g) * 0.1
                elif parts[-1] in ("embed", "sink"):
                    t = torch.randn(part.shape, generator=g)
                else:
                    t = torch.randn(part.shape, generator=g) / math.sqrt(part.shape[-1])
                part.copy_(t.to(device=part.device, dtype=part.dtype))
        self._after_load()

    # --- forward ------------------------------------------------------------------
    def forward_hidden(self, input_ids: torch.Tensor, batch: ForwardBatch) -> torch.Tensor:
        assert batch.seg_start is not None, "this model takes segment batches"
        states: List[LayerState] = batch.kv_caches
        # the norm of whatever reads the stream after each layer
        nxt = [layer.norm1.args for layer in self.layers] + [self.final_norm.args]
        x, h = ops.embed_dyt(input_ids, self.embed_tokens.weight, self.cfg.embed_scale, nxt[0])
        for i, layer in enumerate(self.layers):
            a = layer.mix(h, batch, states[i])
            if layer.mlp is not None:
                h = ops.dyt_residual(x, a, layer.norm1b.args, layer.norm2.args, self.dtype)
                h = ops.dyt_residual(x, layer.mlp(h), layer.norm2b.args, nxt[i + 1], self.dtype)
            else:
                h = ops.dyt_residual(x, a, layer.norm1b.args, nxt[i + 1], self.dtype)
            if self.trace_layers is not None:
                self.trace_layers.append(x.clone())
        return h
