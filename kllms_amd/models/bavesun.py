"""Bavesun: a decoder of parallel layers over an fp32 stream x,
    h = rms(x) (1 + w);   x <- x + (mixer(h) + ff(h))
    x <- x + rms(W_proj (gelu(W_gate x) * e)) w_side
where e is the layer's columns of the token's row in a side table. Mixers,
listed layer by layer in the config: retention (linear attention with a fixed
decay per head, rotary q and k) and latent attention with a sink and an
elementwise gate; the feed-forward is a gated gelu layer, routed squared-relu
experts, or absent. A range of layers may repeat several times with the same
weights, every pass with its own cache and state. The LM head is the
embedding table without its scale.

Kernel plan of one layer run: mixer and feed-forward on h -> add_cast (both
branches into the stream, the stream in the activation type) -> gate product
-> gelu_mul_rows -> projection -> sandwich_residual (post-norm, residual add,
the next reader's norm).
"""

from __future__ import annotations

import hashlib
import math
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..engine.config import BavesunArchConfig, BavesunLayerSpec
from ..engine.kvcache import LayerCacheSpec, LayerState
from ..parallel.tp import ParallelContext
from .listed import ListedLayerLM
from .llama import ForwardBatch
from .mixers import ActFF, CentredNormWeight, LatentAttention, Retention, RoutedExperts, TokenSide, _param


class BavesunLayer(nn.Module):
    def __init__(self, spec: BavesunLayerSpec, index: int, hidden: int, eps: float, side_dim: int, dtype):
        super().__init__()
        self.kind = spec.type
        self.norm1 = CentredNormWeight(hidden)
        self.mix = (Retention(spec.retention, hidden, eps, dtype) if spec.type == "retention"
                    else LatentAttention(spec.latent, hidden, eps, dtype))
        self.mlp = None
        if spec.mlp is not None:
            self.mlp = (ActFF(spec.mlp, hidden, dtype) if spec.mlp.kind == "dense"
                        else RoutedExperts(spec.mlp, hidden, dtype))
        self.side = TokenSide(hidden, side_dim, index, dtype) if side_dim else None

    def checkpoint_map(self, pre: str) -> Dict[str, torch.Tensor]:
        m = {pre + "norm1": self.norm1.weight}
        m.update(self.mix.checkpoint_map(pre + "mix."))
        if self.mlp is not None:
            m.update(self.mlp.checkpoint_map(pre + "mlp."))
        if self.side is not None:
            m.update(self.side.checkpoint_map(pre + "side."))
        return m


class BavesunForCausalLM(ListedLayerLM):
    def __init__(self, cfg: BavesunArchConfig, ctx: Optional[ParallelContext] = None, dtype=torch.bfloat16):
        super().__init__()
        self.cfg = cfg
        self.ctx = ctx or ParallelContext()
        assert self.ctx.world_size == 1, "the Bavesun family runs unsharded (tp_size must be 1)"
        self.dtype = dtype
        self.eps = cfg.rms_norm_eps
        W = cfg.hidden_size
        self.embed_tokens = nn.Embedding(cfg.vocab_size, W, dtype=dtype)
        self.embed_tokens.weight.requires_grad_(False)
        self.side_table = (_param(cfg.vocab_size, len(cfg.layers) * cfg.side_dim, dtype=dtype)
                           if cfg.side_dim else None)
        self.layers = nn.ModuleList([BavesunLayer(sp, i, W, self.eps, cfg.side_dim, dtype)
                                     for i, sp in enumerate(cfg.layers)])
        self.runs: List[int] = cfg.layer_runs()
        self.final_norm = CentredNormWeight(W)
        # the head is the embedding table itself
        self.lm_head = nn.Linear(W, cfg.vocab_size, bias=False, dtype=dtype)
        self.lm_head.weight = self.embed_tokens.weight

    # --- cache layout ---------------------------------------------------------
    def cache_layout(self) -> List[LayerCacheSpec]:
        """One entry per layer run: every pass of the loop keeps its own."""
        return [self.layers[i].mix.cache_spec() for i in self.runs]

    # --- weights ----------------------------------------------------------------
    def checkpoint_map(self) -> Dict[str, torch.Tensor]:
        m = {"embed": self.embed_tokens.weight, "final.norm": self.final_norm.weight}
        if self.side_table is not None:
            m["side.embed"] = self.side_table
        for i, layer in enumerate(self.layers):
            m.update(layer.checkpoint_map(f"l{i}."))
        return m

    def _after_load(self) -> None:
        for norm in [layer.norm1 for layer in self.layers] + [self.final_norm]:
            norm.fold()

    @torch.no_grad()
    def random_init_(self, seed: int = 0) -> None:
        """Deterministic random init, one generator per checkpoint name:
        matrices ~ N(0, 1/in), zero-centred norm weights and sinks small."""
        for name, dst in self.checkpoint_map().items():
            g = torch.Generator(device="cpu")
            g.manual_seed(int(hashlib.md5(f"{seed}/{name}".encode()).hexdigest()[:15], 16))
            parts = name.split(".")
            for part in dst if isinstance(dst, (list, tuple)) else [dst]:
                if parts[-1] == "norm1" or name == "final.norm":
                    t = torch.randn(part.shape, generator=g) * 0.1
                elif parts[-1] == "norm":
                    t = torch.full(part.shape, 0.5 if parts[-2] == "side" else 1.0)
                elif parts[-1] == "sink" or name == "side.embed":
                    t = torch.randn(part.shape, generator=g)
                else:
                    t = torch.randn(part.shape, generator=g) / math.sqrt(part.shape[-1])
                part.copy_(t.to(device=part.device, dtype=part.dtype))
        self._after_load()

    # --- forward ------------------------------------------------------------------
    def forward_hidden(self, input_ids: torch.Tensor, batch: ForwardBatch) -> torch.Tensor:
        assert batch.seg_start is not None, "this model takes segment batches"
        states: List[LayerState] = batch.kv_caches
        eps = self.eps
        x = ops.embed_bigram(input_ids, self.embed_tokens.weight, None, self.cfg.embed_scale, 0, 0, 0, None,
                             batch.state_slots, batch.cu_seqlens, batch.seg_start, batch.token_seg)
        # the norm weight of whatever reads the stream after each layer run
        scales = [self.layers[i].norm1.scale for i in self.runs] + [self.final_norm.scale]
        h, _ = ops.group_norm_pair(x, None, None, scales[0], None, 1, eps, self.dtype)
        for run, i in enumerate(self.runs):
            layer = self.layers[i]
            a = layer.mix(h, batch, states[run])
            b = layer.mlp(h) if layer.mlp is not None else None
            if layer.side is not None:
                y = layer.side(ops.add_cast(x, a, b, self.dtype), input_ids, self.side_table)
                h = ops.sandwich_residual(x, y, layer.side.norm, eps, w_next=scales[run + 1], out_dtype=self.dtype)
            else:
                h, _ = ops.group_norm_pair(x, a, b, scales[run + 1], None, 1, eps, self.dtype)
            if self.trace_layers is not None:
                self.trace_layers.append(x.clone())
        return h
