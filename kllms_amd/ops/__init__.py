"""Op dispatch: HIP/CDNA4 kernels on GPU, torch reference on CPU.

Policy: on a GPU (`tensor.is_cuda`, which on
PyTorch-ROCm means an AMD GPU) the hand-written gfx950 HIP kernels in
``kllms_amd._C`` are the ONLY path — if the extension is missing the op
RAISES instead of silently falling back to eager PyTorch. On CPU the pure
torch reference implementations (torch_ref.py) run, which is what the
GPU-less CI environment uses.

Set ``KLLMS_AMD_FORCE_TORCH_OPS=1`` to force the torch path on GPU (used only
by numerics tests to produce the oracle on-device).
"""

from __future__ import annotations

import os
from typing import Optional, Tuple

import torch

from . import torch_ref

_C = None
_C_err: Optional[str] = None
try:
    from kllms_amd import _C  # type: ignore[no-redef]  # built by setup.py build_ext --inplace
except Exception as e:  # pragma: no cover - import-time probe
    _C = None
    _C_err = str(e)


def hip_available() -> bool:
    return _C is not None


def _force_torch() -> bool:
    return os.environ.get("KLLMS_AMD_FORCE_TORCH_OPS", "0") == "1"


def _hip_or_raise():
    if _C is None:
        raise RuntimeError(
            "kllms_amd HIP extension (kllms_amd/_C*.so) is not built but a GPU "
            "tensor was passed. Build it with `python setup.py build_ext --inplace` "
            f"(PYTORCH_ROCM_ARCH=gfx950). Import error: {_C_err}"
        )
    return _C


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    if x.is_cuda and not _force_torch():
        out = torch.empty_like(x)
        _hip_or_raise().rmsnorm(out, x, weight, eps)
        return out
    return torch_ref.rmsnorm(x, weight, eps)


def fused_add_rmsnorm(
    x: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor, eps: float
) -> Tuple[torch.Tensor, torch.Tensor]:
    if x.is_cuda and not _force_torch():
        # in-place: residual += x; x_out = rmsnorm(residual)
        out = torch.empty_like(x)
        _hip_or_raise().fused_add_rmsnorm(out, x, residual, weight, eps)
        return out, residual
    return torch_ref.fused_add_rmsnorm(x, residual, weight, eps)


def rope_inplace(q: torch.Tensor, k: torch.Tensor, positions: torch.Tensor, cos_sin: torch.Tensor) -> None:
    if q.is_cuda and not _force_torch():
        _hip_or_raise().rope_inplace(q, k, positions, cos_sin)
        return
    torch_ref.rope_inplace(q, k, positions, cos_sin)


def silu_mul(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    if gate.is_cuda and not _force_torch():
        out = torch.empty(gate.shape, dtype=gate.dtype, device=gate.device)
        _hip_or_raise().silu_mul(out, gate, up)
        return out
    return torch_ref.silu_mul(gate, up)


def store_kv(
    k: torch.Tensor,
    v: torch.Tensor,
    k_cache: torch.Tensor,
    v_cache: torch.Tensor,
    slot_mapping: torch.Tensor,
    k_scale: Optional[torch.Tensor] = None,
    v_scale: Optional[torch.Tensor] = None,
) -> None:
    """k_scale/v_scale: [NB, KVH, BS] fp32 per-row dequant scales, REQUIRED
    when the caches are fp8 (written here: s = amax(|row|)/448), None for bf16."""
    if k.is_cuda and not _force_torch():
        none = torch.empty(0, dtype=torch.float32, device=k.device)
        _hip_or_raise().store_kv(
            k, v, k_cache, v_cache, slot_mapping,
            k_scale if k_scale is not None else none,
            v_scale if v_scale is not None else none)
        return
    torch_ref.store_kv(k, v, k_cache, v_cache, slot_mapping, k_scale, v_scale)


def _prefill_tiles(cu_seqlens: torch.Tensor, device) -> tuple:
    """Grouped q-tile metadata for the MFMA prefill kernel: 32-row q-tiles of
    each sequence packed 8 per workgroup (the 8 waves share the K/V LDS
    staging); idle wave slots padded with -1. One host round-trip per prefill
    batch (once per generate() call)."""
    NW = 8
    cu = cu_seqlens.cpu().tolist()
    grp_start, grp_len, grp_qpos0 = [], [], []
    for i in range(len(cu) - 1):
        s, e = cu[i], cu[i + 1]
        L = e - s
        tiles = list(range(0, L, 32))
        for g0 in range(0, len(tiles), NW):
            grp_start.append(s)
            grp_len.append(L)
            grp = tiles[g0 : g0 + NW]
            grp_qpos0.extend(grp + [-1] * (NW - len(grp)))
    t = lambda x: torch.tensor(x, dtype=torch.int32, device=device)
    return t(grp_start), t(grp_qpos0), t(grp_len)


def attn_prefill_varlen(
    q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, cu_seqlens: torch.Tensor, scale: float
) -> torch.Tensor:
    if q.is_cuda and not _force_torch():
        out = torch.empty(q.shape, dtype=q.dtype, device=q.device)
        gs, gq, gl = _prefill_tiles(cu_seqlens, q.device)
        _hip_or_raise().attn_prefill(out, q, k, v, gs, gq, gl, scale)
        return out
    return torch_ref.attn_prefill_varlen(q, k, v, cu_seqlens, scale)


def attn_decode_paged(
    q: torch.Tensor,
    k_cache: torch.Tensor,
    v_cache: torch.Tensor,
    block_tables: torch.Tensor,
    context_lens: torch.Tensor,
    scale: float,
    k_scale: Optional[torch.Tensor] = None,
    v_scale: Optional[torch.Tensor] = None,
) -> torch.Tensor:
    if q.is_cuda and not _force_torch():
        out = torch.empty(q.shape, dtype=q.dtype, device=q.device)
        none = torch.empty(0, dtype=torch.float32, device=q.device)
        _hip_or_raise().attn_decode_paged(
            out, q, k_cache, v_cache, block_tables, context_lens, scale,
            k_scale if k_scale is not None else none,
            v_scale if v_scale is not None else none)
        return out
    return torch_ref.attn_decode_paged(q, k_cache, v_cache, block_tables, context_lens, scale,
                                       k_scale, v_scale)


def sample(
    logits: torch.Tensor,
    temperatures: torch.Tensor,
    top_ps: torch.Tensor,
    top_ks: torch.Tensor,
    seeds: torch.Tensor,
    steps: torch.Tensor,
    mask: Optional[torch.Tensor] = None,
    dbg: Optional[torch.Tensor] = None,
) -> Tuple[torch.Tensor, torch.Tensor]:
    if logits.is_cuda and not _force_torch():
        B = logits.shape[0]
        tokens = torch.empty(B, dtype=torch.long, device=logits.device)
        logprobs = torch.empty(B, dtype=torch.float32, device=logits.device)
        _hip_or_raise().sample(
            tokens, logprobs, logits, temperatures, top_ps, top_ks, seeds, steps,
            mask if mask is not None else torch.empty(0, dtype=torch.int32, device=logits.device),
            dbg if dbg is not None else torch.empty(0, dtype=torch.float32, device=logits.device),
        )
        return tokens, logprobs
    return torch_ref.sample(logits, temperatures, top_ps, top_ks, seeds, steps, mask)


def moe_gateup(
    act: torch.Tensor,
    x: torch.Tensor,
    w_gate_up: torch.Tensor,
    sorted_ids: torch.Tensor,
    pad_offsets: torch.Tensor,
    zeros: torch.Tensor,
) -> None:
    """Grouped MoE gate/up GEMM + fused silu*mul into `act` (sorted-by-expert
    row space). GPU-only (Mixtral prefill hot path); the CPU path keeps the
    per-expert torch loop in models/mixtral.py."""
    _hip_or_raise().moe_gateup(act, x, w_gate_up, sorted_ids, pad_offsets, zeros)


def moe_down(
    y: torch.Tensor,
    act: torch.Tensor,
    w_down: torch.Tensor,
    pad_offsets: torch.Tensor,
) -> None:
    """Grouped MoE down GEMM in sorted-row space (see moe_gateup)."""
    _hip_or_raise().moe_down(y, act, w_down, pad_offsets)


def levenshtein_pairs(
    chars: torch.Tensor,
    lens: torch.Tensor,
    pair_i: torch.Tensor,
    pair_j: torch.Tensor,
) -> torch.Tensor:
    """Batched Myers bit-parallel edit distance over packed [N, 64] uint8
    normalized strings; returns int32 distances per (i, j) pair. GPU-only —
    the CPU consensus path keeps the pure-python DP (utils/text.py)."""
    return _hip_or_raise().levenshtein_pairs(chars, lens, pair_i, pair_j)


# --- sequence-mixer family (kllms_amd._C_seq) -----------------------------------
# fp32 residual stream, block-local paged attention, recurrent mixers. The
# extension is separate from _C so that a model of this family compiles only
# its own kernels in a checkout where nothing is built yet.

_SEQ = None


def _seq():
    global _SEQ
    if _SEQ is None:
        from . import jit

        _SEQ = jit.load("_C_seq")
    return _SEQ


def seq_hip_loaded() -> bool:
    return _SEQ is not None


def _gpu(t: torch.Tensor) -> bool:
    return t.is_cuda and not _force_torch()


def _none(ref: torch.Tensor, dtype=None) -> torch.Tensor:
    return torch.empty(0, dtype=dtype or ref.dtype, device=ref.device)


def embed_rmsnorm(ids, table, weight, eps, pos_table=None, positions=None):
    """fp32 rms(table[ids] (+ pos_table[positions])) * weight."""
    if _gpu(table):
        out = torch.empty((ids.numel(), table.shape[1]), dtype=torch.float32, device=table.device)
        has = pos_table is not None
        _seq().embed_rmsnorm(out, ids, table, weight, eps, pos_table if has else _none(table),
                             positions if has else _none(table, torch.long))
        return out
    return torch_ref.embed_rmsnorm(ids, table, weight, eps, pos_table, positions)


def rmsnorm_cast(x, weight, eps, out_dtype):
    if _gpu(x):
        out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
        _seq().rmsnorm_cast(out, x, weight, eps)
        return out
    return torch_ref.rmsnorm_cast(x, weight, eps, out_dtype)


def sandwich_residual(x, a, w_post, eps, b=None, wa=None, wb=None, w_next=None, out_dtype=None, cast=False):
    """x (fp32 residual, in place) += rms(y) * w_post with y = a, or
    y = (rms(a) wa + rms(b) wb) / 2; returns rms(x) * w_next in a's dtype.
    With w_next None: the new x in a's dtype if ``cast`` (the input of a
    sublayer that reads the stream itself), else None."""
    if _gpu(x):
        want = w_next is not None or cast
        out = torch.empty(a.shape, dtype=a.dtype, device=a.device) if want else _none(a)
        f = _none(x, torch.float32)
        _seq().sandwich_residual(
            x, a, b if b is not None else _none(a), wa if b is not None else f, wb if b is not None else f,
            w_post, w_next if w_next is not None else f, out, eps)
        return out if want else None
    return torch_ref.sandwich_residual(x, a, w_post, eps, b, wa, wb, w_next, out_dtype or a.dtype, cast)


def rope_pairs_store(q, k, v, positions, inv_freq, k_cache, v_cache, slot_mapping, kv_fresh=None) -> None:
    """kv_fresh (GPU only, optional): [T, 2, G, D] buffer that also receives
    this step's rotated keys ([:, 0]) and values ([:, 1]) packed, for the
    dense prefill kernel."""
    if _gpu(q):
        _seq().rope_pairs_store(q, k, v if v is not None else _none(q), positions, inv_freq,
                                k_cache, v_cache, slot_mapping,
                                kv_fresh if kv_fresh is not None else _none(q))
        return
    torch_ref.rope_pairs_store(q, k, v, positions, inv_freq, k_cache, v_cache, slot_mapping)


def attn_masked_paged(q, k_cache, v_cache, block_tables, token_seg, positions, scale, mask_kind, mask_size,
                      keep_first=0, sink=False, gate=None, row_map=None, out=None):
    """Paged softmax attention with a block-local (mask_kind 0) or sliding
    window + kept first tokens (mask_kind 1) causal mask, optional sink term,
    gate per head [T, H] or per element [T, H*Dv]. row_map / out (GPU only):
    serve just the listed rows, writing into an existing [T, H, Dv] tensor
    whose other rows another kernel fills."""
    if _gpu(q):
        if out is None:
            out = torch.empty((q.shape[0], q.shape[1], v_cache.shape[3]), dtype=q.dtype, device=q.device)
        _seq().attn_masked_paged(out, q, k_cache, v_cache, block_tables, token_seg, positions,
                                 gate if gate is not None else _none(q), scale, int(mask_kind), int(mask_size),
                                 int(keep_first), bool(sink),
                                 row_map if row_map is not None else _none(q, torch.int32),
                                 _none(q, torch.float32), _none(q, torch.float32), 0, 0.0,
                                 _none(q, torch.float32), _none(q, torch.float32))
        return out
    assert row_map is None and out is None
    return torch_ref.attn_masked_paged(q, k_cache, v_cache, block_tables, token_seg, positions, scale,
                                       mask_kind, mask_size, keep_first, sink, gate)


def attn_blocklocal_paged(q, k_cache, v_cache, block_tables, token_seg, positions, scale, mask_size,
                          gate=None, row_map=None, out=None):
    """Block-local mask, no sink, per-head gate: a case of attn_masked_paged."""
    if _gpu(q):
        return attn_masked_paged(q, k_cache, v_cache, block_tables, token_seg, positions, scale, 0, mask_size,
                                 0, False, gate, row_map, out)
    assert row_map is None and out is None
    return torch_ref.attn_blocklocal_paged(q, k_cache, v_cache, block_tables, token_seg, positions,
                                           scale, mask_size, gate)


def attn_varlen_mfma(out, q, k, v, grp_start, grp_qpos0, grp_len, scale) -> None:
    """Dense causal MFMA attention over packed pieces (bf16, head size 128;
    GPU only): each piece attends within itself. Tile groups come from
    dense_tile_groups()."""
    _seq().attn_varlen_mfma(out, q, k, v, grp_start, grp_qpos0, grp_len, scale)


def dense_tile_groups(pieces, device):
    """Host metadata for attn_varlen_mfma: pieces = [(first row, length)];
    32-row q-tiles of each piece, 8 per workgroup (idle wave slots = -1)."""
    NW = 8
    gs, gl, gq = [], [], []
    for row0, L in pieces:
        tiles = list(range(0, L, 32))
        for g0 in range(0, len(tiles), NW):
            grp = tiles[g0:g0 + NW]
            gs.append(row0)
            gl.append(L)
            gq.extend(grp + [-1] * (NW - len(grp)))
    t = lambda x: torch.tensor(x, dtype=torch.int32, device=device)
    return t(gs), t(gq), t(gl)


def head_gate(out, gate) -> None:
    """out[t, h, :] *= sigmoid(gate[t, h]) in place."""
    if _gpu(out):
        _seq().head_gate(out, gate)
        return
    out.mul_(torch.sigmoid(gate.float()).unsqueeze(-1).to(out.dtype))


def linear_attn_decay(q, k, v, decay, state, state_slots, cu_seqlens, seg_start):
    if _gpu(q):
        o = torch.empty((q.shape[0], q.shape[1], v.shape[2]), dtype=torch.float32, device=q.device)
        _seq().linear_attn_decay(o, q, k, v, decay, state, state_slots, cu_seqlens, seg_start)
        return o
    return torch_ref.linear_attn_decay(q, k, v, decay, state, state_slots, cu_seqlens, seg_start)


def gated_rmsnorm(o, weight, gate, eps, out_dtype, gate_act="sigmoid"):
    """Grouped RMS norm of o [T, groups, S] fp32 (weight [S] or None) times
    the activated gate (sigmoid or silu)."""
    if _gpu(o):
        out = torch.empty((o.shape[0], o.shape[1] * o.shape[2]), dtype=out_dtype, device=o.device)
        _seq().gated_rmsnorm(out, o, weight if weight is not None else _none(o), gate, eps,
                             0 if gate_act == "sigmoid" else 2)
        return out
    return torch_ref.gated_rmsnorm(o, weight, gate, eps, out_dtype, gate_act)


def causal_conv_silu(x, w, conv_state, state_slots, cu_seqlens, seg_start, token_seg, bias=None):
    if _gpu(x):
        y = torch.empty(x.shape, dtype=x.dtype, device=x.device)
        _seq().causal_conv_silu(y, x, w, conv_state, state_slots, cu_seqlens, seg_start, token_seg,
                                bias if bias is not None else _none(x, torch.float32))
        return y
    return torch_ref.causal_conv_silu(x, w, conv_state, state_slots, cu_seqlens, seg_start, bias)


def gated_delta_rule(q, k, v, beta_logit, a, dt_bias, a_log, state, state_slots, cu_seqlens, seg_start):
    if _gpu(q):
        o = torch.empty((v.shape[0], v.shape[1], v.shape[2]), dtype=torch.float32, device=q.device)
        _seq().gated_delta_rule(o, q, k, v, beta_logit, a, dt_bias, a_log, state, state_slots,
                                cu_seqlens, seg_start)
        return o
    return torch_ref.gated_delta_rule(q, k, v, beta_logit, a, dt_bias, a_log, state, state_slots,
                                      cu_seqlens, seg_start)


def gated_act(gate, up, limit: float, alpha: float, up_bias: float):
    """min(g, limit) sigmoid(alpha min(g, limit)) (clamp(u, +-limit) + up_bias)."""
    if _gpu(gate):
        out = torch.empty(gate.shape, dtype=gate.dtype, device=gate.device)
        _seq().gated_act(out, gate, up, limit, alpha, up_bias)
        return out
    return torch_ref.gated_act(gate, up, limit, alpha, up_bias)


def clamped_glu(gate, up, limit: float, alpha: float):
    if _gpu(gate):
        return gated_act(gate, up, limit, alpha, 1.0)
    return torch_ref.clamped_glu(gate, up, limit, alpha)


def silu_glu(gate, up):
    """silu(gate) * up in the activation dtype (bf16 or fp32)."""
    return gated_act(gate, up, float("inf"), 1.0, 0.0)


def embed_bigram(ids, table, bigram, scale, mul_prev, mul_cur, buckets, tok_state, state_slots, cu_seqlens,
                 seg_start, token_seg, out=None):
    """fp32 rows table[id] * scale (+ the hashed bigram row); ``out``: an
    existing contiguous [T, W] fp32 tensor to fill."""
    if _gpu(table):
        if out is None:
            out = torch.empty((ids.numel(), table.shape[1]), dtype=torch.float32, device=table.device)
        has = bigram is not None
        _seq().embed_bigram(out, ids, table, bigram if has else _none(table), float(scale), int(mul_prev),
                            int(mul_cur), int(buckets), tok_state if has else _none(table, torch.int32),
                            state_slots, cu_seqlens, seg_start, token_seg)
        return out
    x = torch_ref.embed_bigram(ids, table, bigram, scale, mul_prev, mul_cur, buckets, tok_state,
                               state_slots, cu_seqlens, seg_start)
    return x if out is None else out.copy_(x)


def group_norm_pair(x, a, b, w1, w2, groups, eps, out_dtype):
    """x (fp32 residual, in place) += a + b; returns the grouped RMS norm of x
    under two weights (the second may be None)."""
    if _gpu(x):
        h1 = torch.empty(x.shape, dtype=out_dtype, device=x.device)
        h2 = torch.empty(x.shape, dtype=out_dtype, device=x.device) if w2 is not None else None
        f = _none(x, torch.float32)
        e = _none(x, out_dtype)
        _seq().group_norm_pair(x, a if a is not None else e, b if b is not None else e, w1,
                               w2 if w2 is not None else f, h1, h2 if h2 is not None else e, int(groups), eps)
        return h1, h2
    return torch_ref.group_norm_pair(x, a, b, w1, w2, groups, eps, out_dtype)


def cast_concat(x, x0, a, b, out_dtype):
    """x (fp32 residual, in place) += a + b; returns [x | x0] in out_dtype."""
    if _gpu(x):
        out = torch.empty((x.shape[0], 2 * x.shape[1]), dtype=out_dtype, device=x.device)
        e = _none(x, out_dtype)
        _seq().cast_concat(out, x, x0, a if a is not None else e, b if b is not None else e)
        return out
    return torch_ref.cast_concat(x, x0, a, b, out_dtype)


def qk_norm_store(q, k, v, wq, wk, eps, k_cache, v_cache, slot_mapping) -> None:
    if _gpu(q):
        _seq().qk_norm_store(q, k, v, wq, wk, eps, k_cache, v_cache, slot_mapping)
        return
    torch_ref.qk_norm_store(q, k, v, wq, wk, eps, k_cache, v_cache, slot_mapping)


def token_shift_mix(h, mu, shift_state, state_slots, cu_seqlens, seg_start, token_seg, n_act):
    """([n_act, T, W] in h's dtype, [n - n_act, T, W] fp32) mixes of each row
    with its predecessor; carries the last row in shift_state."""
    if _gpu(h):
        T, W = h.shape
        n = mu.shape[0]
        act = torch.empty((n_act, T, W), dtype=h.dtype, device=h.device)
        f32 = torch.empty((n - n_act, T, W), dtype=torch.float32, device=h.device)
        _seq().token_shift_mix(act, f32, h, mu, shift_state, state_slots, cu_seqlens, seg_start, token_seg)
        return act, f32
    return torch_ref.token_shift_mix(h, mu, shift_state, state_slots, cu_seqlens, seg_start, n_act, h.dtype)


def wkv_recurrence(r, k, v, d, w0, u, state, state_slots, cu_seqlens, seg_start):
    if _gpu(r):
        o = torch.empty((r.shape[0], r.shape[1], v.shape[2]), dtype=torch.float32, device=r.device)
        _seq().wkv_recurrence(o, r, k, v, d, w0, u, state, state_slots, cu_seqlens, seg_start)
        return o
    return torch_ref.wkv_recurrence(r, k, v, d, w0, u, state, state_slots, cu_seqlens, seg_start)


def mlstm_recurrence(q, k, v, gates, gate_bias, cap, state, state_slots, cu_seqlens, seg_start):
    if _gpu(q):
        o = torch.empty((q.shape[0], q.shape[1], v.shape[2]), dtype=torch.float32, device=q.device)
        e = _none(q, torch.float32)
        _seq().mlstm_recurrence(o, q, k, v, gates, gate_bias, float(cap), state, state_slots, cu_seqlens,
                                seg_start, e, e)
        return o
    return torch_ref.mlstm_recurrence(q, k, v, gates, gate_bias, cap, state, state_slots, cu_seqlens,
                                      seg_start)


def mlstm_mix_out(q, k, v, gates, gate_bias, cap, state, state_slots, cu_seqlens, seg_start, weight, gate, eps,
                  out_dtype):
    """mlstm_recurrence followed by head_rmsnorm_gate(sigmoid); on the GPU the
    read-out's division happens inside the norm kernel."""
    if _gpu(q):
        T, H, V = q.shape[0], q.shape[1], v.shape[2]
        oe = torch.empty((T, H, V + 1), dtype=torch.float32, device=q.device)
        mt = torch.empty((T, H), dtype=torch.float32, device=q.device)
        _seq().mlstm_recurrence(_none(q, torch.float32), q, k, v, gates, gate_bias, float(cap), state, state_slots,
                                cu_seqlens, seg_start, oe, mt)
        out = torch.empty((T, H * V), dtype=out_dtype, device=q.device)
        _seq().head_rmsnorm_gate(out, oe, weight, gate, eps, 0, mt)
        return out
    o = torch_ref.mlstm_recurrence(q, k, v, gates, gate_bias, cap, state, state_slots, cu_seqlens, seg_start)
    return torch_ref.head_rmsnorm_gate(o, weight, gate, eps, "sigmoid", out_dtype)


def head_rmsnorm_gate(o, weight, gate, eps, gate_act, out_dtype):
    if _gpu(o):
        out = torch.empty((o.shape[0], o.shape[1] * o.shape[2]), dtype=out_dtype, device=o.device)
        _seq().head_rmsnorm_gate(out, o, weight, gate, eps,
                                 0 if gate_act == "sigmoid" else 1, _none(o, torch.float32))
        return out
    return torch_ref.head_rmsnorm_gate(o, weight, gate, eps, gate_act, out_dtype)


_SCORE_KINDS = {"softmax": 0, "sigmoid": 1, "top_softmax": 2}


def moe_route(z, correction, top, group_count, group_keep, score="softmax", renormalize=True, scale=1.0):
    """Routing from fp32 logits z [T, N]: (idx [T, top] int32, w [T, top] fp32)."""
    if _gpu(z):
        idx = torch.empty((z.shape[0], top), dtype=torch.int32, device=z.device)
        w = torch.empty((z.shape[0], top), dtype=torch.float32, device=z.device)
        _seq().moe_route(idx, w, _none(z, torch.int32), z, _none(z),
                         correction if correction is not None else _none(z), int(top), int(group_count),
                         int(group_keep), 0, _SCORE_KINDS[score], bool(renormalize), float(scale))
        return idx, w
    return torch_ref.moe_route(z, correction, top, group_count, group_keep, score, renormalize, scale)


def moe_route_rows(h, router, correction, top, group_count, group_keep, experts, all_experts_form,
                   score="softmax", renormalize=True, scale=1.0):
    """Router GEMV in fp32 + routing in one kernel. Returns (idx, w, rowidx);
    rowidx [T, top] (only when all_experts_form) addresses rows of the
    all-experts output [experts * T, W]: choice * T + row, -1 = identity."""
    T = h.shape[0]
    if _gpu(h):
        idx = torch.empty((T, top), dtype=torch.int32, device=h.device)
        w = torch.empty((T, top), dtype=torch.float32, device=h.device)
        rowidx = torch.empty((T, top), dtype=torch.int32, device=h.device) if all_experts_form else None
        _seq().moe_route(idx, w, rowidx if rowidx is not None else _none(h, torch.int32), h, router,
                         correction if correction is not None else _none(router),
                         int(top), int(group_count), int(group_keep), int(experts),
                         _SCORE_KINDS[score], bool(renormalize), float(scale))
        return idx, w, rowidx
    z = torch.nn.functional.linear(h.float(), router)
    idx, w = torch_ref.moe_route(z, correction, top, group_count, group_keep, score, renormalize, scale)
    rowidx = None
    if all_experts_form:
        t_idx = torch.arange(T, dtype=torch.int32, device=h.device).unsqueeze(1)
        rowidx = torch.where(idx < experts, idx * T + t_idx, torch.full_like(idx, -1))
    return idx, w, rowidx


def moe_combine(rows, h, rowidx, w, out_dtype, extra=None, extra_gate=None):
    """Fixed-order sum of each row's chosen expert rows, weighted by w (None =
    unweighted), plus sigmoid(extra_gate[t]) * extra[t] when given
    (extra_gate: a [T] view, any stride; None: plus extra[t])."""
    if _gpu(h):
        out = torch.empty(h.shape, dtype=out_dtype, device=h.device)
        _seq().moe_combine(out, rows, h, rowidx, w if w is not None else _none(h, torch.float32),
                           extra if extra is not None else _none(h),
                           extra_gate if extra_gate is not None else _none(h))
        return out
    return torch_ref.moe_combine(rows, h, rowidx, w, out_dtype, extra, extra_gate)


def scale_rows(h, src_row, scale):
    """out[i] = h[src_row[i]] * scale[i]: expert inputs that carry their
    routing weight. src_row int32 [n], scale fp32 [n]."""
    if _gpu(h):
        out = torch.empty((src_row.numel(), h.shape[1]), dtype=h.dtype, device=h.device)
        _seq().scale_rows(out, h, src_row, scale)
        return out
    return torch_ref.scale_rows(h, src_row, scale)


def moe_spread_rows(h, idx, w, experts: int):
    """[experts, T, W] inputs of the all-experts form when the routing weight
    sits on the expert's input: w[t, j] * h[t] for row t's j-th choice, zero
    rows for the experts a row did not choose."""
    if _gpu(h):
        out = torch.empty((experts, h.shape[0], h.shape[1]), dtype=h.dtype, device=h.device)
        _seq().moe_spread_rows(out, h, idx, w)
        return out
    return torch_ref.moe_spread_rows(h, idx, w, experts)


def gelu_tanh(x):
    """Tanh-form gelu of a [T, C] row view, in x's dtype."""
    if _gpu(x):
        out = torch.empty(x.shape, dtype=x.dtype, device=x.device)
        _seq().gelu_tanh(out, x)
        return out
    return torch_ref.gelu_tanh(x)


def scale_softcap_(z, scale: float, cap: float) -> None:
    """fp32 logits in place: z * scale, then cap * tanh(. / cap) if cap > 0."""
    if _gpu(z):
        _seq().scale_softcap(z, float(scale), float(cap))
        return
    torch_ref.scale_softcap_(z, scale, cap)


def latent_kv_store(q, dkv, w_norm, eps, positions, inv_freq, cache, slot_mapping, nope_dim) -> None:
    """Rotates the rotated part of every query head in place; norms the
    latent, rotates the shared key part and stores [latent | key part] into
    the paged latent cache."""
    if _gpu(q):
        _seq().latent_kv_store(q, dkv, w_norm, eps, positions, inv_freq, cache, slot_mapping, int(nope_dim))
        return
    torch_ref.latent_kv_store(q, dkv, w_norm, eps, positions, inv_freq, cache, slot_mapping, nope_dim)


def attn_latent_paged(q_abs, q, cache, block_tables, token_seg, positions, scale, mask_size, gate, nope_dim,
                      tile_rows: int = 0, use_mfma: bool = True, key_splits: int = 0, sink=None):
    """Sliding-window softmax attention over the paged latent cache in the
    absorbed form (one shared key/value row per token for all heads):
    returns the heads' weighted latent sums [T, H, C], gated per head. sink
    [H] fp32: one more term exp(sink_h) in the softmax denominator.
    GPU: bf16 rows go through the matrix-unit kernel when the sizes fit it
    (``tile_rows`` = query rows per workgroup, 0 = as many as fit 32 (row,
    head) columns; 1 suits steps of single decoded tokens), fp32 rows and
    other sizes through the plain kernel. ``key_splits`` (with tile_rows 1):
    workgroups that share one row's keys, merged by a second kernel; 0 = as
    many as fill the chip for this step (few rows, long windows), -1 = none."""
    if _gpu(q):
        T, H, C = q.shape[0], q.shape[1], q_abs.shape[2]
        out = torch.empty((T, H, C), dtype=q.dtype, device=q.device)
        ns = 1
        if tile_rows == 1 and use_mfma and q.dtype == torch.bfloat16 and key_splits >= 0:
            # an upper bound of a row's 32-key tiles, from the window or the block table's width
            reach = mask_size if mask_size > 0 else block_tables.shape[1] * cache.shape[2]
            reach = min(reach, block_tables.shape[1] * cache.shape[2])
            tiles = max(1, (reach + 31) // 32)
            groups = T * ((H + 31) // 32)
            # about four tiles per workgroup, and no more workgroups than two per compute unit
            ns = key_splits or max(1, min((tiles + 3) // 4, 512 // max(1, groups)))
            ns = max(1, min(ns, tiles, 64))
        f = torch.float32
        f_none = _none(q, f)
        part_o = torch.empty((T, H, ns, C), dtype=f, device=q.device) if ns > 1 else f_none
        part_ml = torch.empty((T, H, ns, 2), dtype=f, device=q.device) if ns > 1 else f_none
        _seq().attn_latent_paged(out, q_abs, q, cache, block_tables, token_seg, positions,
                                 gate if gate is not None else _none(q), float(scale), int(mask_size),
                                 int(nope_dim), int(tile_rows), bool(use_mfma), part_o, part_ml,
                                 sink if sink is not None else f_none)
        return out
    return torch_ref.attn_latent_paged(q_abs, q, cache, block_tables, token_seg, positions, scale, mask_size,
                                       gate, nope_dim, sink)


def sigmoid_gate_(x, gate) -> None:
    """x [T, C] *= sigmoid(gate) element by element; gate a row view."""
    if _gpu(x):
        _seq().sigmoid_gate(x, gate)
        return
    torch_ref.sigmoid_gate_(x, gate)


def attn_window_sink(q, st, batch, spec, gate):
    """Windowed attention with kept first tokens and a sink for one step's
    rows, keys through the block table (prompt portions, decoded tokens and
    mixes alike)."""
    return attn_masked_paged(q, st.k, st.v, batch.block_tables, batch.token_seg, batch.positions, spec.scale,
                             1, spec.mask_size, spec.keep_first, spec.sink, gate)


def ln_residual_mix(x_in, a, w_post, eps, x_out, streams=None, n_prev=0, dwa=None):
    """x_out = x_in + layernorm(a) * w_post (a None: x_in itself); with
    ``streams`` [L, T, W] the sum is kept as streams[n_prev] and x_out becomes
    sum_{j <= n_prev} dwa[j] * streams[j]. Returns the (mean, rstd) of every
    row of x_out, [T, 2] fp32 — what the next layer norm of the stream needs."""
    if _gpu(x_in):
        stats = torch.empty((x_in.shape[0], 2), dtype=torch.float32, device=x_in.device)
        f = _none(x_in, torch.float32)
        has = streams is not None
        _seq().ln_residual_mix(x_out, x_in, a if a is not None else f, w_post if a is not None else f, stats,
                               streams if has else f, dwa if has else f, int(n_prev), eps)
        return stats
    return torch_ref.ln_residual_mix(x_in, a, w_post, eps, x_out, streams, n_prev, dwa)


def ln_canon(x, stats, w_norm, canon_w, hist, state_slots, cu_seqlens, seg_start, token_seg, out_dtype):
    """Layer norm of the fp32 stream from its row statistics, times w_norm,
    plus the short causal convolution of that normed row with its
    predecessors (canon_w [K, W] taps-major; None = norm only); the
    sequence's last K-1 normed rows are carried in hist [slots, K-1, W] fp32."""
    if _gpu(x):
        out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
        f = _none(x, torch.float32)
        has = canon_w is not None
        i = _none(x, torch.int32)
        _seq().ln_canon(out, x, stats, w_norm, canon_w if has else f, hist if has else f,
                        state_slots if has else i, cu_seqlens if has else i, seg_start if has else i,
                        token_seg if has else i)
        return out
    return torch_ref.ln_canon(x, stats, w_norm, canon_w, hist, state_slots, cu_seqlens, seg_start, out_dtype)


def qk_fullnorm_rope_store(q, k, v, wq, wk, eps, positions, inv_freq, k_cache, v_cache, slot_mapping) -> None:
    """Whole-projection RMS norm of q (in place) and k, half-split rotation of
    the first 2 * len(inv_freq) entries of every head, normed rotated k and v
    into the paged caches. k None: q only."""
    if _gpu(q):
        e = _none(q)
        has = k is not None
        _seq().qk_fullnorm_rope_store(q, k if has else e, v if has else e, wq,
                                      wk if has else _none(q, torch.float32), eps, positions, inv_freq,
                                      k_cache if has else e, v_cache if has else e,
                                      slot_mapping if has else _none(q, torch.long))
        return
    torch_ref.qk_fullnorm_rope_store(q, k, v, wq, wk, eps, positions, inv_freq, k_cache, v_cache, slot_mapping)


def pool_kv_update(k_cache, v_cache, pool_k, pool_v, block_tables, token_seg, positions, run: int,
                   row_map=None) -> None:
    """Means of the cached keys / values of every aligned run of ``run``
    positions that one of this step's rows completes, into the fp32 pooled
    caches. ``row_map`` (int32): the rows to look at, when the caller knows
    which rows end a run; None = every row."""
    if _gpu(k_cache):
        _seq().pool_kv_update(k_cache, v_cache, pool_k, pool_v, block_tables, token_seg, positions, int(run),
                              row_map if row_map is not None else _none(k_cache, torch.int32))
        return
    torch_ref.pool_kv_update(k_cache, v_cache, pool_k, pool_v, block_tables, token_seg, positions, run, row_map)


def attn_window_pool_paged(q, k_cache, v_cache, pool_k, pool_v, block_tables, token_seg, positions, scale,
                           softcap, mask_size, run, key_splits: int = 0):
    """Sliding-window attention over the paged cache with the pooled entries
    of the runs that lie wholly before the window, soft-capped scores; prompt
    portions, decoded tokens and mixes alike. ``key_splits`` (GPU): workgroups
    that share one (row, head)'s keys, merged by a second kernel; 0 = as many
    as fill the chip for this step (few rows, long windows), 1 = none."""
    if _gpu(q):
        out = torch.empty((q.shape[0], q.shape[1], v_cache.shape[3]), dtype=q.dtype, device=q.device)
        f = _none(q, torch.float32)
        has = run > 0
        # steps of few rows: a (row, head)'s key tiles are shared out over several workgroups.
        # An upper bound of the visible keys, from the mask or the block table's width
        T, H = q.shape[0], q.shape[1]
        ctx = block_tables.shape[1] * k_cache.shape[2]
        reach = min(ctx, mask_size + (ctx // run if has else 0)) if mask_size > 0 else ctx
        tiles = (reach + 63) // 64
        ns = key_splits or max(1, min((tiles + 3) // 4, 512 // max(1, T * H), 64))
        part_o = torch.empty((T, H, ns, v_cache.shape[3]), dtype=torch.float32, device=q.device) if ns > 1 else f
        part_ml = torch.empty((T, H, ns, 2), dtype=torch.float32, device=q.device) if ns > 1 else f
        _seq().attn_masked_paged(out, q, k_cache, v_cache, block_tables, token_seg, positions, _none(q),
                                 scale, 2, int(mask_size), 0, False, _none(q, torch.int32),
                                 pool_k if has else f, pool_v if has else f, int(run), float(softcap),
                                 part_o, part_ml)
        return out
    return torch_ref.attn_window_pool_paged(q, k_cache, v_cache, pool_k, pool_v, block_tables, token_seg,
                                            positions, scale, softcap, mask_size, run)


def ssd_recurrence(x, B, C, dt, dt_bias, a_log, skip, state, state_slots, cu_seqlens, seg_start):
    """S <- exp(-exp(a_log) d) S + d B x^T, o = S^T C + skip x with
    d = softplus(dt + dt_bias) per head and token; o [T, H, V] fp32."""
    if _gpu(x):
        o = torch.empty((x.shape[0], x.shape[1], x.shape[2]), dtype=torch.float32, device=x.device)
        _seq().ssd_recurrence(o, x, B, C, dt, dt_bias, a_log, skip, state, state_slots, cu_seqlens, seg_start)
        return o
    return torch_ref.ssd_recurrence(x, B, C, dt, dt_bias, a_log, skip, state, state_slots, cu_seqlens, seg_start)


def gate_group_rmsnorm(o, weight, gate, eps, out_dtype):
    """(o * silu(gate)) RMS-normed in groups, times weight: o [T, groups, S] fp32."""
    if _gpu(o):
        out = torch.empty((o.shape[0], o.shape[1] * o.shape[2]), dtype=out_dtype, device=o.device)
        _seq().gated_rmsnorm(out, o, weight, gate, eps, 1)
        return out
    return torch_ref.gate_group_rmsnorm(o, weight, gate, eps, out_dtype)


RETENTION_CHUNK = 64          # rows per chunk of the chunk-parallel form
RETENTION_MAX_DIM = 128       # largest key size of the chunk-parallel form


def retention_chunks(segs, device):
    """Host metadata of the chunk-parallel form: segs = [(start position,
    rows)] of a step in row order -> (chunks [NC, 4] int32: first row, rows,
    segment, 0; seg_c0 [B + 1] int32: a segment's range of chunks)."""
    chunks, c0, row0 = [], [0], 0
    for b, (_, n) in enumerate(segs):
        chunks += [(row0 + i, min(RETENTION_CHUNK, n - i), b, 0) for i in range(0, n, RETENTION_CHUNK)]
        c0.append(len(chunks))
        row0 += n
    return (torch.tensor(chunks, dtype=torch.int32, device=device).reshape(-1, 4),
            torch.tensor(c0, dtype=torch.int32, device=device))


def retention(q, k, v, decay, positions, inv_freq, state, state_slots, cu_seqlens, seg_start, chunks=None):
    """Half-split rotation of q and k, k scaled by D^-1/2, then
    S <- decay_h S + k v^T, o = S^T q over segments; o [T, H, V] fp32.
    ``chunks`` (GPU, from retention_chunks): the chunk-parallel form; None:
    token by token."""
    if _gpu(q):
        o = torch.empty((q.shape[0], q.shape[1], v.shape[2]), dtype=torch.float32, device=q.device)
        e = _none(q, torch.int32)
        ch, c0 = chunks if chunks is not None else (e, e)
        _seq().retention(o, q, k, v, decay, positions, inv_freq, state, state_slots, cu_seqlens, seg_start, ch, c0)
        return o
    return torch_ref.retention(q, k, v, decay, positions, inv_freq, state, state_slots, cu_seqlens, seg_start)


def retention_mix_out(q, k, v, gate, decay, positions, inv_freq, state, state_slots, cu_seqlens, seg_start, eps,
                      out_dtype, chunks=None, single=False):
    """retention followed by the heads' RMS norm (no weight) and silu gate
    ([T, H*V] logits). ``single`` (GPU): every segment is one row (decode),
    the whole of it runs as one kernel."""
    V = v.shape[2]
    if single and _gpu(q) and q.shape[2] <= 1024 and (V <= 256 or (V % 4 == 0 and V <= 1024)):
        out = torch.empty((q.shape[0], q.shape[1] * V), dtype=out_dtype, device=q.device)
        _seq().retention_step(out, q, k, v, gate, decay, positions, inv_freq, state, state_slots, seg_start, eps)
        return out
    o = retention(q, k, v, decay, positions, inv_freq, state, state_slots, cu_seqlens, seg_start, chunks)
    return gated_rmsnorm(o, None, gate, eps, out_dtype, "silu")


def gelu_glu(gate, up):
    """gelu(gate) * up (tanh form) of two row views, in gate's dtype."""
    if _gpu(gate):
        out = torch.empty(gate.shape, dtype=gate.dtype, device=gate.device)
        _seq().gelu_glu(out, gate, up)
        return out
    return torch_ref.gelu_glu(gate, up)


def relu2(x):
    """max(x, 0)^2 of a [T, C] row view, in x's dtype."""
    if _gpu(x):
        out = torch.empty(x.shape, dtype=x.dtype, device=x.device)
        _seq().relu2(out, x)
        return out
    return torch_ref.relu2(x)


def gelu_mul_rows(z, table, ids, col0: int):
    """gelu(z [T, C]) * table[ids, col0 : col0 + C] in z's dtype."""
    if _gpu(z):
        out = torch.empty(z.shape, dtype=z.dtype, device=z.device)
        _seq().gelu_mul_rows(out, z, table, ids, int(col0))
        return out
    return torch_ref.gelu_mul_rows(z, table, ids, col0)


def add_cast(x, a, b, out_dtype):
    """x (fp32 residual, in place) += a + b (b may be None); returns x in
    out_dtype (fp32: x itself)."""
    if _gpu(x):
        out = x if out_dtype == torch.float32 else torch.empty(x.shape, dtype=out_dtype, device=x.device)
        _seq().add_cast(_none(x, out_dtype) if out is x else out, x, a, b if b is not None else _none(a))
        return out
    return torch_ref.add_cast(x, a, b, out_dtype)


def dyt_residual(x, a, post, nxt, out_dtype):
    """x (fp32 stream, in place) += tanh(alpha a) w + b with post = (alpha, w,
    b); returns tanh(alpha x) w + b with nxt, the next reader's input."""
    if _gpu(x):
        out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
        _seq().dyt_residual(out, x, a, *post, *nxt)
        return out
    return torch_ref.dyt_residual(x, a, post, nxt, out_dtype)


def embed_dyt(ids, table, scale: float, nxt):
    """The stream's start: (x, h) with x = table[ids] * scale in fp32 and h =
    tanh(alpha x) w + b with nxt in the table's dtype."""
    if _gpu(table):
        x = torch.empty((ids.numel(), table.shape[1]), dtype=torch.float32, device=table.device)
        h = torch.empty(x.shape, dtype=table.dtype, device=table.device)
        _seq().embed_dyt(h, x, ids, table, float(scale), *nxt)
        return x, h
    return torch_ref.embed_dyt(ids, table, scale, nxt)


def rmsnorm_rows(x, weight, eps):
    """RMS norm of a [T, C] row view, packed result in x's dtype."""
    if _gpu(x):
        out = torch.empty(x.shape, dtype=x.dtype, device=x.device)
        _seq().rmsnorm_rows(out, x, weight, eps)
        return out
    return torch_ref.rmsnorm_rows(x, weight, eps)


def conv_qkv_store(y, w, conv_state, state_slots, cu_seqlens, seg_start, token_seg, positions, q_cols, temp_coef,
                   temp_every, k_cols=None, v_cols=None, k_cache=None, v_cache=None, slot_mapping=None, single=False):
    """Short causal convolution of a fused projection's rows; k and v columns
    into the paged caches, the q columns times the query temperature returned
    packed [T, width]. ``single``: every segment is one row (the history is
    updated by the same launch)."""
    if _gpu(y):
        q = torch.empty((y.shape[0], q_cols[1]), dtype=y.dtype, device=y.device)
        has = k_cols is not None
        e = _none(y)
        ko, vo = (k_cols[0], v_cols[0]) if has else (0, 0)
        _seq().conv_qkv_store(q, y, w, conv_state, state_slots, cu_seqlens, seg_start, token_seg, positions,
                              int(q_cols[0]), float(temp_coef), int(temp_every), int(ko), int(vo),
                              k_cache if has else e, v_cache if has else e,
                              slot_mapping if has else _none(y, torch.long), bool(single))
        return q
    return torch_ref.conv_qkv_store(y, w, conv_state, state_slots, cu_seqlens, seg_start, positions, q_cols, temp_coef,
                                    temp_every, k_cols, v_cols, k_cache, v_cache, slot_mapping)


def diff_tile_rows(heads: int, kv_heads: int) -> int:
    """Query rows per workgroup of the matrix-unit kernel: four tiles of 32
    columns, of one head each, shared between consecutive rows and up to four
    heads of a key/value head."""
    r = heads // kv_heads
    return 32 if r >= 3 else 128 // r


def diff_tiles(segs, rows: int, device):
    """Host metadata of attn_diff_paged for a step of segments
    [(start position, rows)] in row order: (tiles [NT, 2] int32: first row,
    row count — pieces of at most ``rows`` rows of a segment with two rows or
    more, longest key ranges first; single [NS] int32: the rows of one-row
    segments). Either may be empty."""
    tiles, single, row0 = [], [], 0
    for start, n in segs:
        if n == 1:
            single.append(row0)
        else:
            tiles += [(start + min(n, i + rows), row0 + i, min(rows, n - i)) for i in range(0, n, rows)]
        row0 += n
    tiles = [(r, n) for _, r, n in sorted(tiles, reverse=True)]
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=device)
    return i32(tiles).reshape(-1, 2), i32(single)


def diff_key_splits(rows: int, groups: int, reach: int) -> int:
    """Workgroups that share one row's keys in the decode form: as many as
    fill the chip, at most one per 64-key tile."""
    tiles = max(1, (reach + 63) // 64)
    return max(1, min(tiles, (512 + rows * groups - 1) // max(1, rows * groups), 64))


def attn_diff_paged(q, k_cache, v_cache, block_tables, token_seg, positions, scale, lam, out_scale, eps, plan=None,
                    use_mfma: bool = True, key_splits: int = 0):
    """Differential attention over the paged cache (plain causal):
    rms(softmax_1 v - lam softmax_2 v) * out_scale per head, [T, H, V].
    GPU: bf16 goes through the matrix-unit kernels when the sizes fit them —
    ``plan`` = diff_tiles() of the step, None = every row on its own (decode) —
    and fp32 and other sizes through the plain kernel. ``key_splits``: see
    diff_key_splits (0 = by that rule)."""
    if _gpu(q):
        T, H, V = q.shape[0], q.shape[1], v_cache.shape[3]
        out = torch.empty((T, H, V), dtype=q.dtype, device=q.device)
        f, i = _none(q, torch.float32), _none(q, torch.int32)
        mfma = use_mfma and q.dtype == torch.bfloat16 and _seq().attn_diff_mfma_fits(q.shape[2] // 2, V)
        args = (out, q, k_cache, v_cache, block_tables, token_seg, positions, float(scale), float(lam),
                float(out_scale), float(eps))
        if not mfma:
            _seq().attn_diff_paged(*args, 0, i, f, f)
            return out
        tiles, single = plan if plan is not None else (i, i)
        if tiles.numel():
            _seq().attn_diff_paged(*args, 1, tiles, f, f)
        n = T if plan is None else single.numel()
        if n:
            reach = block_tables.shape[1] * k_cache.shape[2]
            ns = key_splits or diff_key_splits(n, k_cache.shape[1], reach)
            part_o = torch.empty((n, H, 2, ns, V), dtype=torch.float32, device=q.device)
            part_ml = torch.empty((n, H, 2, ns, 2), dtype=torch.float32, device=q.device)
            _seq().attn_diff_paged(*args, 2, single, part_o, part_ml)
        return out
    return torch_ref.attn_diff_paged(q, k_cache, v_cache, block_tables, token_seg, positions, scale, lam, out_scale,
                                     eps)
