"""HIP kernels of the Bavesun family (kllms_amd._C_seq) against the plain
PyTorch reference of the same op (ops/torch_ref.py), in fp32 and bf16, on
sizes that are and are not multiples of the vector and matrix-tile sizes, with
segments that start a sequence, continue one, and end inside a chunk."""

import pytest
import torch

from kllms_amd import ops
from kllms_amd.ops import torch_ref
from test_gpu_mitunex_kernels import _latent_case

pytestmark = pytest.mark.gpu

DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


def close(a, b, dtype, scale=1.0):
    rt, at = (2e-5, 2e-5) if dtype == torch.float32 else (2e-2, 2e-2)
    torch.testing.assert_close(a.float(), b.float(), rtol=rt * scale, atol=at * scale)


def rnd(*shape, dtype=torch.float32, std=1.0, seed=0):
    g = torch.Generator(device="cpu").manual_seed(seed + sum(shape))
    return (torch.randn(*shape, generator=g) * std).to(DEV).to(dtype)


def i32(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


def retention_case(dtype, H, D, V, R2, lengths, starts, slots, seed=0):
    T = sum(lengths)
    hd, hv = H * D, H * V
    pad = lambda n: (n + 7) // 8 * 8
    buf = rnd(T, 2 * pad(hd) + 2 * pad(hv), dtype=dtype, seed=seed)           # one projection's row, four parts
    o = [0, pad(hd), 2 * pad(hd), 2 * pad(hd) + pad(hv)]
    q, k = (buf[:, a:a + hd].unflatten(1, (H, D)) for a in o[:2])
    v, g = buf[:, o[2]:o[2] + hv].unflatten(1, (H, V)), buf[:, o[3]:o[3] + hv]
    cu = [0]
    for n in lengths:
        cu.append(cu[-1] + n)
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lengths)]).to(DEV)
    decay = torch.tensor([1.0 - 2.0 ** -(1 + 1.7 * h) for h in range(H)], device=DEV)
    inv = (500.0 ** (-torch.arange(R2, dtype=torch.float64) / max(R2, 1))).float().to(DEV)
    state = rnd(max(slots) + 2, H, D, V, seed=seed + 1)
    return dict(q=q, k=k, v=v, gate=g, decay=decay, pos=pos, inv=inv, state=state, slots=i32(slots), cu=i32(cu),
                start=i32(starts), segs=list(zip(starts, lengths)))


SIZES = [(4, 64, 32, 32), (3, 20, 12, 6), (2, 128, 128, 64), (5, 32, 48, 8), (2, 7, 5, 2), (1, 16, 136, 0), (3, 96, 40, 48)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,V,R2", SIZES)
@pytest.mark.parametrize("form", ["tokens", "chunks"])
def test_retention_over_segments(dtype, H, D, V, R2, form):
    """Fresh and continued sequences; portions of one, two, a chunk less one,
    exactly one and several chunks, one row more than a chunk."""
    lengths, starts, slots = [70, 1, 2, 64, 63, 200, 65, 33], [0, 7, 0, 5, 1000, 0, 64, 128], [2, 0, 4, 1, 3, 6, 5, 7]
    c = retention_case(dtype, H, D, V, R2, lengths, starts, slots, seed=H + D)
    s1, s2 = c["state"].clone(), c["state"].clone()
    chunks = ops.retention_chunks(c["segs"], DEV) if form == "chunks" else None
    args = (c["slots"], c["cu"], c["start"])
    o1 = ops.retention(c["q"], c["k"], c["v"], c["decay"], c["pos"], c["inv"], s1, *args, chunks)
    o2 = torch_ref.retention(c["q"], c["k"], c["v"], c["decay"], c["pos"], c["inv"], s2, *args)
    torch.testing.assert_close(o1, o2, rtol=1e-4, atol=2e-4)
    torch.testing.assert_close(s1, s2, rtol=1e-4, atol=2e-4)
    assert torch.equal(s1[8], c["state"][8])                     # a slot no segment names stays as it was


def test_retention_decay_of_zero_and_one():
    """A head that forgets everything and one that forgets nothing."""
    c = retention_case(torch.float32, 2, 32, 32, 16, [130, 5], [0, 3], [1, 0], seed=9)
    c["decay"] = torch.tensor([0.0, 1.0], device=DEV)
    s1, s2 = c["state"].clone(), c["state"].clone()
    args = (c["slots"], c["cu"], c["start"])
    o1 = ops.retention(c["q"], c["k"], c["v"], c["decay"], c["pos"], c["inv"], s1, *args,
                       ops.retention_chunks(c["segs"], DEV))
    o2 = torch_ref.retention(c["q"], c["k"], c["v"], c["decay"], c["pos"], c["inv"], s2, *args)
    torch.testing.assert_close(o1, o2, rtol=1e-4, atol=5e-4)
    torch.testing.assert_close(s1, s2, rtol=1e-4, atol=5e-4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,V,R2", SIZES)
def test_retention_step(dtype, H, D, V, R2):
    """Decode in one kernel: update, read-out, head norm and gate."""
    B = 6
    c = retention_case(dtype, H, D, V, R2, [1] * B, [0, 9, 300, 0, 1, 70000], [3, 0, 5, 1, 2, 4], seed=V)
    s1, s2 = c["state"].clone(), c["state"].clone()
    args = (c["slots"], c["cu"], c["start"], 1e-5, dtype)
    a = ops.retention_mix_out(c["q"], c["k"], c["v"], c["gate"], c["decay"], c["pos"], c["inv"], s1, *args, single=True)
    o = torch_ref.retention(c["q"], c["k"], c["v"], c["decay"], c["pos"], c["inv"], s2, *args[:3])
    b = torch_ref.gated_rmsnorm(o, None, c["gate"], 1e-5, dtype, "silu")
    # the angle of the far position: a few fp32 roundings of it move sin and cos
    close(a, b, dtype, scale=10 if dtype == torch.float32 else 1)
    torch.testing.assert_close(s1, s2, rtol=1e-4, atol=1e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("G,S", [(4, 32), (3, 20), (2, 128), (1, 1000), (5, 7)])
def test_head_norm_without_weight_silu_gate(dtype, G, S):
    o = rnd(9, G, S, std=2.0)
    gate = rnd(9, G * S + 8, dtype=dtype, seed=1)[:, :G * S]
    w = rnd(S, seed=2) * 0.1 + 1
    for weight, act in [(None, "silu"), (w, "silu"), (None, "sigmoid"), (w, "sigmoid")]:
        close(ops.gated_rmsnorm(o, weight, gate, 1e-5, dtype, act),
              torch_ref.gated_rmsnorm(o, weight, gate, 1e-5, dtype, act), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cols,stride", [(40, 40), (37, 48), (1024, 2056)])
def test_elementwise_activations(dtype, cols, stride):
    buf = rnd(6, 2 * stride, dtype=dtype, std=2.0)
    a, b = buf[:, :cols], buf[:, stride:stride + cols]
    close(ops.gelu_glu(a, b), torch_ref.gelu_glu(a, b), dtype)
    close(ops.relu2(a), torch_ref.relu2(a), dtype)
    x1, x2 = a.clone(), a.clone()
    ops.sigmoid_gate_(x1, b)
    torch_ref.sigmoid_gate_(x2, b)
    close(x1, x2, dtype)
    z = torch.tensor([[-60.0, -9.0, -1e-3, 0.0, 1e-3, 9.0, 60.0, 1e4]], device=DEV, dtype=dtype)
    close(ops.gelu_glu(z, torch.ones_like(z)), torch_ref.gelu_glu(z, torch.ones_like(z)), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,layers", [(16, 3), (5, 4), (128, 2)])
def test_gelu_times_a_tokens_columns(dtype, dim, layers):
    table = rnd(11, dim * layers, dtype=dtype)
    z = rnd(7, dim, dtype=dtype, seed=1)
    ids = torch.tensor([10, 0, 3, 3, 7, 1, 9], device=DEV)
    for i in range(layers):
        close(ops.gelu_mul_rows(z, table, ids, i * dim), torch_ref.gelu_mul_rows(z, table, ids, i * dim), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [36, 37, 2048])
def test_add_branches_and_cast(dtype, W):
    a, b = rnd(5, W, dtype=dtype), rnd(5, W, dtype=dtype, seed=1)
    for bb in (b, None):
        x1 = rnd(5, W, std=3.0, seed=2)
        x2 = x1.clone()
        h1, h2 = ops.add_cast(x1, a, bb, dtype), torch_ref.add_cast(x2, a, bb, dtype)
        close(x1, x2, torch.float32)
        close(h1, h2, dtype)
        assert h1.dtype == dtype and (dtype != torch.float32 or h1 is x1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,top", [(12, 3), (16, 4), (7, 1), (3, 3), (130, 20)])
def test_route_by_logits(dtype, N, top):
    """The choice is made on the logits (also where their softmax over all
    outputs would underflow), the weights are the softmax over the chosen."""
    T, W = 11, 72
    h = rnd(T, W, dtype=dtype)
    router = rnd(N, W, seed=1) * 0.3
    router[0] *= 100.0                                           # one output far above (or below) the rest
    z = torch.nn.functional.linear(h.float(), router)
    idx, w, rowidx = ops.moe_route_rows(h, router, None, top, 1, 1, N, True, "top_softmax", True)
    ridx, rw = torch_ref.moe_route(z, None, top, 1, 1, "top_softmax", True)
    assert torch.equal(idx, ridx) and torch.equal(ridx, torch.topk(z, top).indices.int())
    close(w, rw, torch.float32, scale=10)
    close(rw, torch.softmax(torch.topk(z, top).values, -1), torch.float32, scale=10)
    assert torch.equal(rowidx, ridx * T + torch.arange(T, device=DEV, dtype=torch.int32)[:, None])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,R,C", [(4, 16, 8, 32), (3, 20, 6, 44), (16, 32, 64, 512), (40, 8, 8, 16), (1, 8, 4, 96)])
@pytest.mark.parametrize("mask", [0, 7])
def test_latent_attention_with_a_sink(dtype, H, D, R, C, mask):
    """Sinks from negligible to dominating, per head, in every launch form."""
    c = _latent_case(dtype, H, D, R, C, 16, [33, 1, 2, 1, 70], [0, 52, 15, 0, 45], seed=H + C)
    sink = torch.linspace(-40.0, 12.0, H).to(DEV) if H > 1 else torch.tensor([1.5], device=DEV)
    call = lambda f, s, **kw: f(c["q_abs"], c["q"], c["cache"], c["bt"], c["tseg"], c["pos"], 0.17, mask, None, D,
                                sink=s, **kw)
    ref = call(torch_ref.attn_latent_paged, sink)
    assert float((ref.float() - call(torch_ref.attn_latent_paged, None).float()).abs().max()) > 0.05
    for kw in [dict(use_mfma=False), dict(tile_rows=0), dict(tile_rows=1, key_splits=-1), dict(tile_rows=1),
               dict(tile_rows=1, key_splits=3), dict(tile_rows=1, key_splits=50)]:
        close(call(ops.attn_latent_paged, sink, **kw), ref, dtype)
