"""HIP kernels of the Dimuvik family (kllms_amd._C_seq) against the plain
PyTorch reference of the same op (ops/torch_ref.py), in fp32 and bf16, on
sizes that are and are not multiples of the vector and matrix-tile sizes, with
segments that start a sequence, continue one, and end inside a key tile."""

import pytest
import torch

from kllms_amd import ops
from kllms_amd.ops import torch_ref

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


def norm_args(W, alpha, seed):
    return torch.tensor([alpha], device=DEV), 1.0 + rnd(W, std=0.3, seed=seed), rnd(W, std=0.3, seed=seed + 1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W", [(1, 8), (5, 20), (3, 2048), (70, 96), (9000, 24), (2, 5120), (33, 7)])
def test_dyt_residual(dtype, T, W):
    x, a = rnd(T, W, std=3.0), rnd(T, W, dtype=dtype, std=2.0, seed=1)
    post, nxt = norm_args(W, 0.7, 2), norm_args(W, 0.3, 4)
    x1, x2 = x.clone(), x.clone()
    close(ops.dyt_residual(x1, a, post, nxt, dtype), torch_ref.dyt_residual(x2, a, post, nxt, dtype), dtype)
    torch.testing.assert_close(x1, x2, rtol=1e-6, atol=2e-6)                # the stream is fp32 in both modes
    table, ids = rnd(50, W, dtype=dtype, seed=6), torch.randint(0, 50, (T,), generator=torch.Generator().manual_seed(7)).to(DEV)
    (x3, h3), (x4, h4) = ops.embed_dyt(ids, table, 1.7, nxt), torch_ref.embed_dyt(ids, table, 1.7, nxt)
    torch.testing.assert_close(x3, x4, rtol=1e-6, atol=1e-6)
    close(h3, h4, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,C,pad", [(1, 24, 0), (7, 80, 48), (130, 768, 8), (5, 13, 3), (3, 1536, 0)])
def test_rmsnorm_rows(dtype, T, C, pad):
    x = rnd(T, C + pad, dtype=dtype, std=0.01)[:, :C]                       # small rows: eps matters
    w = 1.0 + rnd(C, std=0.2, seed=3)
    close(ops.rmsnorm_rows(x, w, 1e-5), torch_ref.rmsnorm_rows(x, w, 1e-5), dtype)


def paged(starts, lengths, G, D2, V, BS, dtype, seed=0):
    """Caches with random content, shuffled block tables, flat slots of the step's rows."""
    nb = [(s + n + BS - 1) // BS for s, n in zip(starts, lengths)]
    perm = torch.randperm(sum(nb) + 3, generator=torch.Generator().manual_seed(seed)).tolist()
    bt = torch.zeros(len(nb), max(nb), dtype=torch.int32)
    pos, seg, slots, at = [], [], [], 0
    for b, n in enumerate(nb):
        bt[b, :n] = torch.tensor(perm[at:at + n], dtype=torch.int32)
        at += n
        for p in range(starts[b], starts[b] + lengths[b]):
            pos.append(p)
            seg.append(b)
            slots.append(int(bt[b, p // BS]) * BS + p % BS)
    k = rnd(sum(nb) + 3, G, BS, D2, dtype=dtype, seed=seed + 1)
    v = rnd(sum(nb) + 3, G, BS, V, dtype=dtype, seed=seed + 2)
    return dict(k=k, v=v, bt=bt.to(DEV), pos=torch.tensor(pos, device=DEV), seg=i32(seg),
                slots=torch.tensor(slots, device=DEV), segs=list(zip(starts, lengths)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("K", [1, 2, 4, 6])
@pytest.mark.parametrize("H,G,D2,V,BS", [(4, 2, 16, 24, 16), (3, 3, 10, 7, 4), (6, 1, 32, 40, 16), (1, 1, 6, 8, 8)])
@pytest.mark.parametrize("own", [True, False])
def test_conv_qkv_store(dtype, K, H, G, D2, V, BS, own):
    starts, lengths = [0, 9, 0, 30, 2], [37, 1, 2, 3, 1]
    for single in (False, True):
        ln = [1] * 5 if single else lengths
        c = paged(starts, ln, G, D2, V, BS, dtype, seed=K + H)
        al = lambda n: (n + 7) // 8 * 8
        q_cols, k_cols = (0, H * D2), (al(H * D2), G * D2)
        v_cols = (k_cols[0] + al(G * D2), G * V)
        C = v_cols[0] + al(G * V) if own else al(H * D2)
        y, w = rnd(sum(ln), C, dtype=dtype), rnd(K, C, std=0.5, seed=5)
        hist = rnd(7, K - 1, C, dtype=dtype, seed=6)
        cu = i32([0] + torch.tensor(ln).cumsum(0).tolist())
        slots, seg_start = i32([3, 0, 6, 1, 4]), i32(starts)
        h1, h2 = hist.clone(), hist.clone()
        k1, k2, v1, v2 = c["k"].clone(), c["k"].clone(), c["v"].clone(), c["v"].clone()
        kv = lambda k, v: (k_cols, v_cols, k, v, c["slots"]) if own else (None, None, None, None, None)
        q1 = ops.conv_qkv_store(y, w, h1, slots, cu, seg_start, c["seg"], c["pos"], q_cols, 0.35, 8, *kv(k1, v1), single)
        q2 = torch_ref.conv_qkv_store(y, w, h2, slots, cu, seg_start, c["pos"], q_cols, 0.35, 8, *kv(k2, v2))
        close(q1, q2, dtype)
        close(k1, k2, dtype)
        close(v1, v2, dtype)
        cols = [torch.arange(o, o + n) for o, n in ((q_cols, k_cols, v_cols) if own else (q_cols,))]
        cols = torch.cat(cols).to(DEV)
        assert torch.equal(h1[..., cols], h2[..., cols])           # carried rows are copies
        assert torch.equal(h1[[2, 5]], hist[[2, 5]])               # slots no segment names stay as they were


SIZES = [(4, 2, 8, 24), (3, 3, 48, 104), (4, 1, 64, 64), (8, 2, 128, 256), (6, 2, 40, 72), (5, 1, 16, 8), (2, 1, 128, 32),
         (1, 1, 24, 200), (2, 2, 5, 7), (40, 1, 8, 16), (3, 1, 136, 40), (4, 4, 32, 136)]


def diff_case(dtype, H, G, D, V, BS, starts, lengths, seed=0, std=1.0):
    c = paged(starts, lengths, G, 2 * D, V, BS, dtype, seed)
    c["q"] = rnd(sum(lengths), H, 2 * D, dtype=dtype, std=std, seed=seed + 3)
    c["args"] = (c["q"], c["k"], c["v"], c["bt"], c["seg"], c["pos"], 1.3 * D ** -0.5, 0.6, 0.7, 1e-5)
    return c


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V", SIZES)
def test_attn_diff_over_segments(dtype, H, G, D, V):
    """Portions that start and end inside, at and after 64-key tiles and
    32-row query tiles, single rows between them, through every form."""
    starts = [0, 63, 0, 64, 127, 5, 200, 31, 0]
    lengths = [130, 1, 2, 65, 1, 33, 3, 1, 1]
    c = diff_case(dtype, H, G, D, V, 16, starts, lengths, seed=H + D)
    want = torch_ref.attn_diff_paged(*c["args"])
    plan = ops.diff_tiles(c["segs"], ops.diff_tile_rows(H, G), DEV)
    close(ops.attn_diff_paged(*c["args"], plan=plan), want, dtype, 1.0 if dtype == torch.float32 else 2.0)
    close(ops.attn_diff_paged(*c["args"], plan=plan, use_mfma=False), want, dtype)
    close(ops.attn_diff_paged(*c["args"], plan=None), want, dtype, 1.0 if dtype == torch.float32 else 2.0)


@pytest.mark.parametrize("splits", [0, 1, 2, 5, 64])
@pytest.mark.parametrize("H,G,D,V,BS", [(8, 2, 128, 256, 16), (4, 4, 40, 88, 4), (3, 1, 16, 40, 64)])
def test_attn_diff_single_rows_and_key_shares(splits, H, G, D, V, BS):
    """Decode: rows of very different lengths; more shares than a short row has tiles."""
    starts = [0, 1, 63, 64, 65, 700, 333]
    c = diff_case(torch.bfloat16, H, G, D, V, BS, starts, [1] * 7, seed=splits)
    close(ops.attn_diff_paged(*c["args"], key_splits=splits), torch_ref.attn_diff_paged(*c["args"]), torch.bfloat16, 2.0)


def test_attn_diff_weights_keep_more_than_bf16():
    """Two maps that nearly cancel: what is left is right to bf16's precision
    of the values although the norm blows it up."""
    H, G, D, V = 2, 1, 32, 64
    c = diff_case(torch.bfloat16, H, G, D, V, 16, [0, 90], [100, 1], seed=5, std=0.2)
    q = c["q"].clone()
    q[:, :, D:] = q[:, :, :D]
    c["k"][..., D:] = c["k"][..., :D]
    args = (q, c["k"], c["v"], c["bt"], c["seg"], c["pos"], 0.2, 0.98, 0.5, 1e-5)
    want = torch_ref.attn_diff_paged(*args).float()
    plan = ops.diff_tiles(c["segs"], ops.diff_tile_rows(H, G), DEV)
    for got in (ops.attn_diff_paged(*args, plan=plan), ops.attn_diff_paged(*args, plan=None)):
        assert float((got.float() - want).pow(2).mean().sqrt()) < 0.01


def test_diff_tiles_plan():
    tiles, single = ops.diff_tiles([(5, 1), (0, 70), (9, 1), (0, 0), (100, 2)], 32, DEV)
    assert single.tolist() == [0, 71]
    assert tiles.tolist() == [[72, 2], [65, 6], [33, 32], [1, 32]]


@pytest.mark.parametrize("T,N,top", [(1, 4, 2), (33, 9, 4), (5, 6, 6)])
def test_route_scale_and_ungated_shared_expert(T, N, top):
    z, corr = rnd(T, N), rnd(N, std=0.3, seed=1)
    i1, w1 = ops.moe_route(z, corr, top, 1, 1, "softmax", False, 1.9)
    i2, w2 = torch_ref.moe_route(z, corr, top, 1, 1, "softmax", False, 1.9)
    assert torch.equal(i1, i2)
    close(w1, w2, torch.float32)
    for W in (16, 13):
        rows, h, extra = rnd(T * top, W), rnd(T, W, seed=2), rnd(T, W, seed=3)
        ridx = torch.arange(T * top, dtype=torch.int32, device=DEV).view(T, top)
        close(ops.moe_combine(rows, h, ridx, w1, torch.float32, extra, None),
              torch_ref.moe_combine(rows, h, ridx, w1, torch.float32, extra, None), torch.float32)
