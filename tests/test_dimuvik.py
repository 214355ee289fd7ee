"""Dimuvik family on the CPU path (fp32) against the plain float64 oracle in
tests/dimuvik_oracle.py: every mechanism alone, then whole models through the
engine's segment step, page and slot reuse, and greedy generation through
generate() and the scheduler. Configurations are small and lopsided: head
counts that are not powers of two, value sizes that differ from key sizes,
one to six taps, a reading layer with another temperature and scale than the
layer it reads, layers without a feed-forward, top 1 and top = all."""

import json
import math
import os

import pytest
import torch

import dimuvik_oracle as O
from kllms_amd import ops
from kllms_amd.engine.config import DimuvikArchConfig, EngineConfig
from kllms_amd.engine.engine import GenRequest, LLMEngine
from kllms_amd.engine.sampling import SamplingParams
from kllms_amd.engine.scheduler import BatchScheduler
from kllms_amd.models.mixers import ActFF, DiffAttention, DynamicTanh, LatentAttention, RoutedExperts
from test_pironex import check, load_module, rows, run_mixers, toks

EPS = 1e-5


def att(heads=4, kv_heads=2, dim=6, vdim=10, conv=3, diff=0.4, scale=0.5, coef=0.5, every=16, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "diff": diff, "scale": scale,
         "q_temp": {"coef": coef, "every": every}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def lat(heads=3, dim=9, rot_dim=6, vdim=7, kv_rank=12, q_rank=11, scale=0.3, base=100.0):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
            "scale": scale, "rot": {"base": base, "dims": rot_dim}}


MLPS = {
    None: None,
    "dense": {"kind": "dense", "ff": 28},
    "moe": {"kind": "moe", "expert": {"ff": 11}, "router": {"experts": 6, "top": 3, "scale": 1.7}, "shared": {"ff": 17}},
    "moe_top1": {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 5, "top": 1, "scale": 1.0}},
    "moe_all": {"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 3, "top": 3, "scale": 0.6}, "shared": {"ff": 8}},
}


def layer(kind, mixer, mlp="dense"):
    return {"type": kind, "mixer": mixer, "mlp": MLPS[mlp]}


def model_cfg(layers, vocab=61, width=24, eps=EPS, scale=1.7):
    return {"architecture": "Dimuvik", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": layers}


# two layers read the cache of layer 1, one of them with a latent layer between; grouped heads
CFG_A = model_cfg([layer("latent_attention", lat(), "moe"),
                   layer("attention", att(), "dense"),
                   layer("attention", att(conv=2, diff=0.7, scale=0.8, coef=0.2, every=5, kv_from=1), "moe"),
                   layer("latent_attention", lat(heads=2, dim=4, rot_dim=2, vdim=5, kv_rank=10, q_rank=6, scale=0.7), None),
                   layer("attention", att(conv=5, diff=0.1, scale=0.6, kv_from=1), "moe_top1")])
# attention first, ungrouped heads, six taps and one tap, no temperature, odd sizes, no shared expert, unscaled embedding
CFG_B = model_cfg([layer("attention", att(heads=3, kv_heads=3, dim=5, vdim=7, conv=6, coef=0.0), "moe_top1"),
                   layer("attention", att(heads=3, kv_heads=3, dim=5, vdim=7, conv=1, diff=0.8, every=1, kv_from=0), None),
                   layer("latent_attention", lat(heads=1, dim=6, rot_dim=4, vdim=5, kv_rank=7, q_rank=20, scale=0.9), "moe_all"),
                   layer("attention", att(heads=4, kv_heads=1, dim=4, vdim=3, conv=2, diff=0.0, every=7), "dense")],
                  vocab=47, width=20, eps=1e-6, scale=1.0)


def write_model(tmp, cfg, seed=0, w=None):
    from safetensors.torch import save_file

    w = w if w is not None else O.random_weights(cfg, seed)
    os.makedirs(tmp, exist_ok=True)
    save_file({k: v.bfloat16().contiguous() for k, v in w.items()}, os.path.join(tmp, "model.safetensors"))
    with open(os.path.join(tmp, "config.json"), "w") as f:
        json.dump(cfg, f)
    return w


def make_engine(path, blocks=64, slots=4, **kw):
    return LLMEngine(EngineConfig(model=str(path), dtype="float32", device="cpu", max_kv_blocks=blocks,
                                  max_state_slots=slots, use_hip_graphs=False, **kw))


@pytest.fixture(scope="module")
def model_a(tmp_path_factory):
    d = tmp_path_factory.mktemp("dim_a")
    w = write_model(str(d), CFG_A, seed=1)
    return CFG_A, w, make_engine(d, blocks=96, kv_block_size=4)


@pytest.fixture(scope="module")
def model_b(tmp_path_factory):
    d = tmp_path_factory.mktemp("dim_b")
    w = write_model(str(d), CFG_B, seed=2)
    return CFG_B, w, make_engine(d, blocks=24, slots=3, kv_block_size=8)


def specs_of(layers, width=24):
    return DimuvikArchConfig.from_checkpoint_config(model_cfg(layers, width=width)).layers


def mixer_of(layers, i, w, width=24):
    sp = specs_of(layers, width)[i]
    if sp.type == "attention":
        mod = DiffAttention(sp.attention, width, EPS, torch.float32)
    else:
        mod = LatentAttention(sp.latent, width, EPS, torch.float32)
    load_module(mod, w, f"l{i}.mix.")
    if sp.type == "attention":
        mod.fold()
    return mod


# --- mechanisms alone -----------------------------------------------------------------

CUTS = [[60], [25] + [1] * 35, [2, 5, 16, 1, 2, 17, 3, 14], [2] * 30, [1] * 60]


def run_mixer(lay, w, h, cuts, page=4):
    return run_mixers([mixer_of([lay], 0, w)], h, cuts, page)[0]


def test_dynamic_tanh():
    """No mean or variance: rows of any scale pass elementwise, each norm with
    its own slope, weight and bias."""
    x, a = rows(5, 24, 1) * torch.logspace(-3, 2, 5, dtype=torch.float64)[:, None], rows(5, 24, 2) * 3.0
    w = {}
    for i, n in enumerate(("post", "next")):
        w[n], w[n + ".b"] = 1.0 + 0.3 * rows(1, 24, 3 + i)[0], 0.3 * rows(1, 24, 5 + i)[0]
        w[n + ".alpha"] = torch.tensor([0.8, -0.3][i], dtype=torch.float64)
    mods = {}
    for n in ("post", "next"):
        mods[n] = DynamicTanh(24)
        for name, dst in mods[n].checkpoint_map(n).items():
            dst.copy_(w[name].reshape(dst.shape).float())
    xs = x.float()
    h = ops.dyt_residual(xs, a.float(), mods["post"].args, mods["next"].args, torch.float32)
    want = x + O.dyt(w, "post", a)
    check(xs, want, atol=1e-5)
    check(h, O.dyt(w, "next", want), atol=1e-5)
    x0, h0 = ops.embed_dyt(torch.tensor([3, 0, 3]), x.float(), 1.7, mods["next"].args)
    check(x0, x[[3, 0, 3]] * 1.7, atol=1e-5)
    check(h0, O.dyt(w, "next", x[[3, 0, 3]] * 1.7), atol=1e-5)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,conv", [(4, 2, 6, 10, 3), (3, 3, 5, 7, 1), (4, 1, 3, 2, 6), (1, 1, 8, 16, 4)])
def test_diff_attention(cuts, heads, kv_heads, dim, vdim, conv):
    lay = layer("attention", att(heads, kv_heads, dim, vdim, conv, scale=1.5), None)
    w = O.random_weights(model_cfg([lay]), 3)
    h = rows(sum(cuts), 24, 4)
    check(run_mixer(lay, w, h, cuts), O.attention(w, "l0.mix.", lay["mixer"], h, EPS))


def test_short_convolution_across_portions_and_the_start():
    """Rows before the sequence count as zero whatever the slot held; biases
    enter the carried rows (they are added before the convolution)."""
    taps, u = rows(5, 3, 6), rows(7, 5, 7)
    y = O.short_conv(u, taps)
    check(y[0], taps[:, 2] * u[0], atol=1e-12)
    check(y[4], taps[:, 0] * u[2] + taps[:, 1] * u[3] + taps[:, 2] * u[4], atol=1e-12)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32)
    hist = torch.full((2, 2, 5), 9.0)
    got = []
    for start, n in [(0, 1), (1, 1), (2, 3), (5, 2)]:
        got.append(ops.conv_qkv_store(u[start:start + n].float(), taps.t().contiguous().float(), hist, i32([1]), i32([0, n]),
                                      i32([start]), i32([0] * n), torch.arange(start, start + n), (0, 5), 0.0, 1))
    check(torch.cat(got), y, atol=1e-5)
    assert torch.equal(hist[0], torch.full((2, 5), 9.0)) and torch.equal(hist[1], u[5:7].float())
    lay = layer("attention", att(), None)
    w = O.random_weights(model_cfg([lay]), 8)
    w["l0.mix.k.b"] = w["l0.mix.k.b"] + 2.0
    h = rows(9, 24, 9)
    check(run_mixer(lay, w, h, [1, 1, 2, 5]), O.attention(w, "l0.mix.", lay["mixer"], h, EPS))


@pytest.mark.parametrize("coef,every", [(0.5, 4), (1.3, 1), (0.4, 7)])
def test_query_temperature_steps_at_its_edges(coef, every):
    """Constant up to position every - 2, the next step at every - 1."""
    assert O.query_temperature(every - 2, coef, every) == 1.0 or every == 1
    assert abs(O.query_temperature(every - 1, coef, every) - (1 + coef * math.log(2))) < 1e-12
    assert abs(O.query_temperature(3 * every - 1, coef, every) - (1 + coef * math.log(4))) < 1e-12
    i32 = lambda x: torch.tensor(x, dtype=torch.int32)
    n = 4 * every + 1
    q = ops.conv_qkv_store(torch.ones(n, 2), torch.ones(1, 2), torch.zeros(1, 0, 2), i32([0]), i32([0, n]), i32([0]), i32([0] * n),
                           torch.arange(n), (0, 2), coef, every)
    check(q[:, 0], torch.tensor([O.query_temperature(p, coef, every) for p in range(n)], dtype=torch.float64), atol=1e-6)
    lay = layer("attention", att(coef=coef, every=every, scale=1.0), None)
    w = O.random_weights(model_cfg([lay]), 10)
    h = rows(n, 24, 11)
    want = O.attention(w, "l0.mix.", lay["mixer"], h, EPS)
    flat = dict(lay["mixer"], q_temp={"coef": 0.0, "every": every})
    assert float((O.attention(w, "l0.mix.", flat, h, EPS) - want)[-1].abs().max()) > 1e-2
    check(run_mixer(lay, w, h, [every, n - every]), want)


@pytest.mark.parametrize("diff", [0.0, 0.5, 0.9])
def test_lambda_and_the_norm_of_the_difference(diff):
    """lambda from its four vectors and the constant; the difference is normed
    per head with eps inside the root (tiny values: eps decides)."""
    lay = layer("attention", att(diff=diff), None)
    w = O.random_weights(model_cfg([lay]), 12)
    w["l0.mix.lq1"] = torch.full((6,), 0.5, dtype=torch.float64)
    w["l0.mix.lk1"] = torch.full((6,), 0.25, dtype=torch.float64)
    w["l0.mix.lq2"], w["l0.mix.lk2"] = w["l0.mix.lq1"] * -1.0, w["l0.mix.lk1"]
    mod = mixer_of([lay], 0, w)
    assert abs(mod.lam - (math.exp(0.75) - math.exp(-0.75) + diff)) < 1e-6
    w["l0.mix.v"], w["l0.mix.v.b"] = w["l0.mix.v"] * 1e-3, w["l0.mix.v.b"] * 1e-3
    h = rows(20, 24, 13)
    want = O.attention(w, "l0.mix.", lay["mixer"], h, EPS)
    assert float((O.attention(w, "l0.mix.", lay["mixer"], h, 1e-9) - want).abs().max()) > 1e-2
    check(run_mixer(lay, w, h, [13, 7]), want)


def test_maps_and_heads_lie_head_by_head():
    """Swapping the two maps of one head changes that head alone, as the
    oracle says; a plain difference of the maps would not see the swap's sign."""
    lay = layer("attention", att(heads=2, kv_heads=1, dim=4, vdim=5, diff=0.3), None)
    w = O.random_weights(model_cfg([lay]), 14)
    w["l0.mix.o"] = torch.eye(24, 10, dtype=torch.float64)
    h = rows(18, 24, 15)
    want = O.attention(w, "l0.mix.", lay["mixer"], h, EPS)
    other = dict(w)
    perm = torch.tensor([0, 1, 2, 3, 4, 5, 6, 7, 12, 13, 14, 15, 8, 9, 10, 11])      # head 1's maps swapped, queries only
    for n in ("q", "q.b", "q.conv"):
        other["l0.mix." + n] = w["l0.mix." + n][perm]
    swapped = O.attention(other, "l0.mix.", lay["mixer"], h, EPS)
    assert float((swapped - want)[5:, 5:10].abs().max()) > 0.1 and float((swapped - want)[:, :5].abs().max()) < 1e-12
    check(run_mixer(lay, other, h, [7, 11]), swapped)


@pytest.mark.parametrize("cuts", [[40], [11, 1, 2, 26], [1] * 40])
def test_reading_layer_uses_the_owners_keys_and_values(cuts):
    """The reader is fed other rows than the owner: its queries, lambda,
    temperature, taps and scale are its own, keys and values the owner's."""
    layers = [layer("attention", att(), None),
              layer("attention", att(conv=5, diff=0.8, scale=1.1, coef=1.0, every=3, kv_from=0), None)]
    w = O.random_weights(model_cfg(layers), 16)
    assert not any(n.startswith("l1.mix.k") or n.startswith("l1.mix.v") for n in w)
    mods = [mixer_of(layers, 0, w), mixer_of(layers, 1, w)]
    h = rows(40, 24, 17)
    own = []
    want0 = O.attention(w, "l0.mix.", layers[0]["mixer"], h, EPS, None, own)
    want1 = O.attention(w, "l1.mix.", layers[1]["mixer"], h, EPS, own[0])
    got = run_mixers(mods, h, cuts)
    check(got[0], want0)
    check(got[1], want1)


def test_diff_far_key_stands_out_at_every_page_border():
    """150 positions on 16-token pages. Under map 1 the last token's queries
    are tied to the key of one particular input: whichever far token carries
    it scores far above the rest, wherever it sits in a page."""
    lay = layer("attention", att(heads=2, kv_heads=1, dim=8, vdim=6, conv=1, scale=3.0, coef=0.0), None)
    w = O.random_weights(model_cfg([lay]), 18)
    for n in ("q", "k", "v"):
        w[f"l0.mix.{n}.conv"] = torch.ones_like(w[f"l0.mix.{n}.conv"])
        w[f"l0.mix.{n}.b"] = w[f"l0.mix.{n}.b"] * 0.0
    asker, answer = rows(2, 24, 19)
    answer = answer * 2.5                                        # a long key: it beats chance matches among 150
    key = w["l0.mix.k"][:8] @ answer
    for hd in range(2):
        r = slice(hd * 16, hd * 16 + 8)
        w["l0.mix.q"][r] = 0.1 * w["l0.mix.q"][r] + torch.outer(key, asker / (asker @ asker))
    m = lay["mixer"]
    for at in (0, 15, 16, 31, 32, 63, 64, 111, 112, 148):
        h = rows(150, 24, 20)
        h[149] = asker
        gone = h.clone()
        h[at] = answer
        want = O.attention(w, "l0.mix.", m, h, EPS)
        assert float((O.attention(w, "l0.mix.", m, gone, EPS)[149] - want[149]).abs().max()) > 0.1
        for cuts in ([150], [100] + [1] * 50) if at in (0, 16, 63) else ([149, 1],):
            check(run_mixer(lay, w, h, cuts, page=16), want, atol=5e-4)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("heads,rot_dim,q_rank", [(3, 6, 11), (1, 2, 30), (4, 8, 5)])
def test_latent_attention_with_query_latent(cuts, heads, rot_dim, q_rank):
    lay = layer("latent_attention", lat(heads=heads, rot_dim=rot_dim, q_rank=q_rank, scale=2.0), None)
    w = O.random_weights(model_cfg([lay]), 21)
    mod = mixer_of([lay], 0, w)
    assert set(mod.inp.parts) == {"dq", "dkv"} and mod.uq.shape == (heads * (9 + rot_dim), q_rank)
    h = rows(sum(cuts), 24, 22)
    check(run_mixers([mod], h, cuts)[0], O.latent_attention(w, "l0.mix.", lay["mixer"], h, EPS))


def test_query_latent_norm_eps_and_weight():
    lay = layer("latent_attention", lat(scale=2.0), None)
    w = O.random_weights(model_cfg([lay]), 23)
    w["l0.mix.dq"] = w["l0.mix.dq"] * 3e-3
    h = rows(15, 24, 24)
    want = O.latent_attention(w, "l0.mix.", lay["mixer"], h, EPS)
    assert float((O.latent_attention(w, "l0.mix.", lay["mixer"], h, 1e-9) - want).abs().max()) > 1e-2
    plain = dict(w, **{"l0.mix.dq.norm": torch.ones(11, dtype=torch.float64)})
    assert float((O.latent_attention(plain, "l0.mix.", lay["mixer"], h, EPS) - want).abs().max()) > 1e-2
    check(run_mixer(lay, w, h, [6, 9]), want)


@pytest.mark.parametrize("sink", [-30.0, 0.0, 25.0])
def test_sink_from_negligible_to_dominating(sink):
    lay = layer("latent_attention", lat(scale=0.5), None)
    w = O.random_weights(model_cfg([lay]), 25)
    w["l0.mix.sink"] = torch.tensor([sink, 0.5, sink / 2], dtype=torch.float64)
    h = rows(40, 24, 26)
    want = O.latent_attention(w, "l0.mix.", lay["mixer"], h, EPS)
    none = dict(w, **{"l0.mix.sink": torch.full((3,), -1e9, dtype=torch.float64)})
    assert float((O.latent_attention(none, "l0.mix.", lay["mixer"], h, EPS)[0] - want[0]).abs().max()) > 1e-2
    for cuts in ([40], [1] * 40, [15, 2, 23]):
        check(run_mixer(lay, w, h, cuts), want)


@pytest.mark.parametrize("T", [1, 7, 90])
def test_squared_relu_feed_forward(T):
    lay = layer("attention", att(), "dense")
    w = O.random_weights(model_cfg([lay]), 27)
    spec = specs_of([lay])[0].mlp
    assert spec.act == "relu2" and not spec.gated
    mod = ActFF(spec, 24, torch.float32)
    load_module(mod, w, "l0.mlp.")
    h = rows(T, 24, 28) * 2.0
    check(mod(h.float()), O.dense_ff(w, "l0.mlp.", h))


@pytest.mark.parametrize("T", [1, 7, 90])
@pytest.mark.parametrize("mlp", ["moe", "moe_top1", "moe_all"])
def test_routed_experts(mlp, T):
    """Both forms: all experts on few rows, sorted rows on many; with and
    without a shared expert, scales above, at and below one."""
    lay = layer("attention", att(), mlp)
    w = O.random_weights(model_cfg([lay]), 29)
    spec = specs_of([lay])[0].mlp
    assert spec.score == "softmax" and not spec.renormalize and spec.correction
    assert (spec.shared is not None) == ("shared" in lay["mlp"]) and spec.scale == lay["mlp"]["router"]["scale"]
    mod = RoutedExperts(spec, 24, torch.float32)
    load_module(mod, w, "l0.mlp.")
    h = rows(T, 24, 30) * 1.5
    check(mod(h.float()), O.moe_ff(w, "l0.mlp.", lay["mlp"], h))


def test_router_correction_moves_the_choice_but_not_the_weights():
    z = torch.tensor([[1.0, 2.0, 0.5, -1.0], [0.0, 0.0, 3.0, 0.1]])
    corr = torch.tensor([0.0, -0.9, 0.0, 0.8])
    idx, w = ops.moe_route(z, corr, 2, 1, 1, "softmax", False, 1.9)
    for t in range(2):
        oi, ow = O.route(z[t].double(), corr.double(), 2, 1.9)
        assert idx[t].tolist() == oi
        check(w[t], ow, atol=1e-6)
    assert idx[0].tolist() == [3, 0] and float(w[0].sum()) < 1.0       # neither the largest logit nor renormalised


def test_diff_tiles_cover_every_row_once():
    for rows_ in (32, 64, 128):
        segs = [(0, 1), (3, 200), (9, 2), (0, 0), (70, 1), (0, 33)]
        tiles, single = ops.diff_tiles(segs, rows_, "cpu")
        seg_of = [b for b, (_, n) in enumerate(segs) for _ in range(n)]
        seen = single.tolist()
        for r, n in tiles.tolist():
            assert 1 <= n <= rows_ and len({seg_of[i] for i in range(r, r + n)}) == 1
            seen += list(range(r, r + n))
        assert sorted(seen) == list(range(len(seg_of))) and single.tolist() == [0, 203]
    assert [ops.diff_tile_rows(h, g) for h, g in [(4, 4), (4, 2), (6, 2), (8, 1)]] == [128, 64, 32, 32]


# --- whole models through the engine ------------------------------------------------

def run_cuts(eng, ids, cuts):
    seq = eng.open_sequence()
    outs, at = [], 0
    for n in cuts:
        outs.append(eng.step_segments([(seq, ids[at:at + n], list(range(n)))]))
        at += n
    eng.kv.free_sequence(seq)
    return torch.cat(outs)


def test_whole_prompt_and_first_tokens(model_a):
    cfg, w, eng = model_a
    ids = toks(45, cfg["vocab"], 20)
    want = O.forward(cfg, w, ids)
    check(run_cuts(eng, ids, [45]), want)
    check(run_cuts(eng, ids[:1], [1]), want[:1])
    check(run_cuts(eng, ids[:3], [1, 1, 1]), want[:3])


def test_cache_entries_and_stream_after_every_layer(model_a):
    cfg, w, eng = model_a
    L = eng.kv.layers
    assert L[2].shared_kv and L[4].shared_kv and L[2].k is L[1].k and L[4].v is L[1].v
    assert L[1].k.shape[1:] == (2, 4, 12) and L[1].v.shape[1:] == (2, 4, 10) and L[0].k.shape[-1] == 18
    assert L[1].conv.shape[1] == 2 and L[2].conv.shape[1:] == (1, 48) and L[4].conv.shape[1] == 4
    assert eng.model.lm_head.weight is not eng.model.embed_tokens.weight
    ids = toks(14, cfg["vocab"], 21)
    want = []
    O.forward(cfg, w, ids, want)
    eng.model.trace_layers = []
    try:
        run_cuts(eng, ids, [5, 9])
        got = eng.model.trace_layers
    finally:
        eng.model.trace_layers = None
    assert len(got) == 10 and len(want) == 5
    for i, b in enumerate(want):
        check(torch.cat([got[i], got[5 + i]]), b, atol=5e-4)


def test_prefill_then_decode_long(model_a):
    cfg, w, eng = model_a
    ids = toks(4 + 130, cfg["vocab"], 22)
    check(run_cuts(eng, ids, [4] + [1] * 130), O.forward(cfg, w, ids), atol=5e-4)


@pytest.mark.parametrize("cuts", [[2] * 20, [7, 2, 13, 1, 1, 16], [3, 9, 2, 2, 24], [39, 1]])
def test_portions(model_a, cuts):
    cfg, w, eng = model_a
    ids = toks(sum(cuts), cfg["vocab"], 23)
    check(run_cuts(eng, ids, cuts), O.forward(cfg, w, ids))


def test_mixed_batches_reuse_pages_and_slots(model_b):
    """Five unequal requests through three slots and a pool smaller than their
    sum (8-token pages): portions beside single tokens, requests that pause,
    slots and pages that change hands."""
    cfg, w, eng = model_b
    reqs = {n: toks(L, cfg["vocab"], 30 + i) for i, (n, L) in enumerate(
        [("a", 70), ("b", 9), ("c", 33), ("d", 2), ("e", 41)])}
    want = {n: O.forward(cfg, w, ids) for n, ids in reqs.items()}
    plan = [[("a", 30), ("b", 2)], [("a", 1), ("b", 6), ("c", 20)], [("c", 1), ("b", 1)],        # b ends
            [("a", 2), ("d", 2), ("c", 12)],                                                   # d, c end
            [("a", 37), ("e", 1)], [("e", 40)]]
    at = {n: 0 for n in reqs}
    live = {}
    for step in plan:
        entries = []
        for n, c in step:
            if n not in live:
                live[n] = eng.open_sequence()
            entries.append((live[n], reqs[n][at[n]:at[n] + c], list(range(c))))
        got = eng.step_segments(entries)
        r = 0
        for n, c in step:
            check(got[r:r + c], want[n][at[n]:at[n] + c])
            r += c
            at[n] += c
            if at[n] == len(reqs[n]):
                eng.kv.free_sequence(live.pop(n))
    assert not live and eng.kv.slots.num_free == 3 and eng.kv.allocator.num_free == eng.kv.num_blocks


def test_batch_rows_equal_rows_alone(model_a):
    cfg, w, eng = model_a
    a, b, c = toks(19, cfg["vocab"], 44), toks(3, cfg["vocab"], 45), toks(40, cfg["vocab"], 46)
    alone = [run_cuts(eng, x, [len(x)]) for x in (a, b, c)]
    seqs = [eng.open_sequence() for _ in range(3)]
    got = eng.step_segments([(s, x, list(range(len(x)))) for s, x in zip(seqs, (a, b, c))])
    for s in seqs:
        eng.kv.free_sequence(s)
    torch.testing.assert_close(got, torch.cat(alone), rtol=1e-5, atol=1e-5)


def test_used_pages_and_slots_are_not_inherited(model_a):
    cfg, w, eng = model_a
    a, b = toks(37, cfg["vocab"], 40), toks(21, cfg["vocab"], 41)
    s = eng.open_sequence()
    eng.step_segments([(s, a, [])])
    blocks, slot = list(s.blocks), s.state_slot
    eng.kv.free_sequence(s)
    s2 = eng.open_sequence()
    out = eng.step_segments([(s2, b[:1], [0]), ])
    assert set(s2.blocks) & set(blocks) and s2.state_slot == slot
    out = torch.cat([out, eng.step_segments([(s2, b[1:], list(range(20)))])])
    check(out, O.forward(cfg, w, b))
    eng.kv.free_sequence(s2)


def test_second_configuration_in_portions(model_b):
    cfg, w, eng = model_b
    ids = toks(50, cfg["vocab"], 42)
    want = O.forward(cfg, w, ids)
    check(run_cuts(eng, ids, [50]), want)
    check(run_cuts(eng, ids, [3, 1, 1, 2, 23, 2, 18]), want)
    check(run_cuts(eng, ids, [10] + [1] * 40), want)


def oracle_greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(O.forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


def test_greedy_generation_and_fork(model_a):
    """n = 2 forks the prompt's sequence: the tail page and the carried
    convolution rows are copied, and both streams go on like the oracle."""
    cfg, w, eng = model_a
    p1, p2 = toks(21, cfg["vocab"], 50), toks(5, cfg["vocab"], 51)
    sp = lambda n: SamplingParams(temperature=0.0, max_tokens=n)
    outs = eng.generate([GenRequest(prompt_ids=p1, n=2, sampling=sp(7)), GenRequest(prompt_ids=p2, n=1, sampling=sp(9))])
    want1, want2 = oracle_greedy(cfg, w, p1, 7), oracle_greedy(cfg, w, p2, 9)
    assert [s.token_ids for s in outs[0].streams] == [want1, want1]
    assert outs[1].streams[0].token_ids == want2
    assert eng.kv.slots.num_free == eng.kv.slots.num_slots and eng.kv.allocator.num_free == eng.kv.num_blocks


def test_scheduler_chunked_prefill_and_merge(tmp_path):
    w = write_model(str(tmp_path), CFG_A, seed=1)
    eng = make_engine(tmp_path, blocks=128, slots=8, prefill_chunk_tokens=8, max_batch_size=4)
    sched = BatchScheduler(eng)
    try:
        p1, p2 = toks(29, CFG_A["vocab"], 52), toks(6, CFG_A["vocab"], 53)
        sp = lambda n: SamplingParams(temperature=0.0, max_tokens=n)
        f1 = sched.submit(GenRequest(prompt_ids=p1, n=1, sampling=sp(6)))
        f2 = sched.submit(GenRequest(prompt_ids=p2, n=2, sampling=sp(8)))
        o1, o2 = f1.result(timeout=120), f2.result(timeout=120)
    finally:
        sched.shutdown()
    assert o1.streams[0].token_ids == oracle_greedy(CFG_A, w, p1, 6)
    want2 = oracle_greedy(CFG_A, w, p2, 8)
    assert [s.token_ids for s in o2.streams] == [want2, want2]
    assert eng.kv.slots.num_free == eng.kv.slots.num_slots


def test_config_reader_takes_everything_from_the_file(tmp_path):
    write_model(str(tmp_path), CFG_B, seed=2)
    arch = EngineConfig(model=str(tmp_path)).resolve_arch()
    assert arch.arch == "dimuvik" and arch.vocab_size == 47 and arch.hidden_size == 20 and not arch.tie_word_embeddings
    assert arch.rms_norm_eps == 1e-6 and arch.embed_scale == 1.0
    assert [l.type for l in arch.layers] == ["attention", "attention", "latent_attention", "attention"]
    a0, a1, a3 = (arch.layers[i].attention for i in (0, 1, 3))
    assert (a0.heads, a0.kv_heads, a0.dim, a0.vdim, a0.conv, a0.diff, a0.scale) == (3, 3, 5, 7, 6, 0.4, 0.5)
    assert (a0.temp_coef, a0.temp_every, a0.kv_from) == (0.0, 16, None)
    assert (a1.conv, a1.diff, a1.temp_every, a1.kv_from) == (1, 0.8, 1, 0)
    assert (a3.heads, a3.kv_heads, a3.diff, a3.temp_coef, a3.temp_every) == (4, 1, 0.0, 0.5, 7)
    la = arch.layers[2].latent
    assert (la.heads, la.dim, la.rot_dim, la.vdim, la.kv_rank, la.q_rank, la.scale) == (1, 6, 4, 5, 7, 20, 0.9)
    assert la.sink and not la.elem_gate and not la.head_gate and la.mask_size == 0
    assert (la.rot.base, la.rot.dims, la.rot.layout) == (100.0, 4, "pairs")
    m0, m2, m3 = arch.layers[0].mlp, arch.layers[2].mlp, arch.layers[3].mlp
    assert (m0.experts, m0.top, m0.ff, m0.scale, m0.shared) == (5, 1, 16, 1.0, None) and arch.layers[1].mlp is None
    assert (m2.experts, m2.top, m2.scale, m2.shared.ff, m2.shared.gated) == (3, 3, 0.6, 8, False) and m3.ff == 28
    for i, where, field, value in [(1, "mixer", "kv_from", 2), (1, "mixer", "kv_from", 1), (3, "mixer", "kv_from", 1),
                                   (3, "mixer", "kv_from", 0), (0, None, "type", "mamba2")]:
        bad = json.loads(json.dumps(CFG_B))
        (bad["layers"][i][where] if where else bad["layers"][i])[field] = value
        with pytest.raises(ValueError):
            DimuvikArchConfig.from_checkpoint_config(bad)


def test_checkpoint_with_a_tensor_missing_or_misshapen(tmp_path):
    w = O.random_weights(CFG_B, 2)
    write_model(str(tmp_path / "a"), CFG_B, w={k: v for k, v in w.items() if k != "l2.norm1b.alpha"})
    with pytest.raises(RuntimeError, match="alpha"):
        make_engine(tmp_path / "a")
    write_model(str(tmp_path / "b"), CFG_B, w=dict(w, **{"l0.mix.q.conv": w["l0.mix.q.conv"][:, 1:]}))
    with pytest.raises(RuntimeError, match="q.conv"):
        make_engine(tmp_path / "b")


def test_presets_build_and_generate():
    eng = LLMEngine(EngineConfig(model="tiny-dimuvik", dtype="float32", device="cpu", max_kv_blocks=64,
                                 max_state_slots=4, use_hip_graphs=False))
    assert [l.attention.kv_from if l.attention else -1 for l in eng.arch.layers] == [-1, None, 1, -1]
    out = eng.generate([GenRequest(prompt_ids=toks(9, 512, 60), n=2, sampling=SamplingParams(temperature=0.0, max_tokens=5))])
    assert len(out[0].streams) == 2 and out[0].streams[0].token_ids == out[0].streams[1].token_ids


def test_trace_replay_cli(tmp_path):
    import subprocess
    import sys

    import numpy as np

    cfg = CFG_B
    mdir, out = tmp_path / "m", tmp_path / "out"
    w = write_model(str(mdir), cfg, seed=4)
    a, b = toks(20, cfg["vocab"], 61), toks(5, cfg["vocab"], 62)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:18], "want": [0, 17]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[18:19], "want": []},
                                     {"id": "b", "tokens": b, "want": [4]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[19:], "want": [0]}], "end": ["a"]}]
    exe = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "trace_run")
    r = subprocess.run([sys.executable, exe, "--model", str(mdir), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "64", "--device", "cpu"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    la, lb = O.forward(cfg, w, a), O.forward(cfg, w, b)
    rd = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"]).copy())
    check(rd(0), la[[0, 17]])
    check(rd(1), lb[[4]])
    check(rd(2), la[[19]])
