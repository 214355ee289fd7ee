"""Bavesun family on the CPU path (fp32) against the plain float64 oracle in
tests/bavesun_oracle.py: every mechanism alone, then whole models through the
engine's segment step, page and slot reuse, and greedy generation through
generate() and the scheduler. Configurations are small and lopsided: head
counts that are not powers of two, value sizes that differ from key sizes,
partly and fully rotated heads, layers without a feed-forward, loops that
begin and end inside the model and models without one, top 1 and top = all."""

import json
import math
import os

import pytest
import torch

import bavesun_oracle as O
from kllms_amd import ops
from kllms_amd.engine.config import BavesunArchConfig, EngineConfig
from kllms_amd.engine.engine import GenRequest, LLMEngine
from kllms_amd.engine.sampling import SamplingParams
from kllms_amd.engine.scheduler import BatchScheduler
from kllms_amd.models.mixers import ActFF, CentredNormWeight, LatentAttention, Retention, RoutedExperts, TokenSide
from test_pironex import check, dirty_cache, load_module, rows, run_mixers, seg_batch, toks

EPS = 1e-5


def ret(heads=3, dim=10, vdim=7, decay=(0.5, 0.9, 0.99), rot=6, base=50.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay), "rot": {"base": base, "dims": rot}}


def lat(heads=3, dim=9, rot_dim=6, vdim=7, kv_rank=12, scale=0.3, base=100.0):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
            "rot": {"base": base, "dims": rot_dim}}


MLPS = {
    None: None,
    "dense": {"kind": "dense", "ff": 28},
    "moe": {"kind": "moe", "expert": {"ff": 11}, "router": {"experts": 6, "top": 3}},
    "moe_top1": {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 5, "top": 1}},
    "moe_all": {"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 3, "top": 3}},
}


def layer(kind, mixer, mlp="dense"):
    return {"type": kind, "mixer": mixer, "mlp": MLPS[mlp]}


def model_cfg(layers, vocab=61, width=24, eps=EPS, scale=1.7, dim=5, loop=None):
    return {"architecture": "Bavesun", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "token_side": {"dim": dim}, "layers": layers, "loop": loop}


# the loop begins and ends inside the model and holds both mixers
CFG_A = model_cfg([layer("latent_attention", lat(), "moe"),
                   layer("retention", ret(), "moe_top1"),
                   layer("latent_attention", lat(heads=5, dim=4, rot_dim=2, vdim=3, kv_rank=10, scale=0.7), "dense"),
                   layer("retention", ret(heads=2, dim=6, vdim=9, decay=(0.97, 0.6), rot=6, base=1000.0), None)],
                  loop={"start": 1, "stop": 3, "times": 3})
# no loop, one head of each kind, unrotated retention, a scale of one, a last layer without a feed-forward
CFG_B = model_cfg([layer("retention", ret(heads=1, dim=8, vdim=8, decay=(0.999,), rot=0), "dense"),
                   layer("retention", ret(heads=4, dim=4, vdim=5, decay=(1.0, 0.9, 0.8, 0.0), rot=2), "moe_all"),
                   layer("latent_attention", lat(heads=1, dim=6, rot_dim=4, vdim=5, kv_rank=7, scale=0.9), None)],
                  vocab=47, width=20, eps=1e-6, scale=1.0, dim=8)
del CFG_B["loop"]


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
    d = tmp_path_factory.mktemp("bav_a")
    w = write_model(str(d), CFG_A, seed=1)
    return CFG_A, w, make_engine(d, blocks=96, kv_block_size=4)


@pytest.fixture(scope="module")
def model_b(tmp_path_factory):
    d = tmp_path_factory.mktemp("bav_b")
    w = write_model(str(d), CFG_B, seed=2)
    return CFG_B, w, make_engine(d, blocks=24, slots=3, kv_block_size=8)


def arch_of(lay, width=24):
    return BavesunArchConfig.from_checkpoint_config(model_cfg([lay], width=width)).layers[0]


def mixer_of(lay, w, width=24):
    sp = arch_of(lay, width)
    mod = (Retention(sp.retention, width, EPS, torch.float32) if lay["type"] == "retention"
           else LatentAttention(sp.latent, width, EPS, torch.float32))
    load_module(mod, w, "l0.mix.")
    return mod


# --- mechanisms alone -----------------------------------------------------------------

CUTS = [[60], [25] + [1] * 35, [2, 5, 16, 1, 2, 17, 3, 14], [2] * 30, [1] * 60]


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("rot,vdim", [(6, 7), (10, 10), (0, 3), (2, 12)])
def test_retention(cuts, rot, vdim):
    lay = layer("retention", ret(rot=rot, vdim=vdim), None)
    w = O.random_weights(model_cfg([lay]), 3)
    h = rows(sum(cuts), 24, 4)
    check(run_mixers([mixer_of(lay, w)], h, cuts)[0], O.retention(w, "l0.mix.", lay["mixer"], h, EPS))


def test_retention_state_carries_a_far_token():
    """With a slow decay the first token, made large, still moves the output
    120 steps on; with a fast one it does not."""
    h = rows(121, 24, 14)
    h[0] *= 30.0
    other = h.clone()
    other[0] = rows(1, 24, 15)[0]
    for decay, seen in [((0.999, 0.995, 0.9999), True), ((0.5, 0.6, 0.4), False)]:
        lay = layer("retention", ret(decay=decay), None)
        w = O.random_weights(model_cfg([lay]), 13)
        want = O.retention(w, "l0.mix.", lay["mixer"], h, EPS)
        moved = float((O.retention(w, "l0.mix.", lay["mixer"], other, EPS)[120] - want[120]).abs().max())
        assert (moved > 1e-2) == seen
        for cuts in ([121], [1] * 121, [60, 2, 59]):
            check(run_mixers([mixer_of(lay, w)], h, cuts)[0], want, atol=5e-4)


def test_retention_norm_is_per_head_and_eps_inside_the_root():
    """Read-outs near zero: eps decides their scale, head by head."""
    lay = layer("retention", ret(), None)
    w = O.random_weights(model_cfg([lay]), 5)
    w["l0.mix.v"] = w["l0.mix.v"] * torch.tensor([1e-3, 1.0, 1e-2], dtype=torch.float64).repeat_interleave(7)[:, None]
    h = rows(12, 24, 6)
    want = O.retention(w, "l0.mix.", lay["mixer"], h, EPS)
    assert float((want - O.retention(w, "l0.mix.", lay["mixer"], h, 1e-7)).abs().max()) > 1e-2
    check(run_mixers([mixer_of(lay, w)], h, [12])[0], want)


def test_rotations_pair_as_each_mixer_says():
    """Retention pairs entry i with i + dims/2 of the rotated part, latent
    attention 2i with 2i+1."""
    v = torch.arange(1.0, 9.0, dtype=torch.float64)
    half, pairs = O.rotate(v, 3, 10.0, 4, "half"), O.rotate(v, 3, 10.0, 4, "pairs")
    a0, a1 = 3.0, 3.0 * 10.0 ** -0.5
    assert abs(float(half[0]) - (1 * math.cos(a0) - 3 * math.sin(a0))) < 1e-12
    assert abs(float(half[3]) - (4 * math.cos(a1) + 2 * math.sin(a1))) < 1e-12
    assert abs(float(pairs[1]) - (2 * math.cos(a0) + 1 * math.sin(a0))) < 1e-12
    assert torch.equal(half[4:], v[4:]) and torch.equal(pairs[4:], v[4:])
    # one step from a zero state: o = (k . q) v with both rotated alike, so feed different positions
    inv = torch.tensor([1.0, 10.0 ** -0.5])
    q, k = rows(2, 8, 1).float().view(2, 1, 8), rows(2, 8, 2).float().view(2, 1, 8)
    state = torch.zeros(1, 1, 8, 1)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32)
    o = ops.retention(q, k, torch.tensor([[[1.0]], [[0.0]]]), torch.tensor([1.0]), torch.tensor([4, 9]), inv, state,
                      i32([0]), i32([0, 2]), i32([0]))
    want = O.rotate(q[1, 0].double(), 9, 10.0, 4, "half") @ O.rotate(k[0, 0].double(), 4, 10.0, 4, "half") / 8 ** 0.5
    check(o[1].view(1), want.view(1), atol=1e-5)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("heads,rot_dim", [(3, 6), (1, 2), (4, 8)])
def test_latent_attention_with_sink_and_element_gate(cuts, heads, rot_dim):
    lay = layer("latent_attention", lat(heads=heads, rot_dim=rot_dim, scale=2.0), None)
    w = O.random_weights(model_cfg([lay]), 7)
    mod = mixer_of(lay, w)
    assert mod.inp.parts["g"][1] == heads * 7 and mod.sink.shape == (heads,)
    h = rows(sum(cuts), 24, 8)
    check(run_mixers([mod], h, cuts)[0], O.latent_attention(w, "l0.mix.", lay["mixer"], h, EPS))


@pytest.mark.parametrize("sink", [-30.0, 0.0, 25.0])
def test_sink_from_negligible_to_dominating(sink):
    """A very low sink leaves the plain softmax, a high one takes nearly all
    the weight; it is not scaled and counts once whatever the length."""
    lay = layer("latent_attention", lat(scale=0.5), None)
    w = O.random_weights(model_cfg([lay]), 9)
    w["l0.mix.sink"] = torch.tensor([sink, 0.5, sink / 2], dtype=torch.float64)
    h = rows(40, 24, 10)
    want = O.latent_attention(w, "l0.mix.", lay["mixer"], h, EPS)
    none = dict(w)
    none["l0.mix.sink"] = torch.full((3,), -1e9, dtype=torch.float64)
    assert float((O.latent_attention(none, "l0.mix.", lay["mixer"], h, EPS)[0] - want[0]).abs().max()) > 1e-2
    for cuts in ([40], [1] * 40, [15, 2, 23]):
        check(run_mixers([mixer_of(lay, w)], h, cuts)[0], want)


def test_far_key_stands_out_at_every_page_border():
    """150 positions on 16-token pages. The last token's queries are tied to
    the keys of one particular input: whichever far token carries that input
    scores far above the others, and the output follows it wherever it sits
    in a page."""
    lay = layer("latent_attention", lat(heads=2, dim=12, rot_dim=2, kv_rank=12, scale=4.0), None)
    w = O.random_weights(model_cfg([lay]), 11)
    asker, answer = rows(2, 24, 12)
    c = O.rms(w["l0.mix.dkv"][:12] @ answer, EPS) * w["l0.mix.dkv.norm"]
    for n in range(2):
        r = slice(n * 14, n * 14 + 12)
        w["l0.mix.q"][r] = 0.1 * w["l0.mix.q"][r] + torch.outer(w["l0.mix.uk"][n * 12:(n + 1) * 12] @ c, asker / (asker @ asker))
    mod = mixer_of(lay, w)
    m = lay["mixer"]
    for at in (0, 15, 16, 31, 32, 47, 111, 112, 148):
        h = rows(150, 24, 13)
        h[149] = asker
        gone = h.clone()
        h[at] = answer
        want = O.latent_attention(w, "l0.mix.", m, h, EPS)
        assert float((O.latent_attention(w, "l0.mix.", m, gone, EPS)[149] - want[149]).abs().max()) > 0.1
        for cuts in ([150], [100] + [1] * 50) if at in (0, 16, 47) else ([149, 1],):
            check(run_mixers([mod], h, cuts, page=16)[0], want, atol=5e-4)


@pytest.mark.parametrize("T", [1, 7, 90])
def test_gated_gelu_feed_forward(T):
    lay = layer("retention", ret(), "dense")
    w = O.random_weights(model_cfg([lay]), 16)
    spec = arch_of(lay).mlp
    assert spec.gated and spec.act == "gelu_tanh"
    mod = ActFF(spec, 24, torch.float32)
    load_module(mod, w, "l0.mlp.")
    h = rows(T, 24, 17) * 2.0
    check(mod(h.float()), O.dense_ff(w, "l0.mlp.", h))


@pytest.mark.parametrize("T", [1, 7, 90])
@pytest.mark.parametrize("mlp", ["moe", "moe_top1", "moe_all"])
def test_squared_relu_experts(mlp, T):
    """Both forms: all experts on few rows, sorted rows on many."""
    lay = layer("retention", ret(), mlp)
    w = O.random_weights(model_cfg([lay]), 18)
    spec = arch_of(lay).mlp
    assert spec.act == "relu2" and spec.score == "top_softmax" and not spec.correction and spec.shared is None
    mod = RoutedExperts(spec, 24, torch.float32)
    load_module(mod, w, "l0.mlp.")
    h = rows(T, 24, 19) * 1.5
    check(mod(h.float()), O.moe_ff(w, "l0.mlp.", lay["mlp"], h))


def test_router_chooses_by_logits_far_apart():
    """Logits whose softmax over all outputs underflows are still told apart;
    the weights are the softmax over the chosen ones."""
    z = torch.tensor([[300.0, 20.0, 30.0, -5.0, 25.0], [1.0, 1.5, 0.5, 1.25, -3.0]])
    idx, w = ops.moe_route(z, None, 3, 1, 1, "top_softmax", True)
    for t in range(2):
        oi, ow = O.route(z[t].double(), 3)
        assert idx[t].tolist() == oi
        check(w[t], ow, atol=1e-6)
    assert idx[0].tolist() == [0, 2, 4]


def test_centred_norm_weight():
    norm = CentredNormWeight(24)
    wz = 0.3 * rows(1, 24, 20)[0]
    norm.weight.copy_(wz.float())
    norm.fold()
    x = rows(5, 24, 21) * 1e-2
    check(ops.rmsnorm_cast(x.float(), norm.scale, EPS, torch.float32), O.norm_about_zero(x, wz, EPS))
    a, b = rows(5, 24, 22), rows(5, 24, 23)
    xs = x.float()
    h, _ = ops.group_norm_pair(xs, a.float(), b.float(), norm.scale, None, 1, EPS, torch.float32)
    check(xs, x + a + b)
    check(h, O.norm_about_zero(x + a + b, wz, EPS))


@pytest.mark.parametrize("index", [0, 1, 2])
def test_token_side_input_reads_its_own_columns(index):
    cfg = model_cfg([layer("retention", ret(), None)] * 3)
    w = O.random_weights(cfg, 24)
    mod = TokenSide(24, 5, index, torch.float32)
    load_module(mod, w, f"l{index}.side.")
    x, ids = rows(6, 24, 25), [3, 60, 0, 3, 17, 5]
    y = mod(x.float(), torch.tensor(ids), w["side.embed"].float())
    xs = x.float()
    ops.sandwich_residual(xs, y, mod.norm, EPS, w_next=torch.ones(24), out_dtype=torch.float32)
    check(xs, x + O.token_side(w, cfg, index, x, ids, EPS))
    assert float((O.token_side(w, cfg, (index + 1) % 3, x, ids, EPS) - O.token_side(w, cfg, index, x, ids, EPS)).abs().max()) > 0.1


def test_retention_chunk_plan():
    """Chunks cover the step's rows in order, never across segments."""
    ch, c0 = ops.retention_chunks([(0, 64), (9, 1), (0, 0), (5, 130), (0, 65)], "cpu")
    assert c0.tolist() == [0, 1, 2, 2, 5, 7]
    assert ch.tolist() == [[0, 64, 0, 0], [64, 1, 1, 0], [65, 64, 3, 0], [129, 64, 3, 0], [193, 2, 3, 0],
                           [195, 64, 4, 0], [259, 1, 4, 0]]


def test_layer_order_with_and_without_a_loop():
    arch = BavesunArchConfig.from_checkpoint_config(CFG_A)
    assert arch.layer_runs() == O.layer_order(CFG_A) == [0, 1, 2, 1, 2, 1, 2, 3]
    assert BavesunArchConfig.from_checkpoint_config(CFG_B).layer_runs() == [0, 1, 2]
    for lp, want in [({"start": 0, "stop": 4, "times": 2}, [0, 1, 2, 3] * 2), ({"start": 3, "stop": 4, "times": 1}, [0, 1, 2, 3])]:
        assert BavesunArchConfig.from_checkpoint_config(dict(CFG_A, loop=lp)).layer_runs() == want
    for bad in ({"start": 2, "stop": 2, "times": 2}, {"start": 0, "stop": 5, "times": 2}, {"start": 0, "stop": 1, "times": 0}):
        with pytest.raises(ValueError):
            BavesunArchConfig.from_checkpoint_config(dict(CFG_A, loop=bad))


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


def test_every_pass_has_its_own_entry_and_the_stream_matches_after_it(model_a):
    cfg, w, eng = model_a
    L = eng.kv.layers
    assert [st.rec is not None for st in L] == [False, True, False, True, False, True, False, True]
    assert L[0].k.shape[-1] == 18 and L[2].k.shape[-1] == 12 and L[2].k is not L[4].k and L[0].v.numel() == 0
    assert L[1].rec.shape[1:] == (3, 10, 7) and L[7].rec.shape[1:] == (2, 6, 9)
    assert eng.model.lm_head.weight is eng.model.embed_tokens.weight
    ids = toks(14, cfg["vocab"], 21)
    want = []
    O.forward(cfg, w, ids, want)
    eng.model.trace_layers = []
    try:
        run_cuts(eng, ids, [5, 9])
        got = eng.model.trace_layers
    finally:
        eng.model.trace_layers = None
    assert len(got) == 16 and len(want) == 8
    for i, b in enumerate(want):
        check(torch.cat([got[i], got[8 + i]]), b, atol=5e-4)


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
    out = eng.step_segments([(s2, b, list(range(21)))])
    assert set(s2.blocks) & set(blocks) and s2.state_slot == slot
    check(out, O.forward(cfg, w, b))
    eng.kv.free_sequence(s2)


def test_second_configuration_in_portions(model_b):
    cfg, w, eng = model_b
    ids = toks(50, cfg["vocab"], 42)
    want = O.forward(cfg, w, ids)
    check(run_cuts(eng, ids, [50]), want)
    check(run_cuts(eng, ids, [3, 1, 1, 2, 23, 2, 18]), want)
    check(run_cuts(eng, ids, [10] + [1] * 40), want)


def test_model_without_a_side_table(tmp_path):
    """No token_side entry: the layers end with their own residual add."""
    cfg = {k: v for k, v in CFG_B.items() if k != "token_side"}
    w = {k: v for k, v in O.random_weights(CFG_B, 6).items() if "side" not in k}
    write_model(str(tmp_path), cfg, w=w)
    eng = make_engine(tmp_path)
    assert eng.model.side_table is None
    ids = toks(12, cfg["vocab"], 47)
    full = dict(w, **{"side.embed": torch.zeros(cfg["vocab"], 24, dtype=torch.float64)})
    for i in range(3):
        full[f"l{i}.side.gate"], full[f"l{i}.side.proj"] = torch.zeros(8, 20).double(), torch.zeros(20, 8).double()
        full[f"l{i}.side.norm"] = torch.zeros(20).double()
    check(run_cuts(eng, ids, [5, 7]), O.forward(CFG_B, full, ids))


def oracle_greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(O.forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


def test_greedy_generation_and_fork(model_a):
    """n = 2 forks the prompt's sequence: the tail page and the slot of every
    pass are copied, and both streams go on like the oracle."""
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
    assert arch.arch == "bavesun" and arch.vocab_size == 47 and arch.hidden_size == 20 and arch.tie_word_embeddings
    assert arch.rms_norm_eps == 1e-6 and arch.embed_scale == 1.0 and arch.side_dim == 8 and arch.loop is None
    assert [l.type for l in arch.layers] == ["retention", "retention", "latent_attention"]
    r0, r1 = arch.layers[0].retention, arch.layers[1].retention
    assert (r0.heads, r0.dim, r0.vdim, r0.decay, r0.rot.dims) == (1, 8, 8, [0.999], 0)
    assert (r1.heads, r1.dim, r1.vdim, r1.decay) == (4, 4, 5, [1.0, 0.9, 0.8, 0.0])
    assert (r1.rot.base, r1.rot.dims, r1.rot.layout) == (50.0, 2, "half")
    la = arch.layers[2].latent
    assert (la.heads, la.dim, la.rot_dim, la.vdim, la.kv_rank, la.scale) == (1, 6, 4, 5, 7, 0.9)
    assert la.sink and la.elem_gate and not la.head_gate and la.mask_size == 0 and la.rot.layout == "pairs"
    assert (la.rot.base, la.rot.dims) == (100.0, 4)
    m0, m1 = arch.layers[0].mlp, arch.layers[1].mlp
    assert m0.ff == 28 and m0.gated and (m1.experts, m1.top, m1.ff) == (3, 3, 8) and arch.layers[2].mlp is None
    for field, value in [("decay", [0.9]), ("type", "attention")]:
        bad = json.loads(json.dumps(CFG_B))
        (bad["layers"][1]["mixer"] if field == "decay" else bad["layers"][1])[field] = value
        with pytest.raises(ValueError):
            BavesunArchConfig.from_checkpoint_config(bad)


def test_checkpoint_with_a_tensor_missing_or_misshapen(tmp_path):
    w = O.random_weights(CFG_B, 2)
    write_model(str(tmp_path / "a"), CFG_B, w={k: v for k, v in w.items() if k != "l2.mix.sink"})
    with pytest.raises(RuntimeError, match="sink"):
        make_engine(tmp_path / "a")
    write_model(str(tmp_path / "b"), CFG_B, w=dict(w, **{"side.embed": w["side.embed"][:, :-1]}))
    with pytest.raises(RuntimeError, match="side.embed"):
        make_engine(tmp_path / "b")


def test_presets_build_and_generate():
    eng = LLMEngine(EngineConfig(model="tiny-bavesun", dtype="float32", device="cpu", max_kv_blocks=64,
                                 max_state_slots=4, use_hip_graphs=False))
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
