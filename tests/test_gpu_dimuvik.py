"""Dimuvik family on the GPU: the engine with its HIP kernels (fp32 exact mode
and bf16 serving mode) against the float64 oracle, through mixed schedules
with page and slot reuse, prompt portions beside decoded tokens, long
decoding, far keys at tile borders, and greedy generation through generate()."""

import pytest
import torch

import dimuvik_oracle as O
from kllms_amd import ops
from kllms_amd.engine.config import EngineConfig
from kllms_amd.engine.engine import GenRequest, LLMEngine
from kllms_amd.engine.sampling import SamplingParams
from test_dimuvik import CFG_A, CFG_B, att, lat, layer, model_cfg, oracle_greedy, toks, write_model
from test_zutalix import run_schedule

pytestmark = pytest.mark.gpu

# sizes the vector and matrix-tile paths take
CFG_C = model_cfg([layer("attention", att(heads=6, kv_heads=2, dim=24, vdim=40, conv=4, scale=0.3, every=32), "moe"),
                   layer("attention", att(heads=6, kv_heads=2, dim=24, vdim=40, conv=3, scale=0.25, diff=0.6, kv_from=0), "dense"),
                   layer("latent_attention", lat(heads=4, dim=24, rot_dim=16, vdim=32, kv_rank=64, q_rank=56, scale=0.2, base=1e4), "dense"),
                   layer("attention", att(heads=2, kv_heads=2, dim=56, vdim=72, conv=2, scale=0.2, diff=0.2, every=50), "moe_all")],
                  vocab=128, width=96)


def gpu_engine(path, dtype, **kw):
    return LLMEngine(EngineConfig(model=str(path), dtype=dtype, device="cuda", max_kv_blocks=96,
                                  max_state_slots=6, use_hip_graphs=False, **kw))


SCHED = [[("a", 16)], [("a", 3), ("b", 20)], [("a", 1), ("b", 1), ("c", 30)], [("a", 10), ("b", 2), ("c", 1)],
         [("a", 20), ("c", 6)], [("d", 2), ("e", 8)], [("d", 1), ("e", 1), ("f", 7)], [("d", 30), ("f", 1)],
         [("d", 8), ("f", 22)]]
LENS = {"a": 50, "b": 23, "c": 37, "d": 41, "e": 9, "f": 30}


@pytest.mark.parametrize("cfg,seed", [(CFG_A, 1), (CFG_B, 2), (CFG_C, 3)])
def test_fp32_mixed_schedule_matches_oracle(tmp_path, cfg, seed):
    w = write_model(str(tmp_path), cfg, seed=seed)
    eng = gpu_engine(tmp_path, "float32")
    prompts = {r: toks(n, cfg["vocab"], 10 + i) for i, (r, n) in enumerate(LENS.items())}
    got = run_schedule(eng, SCHED, prompts)
    assert ops.seq_hip_loaded()
    for r in LENS:
        torch.testing.assert_close(got[r].double().cpu(), O.forward(cfg, w, prompts[r]), rtol=1e-4, atol=3e-4)
    assert eng.kv.allocator.num_free == eng.kv.num_blocks


@pytest.mark.parametrize("cfg,seed", [(CFG_A, 1), (CFG_C, 3)])
def test_fp32_long_prompt_long_decode_and_both_expert_forms(tmp_path, monkeypatch, cfg, seed):
    """A prompt of several key tiles whole, in portions that end inside, at
    and after a tile's edge, and token by token; experts' rows sorted by
    expert instead of every expert on every row."""
    w = write_model(str(tmp_path), cfg, seed=seed)
    eng = gpu_engine(tmp_path, "float32")
    p = toks(214, cfg["vocab"], 7)
    want = O.forward(cfg, w, p)
    for plan in ([214], [4] + [1] * 210, [64, 63, 1, 2, 65, 19], [130, 2, 2, 80]):
        got = run_schedule(eng, [[("x", n)] for n in plan], {"x": p})["x"]
        torch.testing.assert_close(got.double().cpu(), want, rtol=1e-4, atol=5e-4)
    from kllms_amd.models.mixers import RoutedExperts

    monkeypatch.setattr(RoutedExperts, "DENSE_MAX_ROWS", 0)
    got = run_schedule(eng, [[("z", 100)], [("z", 1)], [("z", 113)]], {"z": p})["z"]
    torch.testing.assert_close(got.double().cpu(), want, rtol=1e-4, atol=5e-4)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation(tmp_path, dtype):
    cfg = CFG_A
    w = write_model(str(tmp_path), cfg, seed=1)
    p1, p2 = toks(21, cfg["vocab"], 40), toks(5, cfg["vocab"], 41)
    sp = lambda n: SamplingParams(temperature=0.0, max_tokens=n)
    eng = gpu_engine(tmp_path, dtype, max_seq_len=256)
    out = eng.generate([GenRequest(prompt_ids=p1, n=2, sampling=sp(40)), GenRequest(prompt_ids=p2, n=1, sampling=sp(25))])
    assert out[0].streams[0].token_ids == out[0].streams[1].token_ids and len(out[1].streams[0].token_ids) == 25
    if dtype == "float32":
        assert out[0].streams[0].token_ids[:8] == oracle_greedy(cfg, w, p1, 8)
        assert out[1].streams[0].token_ids[:8] == oracle_greedy(cfg, w, p2, 8)
    assert eng.kv.allocator.num_free == eng.kv.num_blocks


@pytest.mark.parametrize("cfg,seed", [(CFG_A, 1), (CFG_B, 2), (CFG_C, 3)])
def test_bf16_close_to_oracle_and_cut_invariant(tmp_path, cfg, seed):
    """Serving mode: bf16 GEMMs, convolution rows and caches; fp32 stream,
    norms, scores, weights and the difference of the maps; sizes that are and
    are not multiples of the kernels' vector width."""
    w = write_model(str(tmp_path), cfg, seed=seed)
    eng = gpu_engine(tmp_path, "bfloat16")
    p = toks(150, cfg["vocab"], 5)
    want = O.forward(cfg, w, p)
    whole = run_schedule(eng, [[("x", 150)]], {"x": p})["x"].double().cpu()
    cut = run_schedule(eng, [[("x", n)] for n in [2, 30, 1, 1, 31, 63, 22]], {"x": p})["x"].double().cpu()
    single = run_schedule(eng, [[("x", 100)]] + [[("x", 1)]] * 50, {"x": p})["x"].double().cpu()
    # nine rows in ten: in a row with two choice scores closer than a bf16 rounding another expert may be chosen
    err = lambda a, b: float((a - b).pow(2).mean(-1).sqrt().quantile(0.9) / want.std())
    assert err(whole, want) < 0.05
    assert err(cut, whole) < 0.05
    assert err(single, whole) < 0.05


def test_bf16_far_key_at_tile_borders(tmp_path):
    """An asking token whose map-1 queries are tied to one key, which sits at
    page and key-tile borders far back: asked from a prompt and decoded alone,
    the answer moves the output the way it moves the oracle's."""
    cfg = model_cfg([layer("attention", att(heads=4, kv_heads=2, dim=16, vdim=32, conv=1, scale=2.0, coef=0.0), None)],
                    vocab=64, width=64)
    w = O.random_weights(cfg, 8)
    for n in ("q", "k", "v"):
        w[f"l0.mix.{n}.conv"] = torch.ones_like(w[f"l0.mix.{n}.conv"])
    for n in ("lq1", "lk1", "lq2", "lk2"):
        w["l0.mix." + n] = torch.zeros(16, dtype=torch.float64)
    asker, answer = 5, 9
    w["embed"][answer] *= 3.0
    h = O.dyt(w, "l0.norm1", w["embed"][[asker, answer]] * cfg["embedding"]["scale"])
    key = (w["l0.mix.k"] @ h[1] + w["l0.mix.k.b"]).view(2, 2, 16)
    wq = w["l0.mix.q"].view(4, 2, 16, 64)
    for hd in range(4):
        wq[hd, 0] = 0.1 * wq[hd, 0] + torch.outer(key[hd // 2, 0], h[0] / (h[0] @ h[0]))
    w["l0.mix.q"] = w["l0.mix.q"].bfloat16().double()
    write_model(str(tmp_path), cfg, w=w)
    eng = gpu_engine(tmp_path, "bfloat16")
    base = [t if t not in (asker, answer) else 20 for t in toks(300, 64, 9)]
    base[-1] = asker
    gone = O.forward(cfg, w, base)[-1]
    for at in (0, 15, 16, 63, 64, 127, 128, 255, 256, 298):
        ids = list(base)
        ids[at] = answer
        want = O.forward(cfg, w, ids)[-1]
        moved = float((want - gone).pow(2).mean().sqrt())
        assert moved > 0.1
        for plan in ([300], [299, 1], [100, 150, 50]):
            got = run_schedule(eng, [[("x", n)] for n in plan], {"x": ids})["x"][-1].double().cpu()
            assert float((got - want).pow(2).mean().sqrt()) < 0.2 * moved


def test_preset_generates_on_gpu():
    eng = LLMEngine(EngineConfig(model="mid-dimuvik", device="cuda", max_kv_blocks=512, max_state_slots=16,
                                 use_hip_graphs=False, max_seq_len=1024))
    out = eng.generate([GenRequest(prompt_ids=list(range(1, 300)), n=3,
                                   sampling=SamplingParams(temperature=0.8, max_tokens=24, seed=3))])
    assert all(len(s.token_ids) > 0 for s in out[0].streams)
    assert eng.kv.allocator.num_free == eng.kv.num_blocks
