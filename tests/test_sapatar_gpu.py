"""Sapatar on the GPU: the engine with the HIP kernels (stream rows with
several shifts, memory scan and step, windowed fp32 vector-ALU and bf16 MFMA
attention, gated grouped experts, captured decode graphs) against the float64
oracle, on the schedules and the crafted cases of tests/test_sapatar.py."""
import copy
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))
import sapatar_oracle as oracle  # noqa: E402
import test_fusipel as tf  # noqa: E402
import test_sapatar as tm  # noqa: E402
from test_fuvuvik_gpu import REQS, STEPS, gpu_engine, rows_over  # noqa: E402,F401

from gpustack_amd import ops  # noqa: E402
from gpustack_amd.engine import SamplingParams  # noqa: E402

pytestmark = pytest.mark.gpu

# sizes the MFMA attention, the grouped expert kernels and the 16-byte row
# paths accept, still unlike each other
ALIGNED = dict(width=128, vocab=97, streams=4, layers=[
    oracle.parallel_layer(heads=6, kv_heads=3, dim=64, vdim=48, size=37,
                          scale=0.2, rot_dims=48, base=500.0, r_heads=3,
                          r_dim=40, r_vdim=24, cap=9.0,
                          mlp=oracle.moe(7, 3, 64, 72)),
    oracle.retention_layer(heads=2, dim=72, vdim=56, rot_dims=48, base=900.0,
                           mlp=oracle.moe(4, 2, 128, 16)),
    oracle.wkv_layer(heads=3, dim=80, mlp=oracle.moe(5, 1, 64, 40)),
    oracle.parallel_layer(heads=2, kv_heads=2, dim=32, vdim=32, size=130,
                          scale=0.25, rot_dims=16, base=2000.0, r_heads=1,
                          r_dim=136, r_vdim=128, mlp=None),
])
ALIGNED["layers"] += [oracle.again(ALIGNED["layers"], 2),
                      oracle.again(ALIGNED["layers"], 0)]


def _model(tmp_path, kw, seed=3, **wkw):
    cfg = oracle.make_config(**kw)
    w = oracle.make_weights(cfg, seed=seed, **wkw)
    return cfg, w, oracle.save_model(tmp_path / "m", cfg, w)


def _kw(name):
    return {} if name == "default" else ALIGNED


def settled(kw):
    """The same with every expert chosen. In bf16, a router close to a tie
    sends a token to other experts than the oracle's, which is no fault;
    where all are chosen there are no ties, and rows can be bounded."""
    kw = copy.deepcopy(kw or dict(layers=oracle.make_config()["layers"]))
    for ent in kw["layers"]:
        if ent["mlp"]:
            ent["mlp"]["router"]["top"] = ent["mlp"]["router"]["experts"]
    return kw


@pytest.mark.parametrize("name", ["default", "aligned"])
def test_fp32_engine_matches_oracle(tmp_path, gpu_engine, name):
    cfg, w, d = _model(tmp_path, _kw(name))
    eng = gpu_engine(d)
    reqs = {i: tf.tokens_for(cfg, n, 70 + n) for i, n in REQS.items()}
    got = tf.replay(eng, reqs, STEPS)
    for i, t in reqs.items():
        assert tf.err(got[i], oracle.forward(cfg, w, t)) < 5e-4, i


@pytest.mark.parametrize("name", ["default", "aligned"])
def test_bf16_engine_with_block_and_slot_reuse(tmp_path, gpu_engine, name):
    """bf16 serving path (MFMA attention for the aligned sizes, the fp32
    vector path for the others) in a pool that every repetition refills,
    with as many state slots as live requests."""
    cfg, w, d = _model(tmp_path, settled(_kw(name)))
    eng = gpu_engine(d, dtype="bfloat16", blocks=18)
    kv = eng.runner.kv
    if name == "aligned":
        for i, D in ((0, 64), (3, 32)):
            q = torch.empty(1, 1, D, dtype=torch.bfloat16, device="cuda")
            assert ops._load_paged().paged_attention_uses_mfma(
                q, kv.k_caches[i], kv.v_caches[i])
    for rnd in range(3):
        reqs = {i: tf.tokens_for(cfg, n, 80 + n + rnd) for i, n in REQS.items()}
        got = tf.replay(eng, reqs, STEPS)
        over = sum(rows_over(got[i], oracle.forward(cfg, w, t), 0.15) * len(t)
                   for i, t in reqs.items())
        assert over <= 0.1 * sum(REQS.values()), rnd
        assert kv.state_allocator.num_free == 4


def test_bf16_logits_do_not_depend_on_the_schedule(tmp_path, gpu_engine):
    for kw, share in ((settled(ALIGNED), 0.0), (ALIGNED, 0.25)):
        cfg, w, d = _model(tmp_path / str(share), kw)
        eng = gpu_engine(d, dtype="bfloat16")
        reqs = {i: tf.tokens_for(cfg, n, 90 + n) for i, n in REQS.items()}
        mixed = tf.replay(eng, reqs, STEPS)
        for i, t in reqs.items():
            whole = tf.replay(eng, {i: t}, [[(i, len(t))]])[i]
            assert rows_over(mixed[i], whole.double(), 0.15) <= share, i


@pytest.mark.parametrize("sizes", [[2] * 20, [3, 2, 5, 2, 16, 1, 1, 17, 2, 11],
                                   [33, 1, 1, 40], [70, 2, 129]])
@pytest.mark.parametrize("name", ["default", "aligned"])
def test_portions_fp32(tmp_path, gpu_engine, sizes, name):
    cfg, w, d = _model(tmp_path, _kw(name))
    toks = tf.tokens_for(cfg, sum(sizes), 3)
    got = tf.replay(gpu_engine(d), {"a": toks}, [[("a", n)] for n in sizes])["a"]
    assert tf.err(got, oracle.forward(cfg, w, toks)) < 5e-4


def test_other_sizes_fp32_and_bf16(tmp_path, gpu_engine):
    """One head, heads of one channel, windows of one, many heads per key
    head, wide states, more streams than the wide row kernel takes, sizes
    that no vector path divides, no feed-forward, one expert."""
    layers = [
        oracle.parallel_layer(heads=1, kv_heads=1, dim=4, vdim=3, size=1,
                              rot_dims=2, r_heads=1, r_dim=1, r_vdim=1,
                              cap=15.0, mlp=None),
        oracle.retention_layer(heads=5, dim=3, vdim=13, rot_dims=2,
                               mlp=oracle.moe(1, 1, 5, 7)),
        oracle.wkv_layer(heads=1, dim=1),
        oracle.parallel_layer(heads=36, kv_heads=2, dim=6, vdim=2, size=500,
                              rot_dims=6, r_heads=2, r_dim=300, r_vdim=20,
                              mlp=oracle.moe(3, 3, 11, 1)),
        oracle.retention_layer(heads=1, dim=260, vdim=70, rot_dims=100,
                               mlp=None),
        oracle.wkv_layer(heads=2, dim=90, mlp=None),
    ]
    for streams, width in ((1, 18), (7, 13)):
        cfg, w, d = _model(tmp_path / str(width),
                           dict(width=width, streams=streams, layers=layers),
                           rank=5)
        toks = tf.tokens_for(cfg, 37, 11)
        steps = [[("a", 11)], [("a", 2)], [("a", 19)]] + [[("a", 1)]] * 5
        ref = oracle.forward(cfg, w, toks)
        got = tf.replay(gpu_engine(d), {"a": toks}, steps)["a"]
        assert tf.err(got, ref) < 5e-4
        got = tf.replay(gpu_engine(d, dtype="bfloat16"), {"a": toks}, steps)["a"]
        assert rows_over(got, ref, 0.25) <= 0.1


def test_long_decoding_fp32(tmp_path, gpu_engine):
    cfg, w, d = _model(tmp_path, ALIGNED)
    toks = tf.tokens_for(cfg, 5 + 140, 13)
    got = tf.replay(gpu_engine(d), {"a": toks},
                    [[("a", 5)]] + [[("a", 1)]] * 140)["a"]
    assert tf.err(got, oracle.forward(cfg, w, toks)) < 5e-4


@pytest.mark.parametrize("far_pos", [0, 16, 511, 700])
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_key_among_a_thousand(tmp_path, gpu_engine, far_pos, decode, dtype):
    """Long enough for a decode row's keys to be split over workgroups."""
    cfg, w, d, toks = tm.standout_model(tmp_path, far_pos, 1100, 1100)
    ref = oracle.forward(cfg, w, toks)[-1:]
    n = len(toks)
    steps = [[("a", n - 1)], [("a", 1)]] if decode else [[("a", n)]]
    got = tf.replay(gpu_engine(d, dtype=dtype, blocks=80), {"a": toks},
                    steps)["a"][-1:]
    assert tf.err(got, ref) < (5e-4 if dtype == "float32" else 0.15)


@pytest.mark.parametrize("window,far_pos", [(7, 75), (7, 76), (3, 79), (3, 80),
                                            (19, 63), (19, 64), (1, 81)])
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_window_edge(tmp_path, gpu_engine, window, far_pos, decode, dtype):
    n = 83
    cfg, w, d, toks = tm.standout_model(tmp_path, far_pos, n, window)
    ref = oracle.forward(cfg, w, toks)[-1:]
    steps = [[("a", n - 1)], [("a", 1)]] if decode \
        else [[("a", 40)], [("a", n - 40)]]
    got = tf.replay(gpu_engine(d, dtype=dtype), {"a": toks}, steps)["a"][-1:]
    assert tf.err(got, ref) < (5e-4 if dtype == "float32" else 0.15)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_generation_with_graphs(tmp_path, gpu_engine, dtype):
    """Greedy generation through the scheduler, chunked prefill and (bf16)
    the captured decode graphs; fp32 must reproduce the oracle's tokens."""
    cfg, w, d = _model(tmp_path, ALIGNED)
    eng = gpu_engine(d, dtype=dtype, blocks=40, max_prefill_tokens=32)
    assert eng.runner.model.graph_capturable() == (dtype == "bfloat16")
    prompts = [tf.tokens_for(cfg, n, 60 + n) for n in (45, 7, 30)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0,
                                                ignore_eos=True))
    assert all(len(o) == 12 for o in outs)
    if dtype == "float32":
        for p, o in zip(prompts, outs):
            assert o == oracle.greedy(cfg, w, p, 12)
    # a second round re-uses blocks, slots and graphs
    outs2 = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0,
                                                 ignore_eos=True))
    assert outs2 == outs


def test_captured_decoding_equals_eager(tmp_path, gpu_engine):
    """The tokens a captured decode graph picks, step after step, are those
    of single-row steps that run eagerly from the same prompt."""
    cfg, w, d = _model(tmp_path, ALIGNED, seed=4)
    eng = gpu_engine(d, dtype="bfloat16", blocks=40)
    prompts = [tf.tokens_for(cfg, n, 30 + n) for n in (21, 5, 40)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=16, temperature=0.0,
                                                ignore_eos=True))
    for p, o in zip(prompts, outs):
        toks = p + o[:-1]
        got = tf.replay(eng, {"a": toks}, [[("a", len(p))]]
                        + [[("a", 1)]] * 15)["a"][len(p) - 1:]
        # the choice is the eager row's best token, or within rounding of it
        best = got.max(-1)[0]
        mine = got.gather(1, torch.tensor(o)[:, None])[:, 0]
        assert float((best - mine).max()) < 0.1
