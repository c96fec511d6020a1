"""Fuvuvik through the engine (scheduler, paged pools, state slots, model
runner, ops) against the plain float64 oracle in tests/fuvuvik_oracle.py.

Every test writes its own small checkpoint (config.json + safetensors with
random bf16 weights) and loads it like a served model. The engine runs in
fp32 here so that a structural fault — a key on the wrong side of a chunk's
border, a lost state, a previous row taken from another request, a
convolution input missing at a portion's start, streams mixed the wrong way
round — shows far above the rounding floor; one test repeats the comparison
in bf16. Chunks are a few tokens long, so every key inside one carries
weight.
"""
import copy
import functools
import io
import json
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))
import fuvuvik_oracle as oracle  # noqa: E402
from test_fusipel import err, make_engine, replay, tokens_for  # noqa: E402

from gpustack_amd import ops  # noqa: E402
from gpustack_amd.engine import SamplingParams  # noqa: E402
from gpustack_amd.engine.config import (GruMixerSpec, ModelSpec,  # noqa: E402
                                        PagedMixerSpec)

TOL = 2e-4      # fp32 engine against the float64 oracle


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    cfg = oracle.make_config()
    w = oracle.make_weights(cfg, seed=3)
    d = oracle.save_model(tmp_path_factory.mktemp("fuvuvik"), cfg, w)
    return cfg, w, d


def _one(tmp_path, layers, n=41, seed=0, width=22, streams=3, steps=None,
         dtype="float32", change=None):
    """A model of the given layers: whole prompt (or `steps`) vs oracle."""
    cfg = oracle.make_config(width=width, streams=streams, layers=layers)
    w = oracle.make_weights(cfg, seed=seed)
    if change is not None:
        change(w)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, n, seed + 11)
    got = replay(make_engine(d, dtype=dtype), {"a": toks},
                 steps or [[("a", n)]])["a"]
    return err(got, oracle.forward(cfg, w, toks))


# ---- configuration ------------------------------------------------------------

def test_config_is_read_from_the_file(model):
    cfg, _, d = model
    spec = ModelSpec.from_dir(d)
    assert spec.architecture == "Fuvuvik" and spec.fp32_residual
    assert spec.vocab_size == cfg["vocab"] and spec.hidden_size == cfg["width"]
    assert spec.rms_norm_eps == cfg["norm"]["eps"]
    assert spec.embed_scale == cfg["embedding"]["scale"]
    assert spec.streams == cfg["streams"]
    assert spec.token_shift and spec.residual_gate and spec.has_state
    assert not spec.tie_word_embeddings
    assert [type(ls.mixer) for ls in spec.layers] == [
        PagedMixerSpec, PagedMixerSpec, GruMixerSpec, GruMixerSpec,
        PagedMixerSpec]
    for ls, ent in zip(spec.layers, cfg["layers"]):
        m, c = ls.mixer, ent["mixer"]
        if ent["type"] == "mingru":
            assert m.width == c["width"]
        else:
            assert (m.heads, m.kv_heads, m.qk_dim, m.v_dim, m.scale,
                    m.rot.dims, m.rot.base, m.rot.layout, m.out_gate) == (
                c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["scale"],
                c["rot"]["dims"], c["rot"]["base"], "half", True)
            if ent["type"] == "attention":
                assert (m.conv, m.unit_norm, m.chunk, m.unit_sink) == (
                    c["conv"], True, 0, False)
            else:
                assert (m.conv, m.unit_norm, m.chunk, m.unit_sink) == (
                    0, False, c["mask"]["size"], True)
        if ent["mlp"] is None:
            assert ls.mlp is None
        else:
            assert (ls.mlp.ff, ls.mlp.act, ls.mlp.gated) == (
                ent["mlp"]["ff"], "gelu_tanh", True)
    c0, c1, c2 = (cfg["layers"][i]["mixer"] for i in (0, 1, 2))
    pools = spec.kv_pool_widths()
    assert pools[0] == ("kv", c0["kv_heads"], c0["dim"], c0["vdim"])
    assert pools[2] == ("state",)
    shapes = spec.state_pool_shapes()
    assert shapes[0] is None and shapes[2] == (1, 1, c2["width"], 0, 0)
    conv = (c1["heads"] + c1["kv_heads"]) * c1["dim"] \
        + c1["kv_heads"] * c1["vdim"]
    assert shapes[1] == (0, 0, 0, c1["conv"] - 1, conv)
    # fp32 recurrences, convolution rows and a previous row per layer
    assert spec.state_bytes_per_slot(2) == (
        4 * (c2["width"] + cfg["layers"][3]["mixer"]["width"])
        + 2 * (c1["conv"] - 1) * conv + 2 * len(cfg["layers"]) * cfg["width"])


def test_weight_count_matches_the_checkpoint(model):
    cfg, w, d = model
    n = sum(t.numel() for t in w.values())
    assert ModelSpec.from_dir(d).weight_bytes(2) == 2 * n


def test_bad_configurations_are_refused():
    bad = [
        [oracle.attention_layer(heads=3, kv_heads=2)],
        [oracle.chunk_layer(rot_dims=8, dim=6)],
        [oracle.chunk_layer(rot_dims=3)],
        [oracle.chunk_layer(size=0)],
        [oracle.attention_layer(conv=0)],
        [oracle.mingru_layer(width=0)],
    ]
    for layers in bad:
        with pytest.raises(ValueError):
            ModelSpec.from_hf_config(oracle.make_config(layers=layers))
    with pytest.raises(ValueError):
        ModelSpec.from_hf_config(oracle.make_config(streams=0))
    cfg = oracle.make_config(layers=[oracle.mingru_layer()])
    cfg["layers"][0]["type"] = "other"
    with pytest.raises(NotImplementedError):
        ModelSpec.from_hf_config(cfg)
    cfg = oracle.make_config(layers=[oracle.mingru_layer(ff=4)])
    cfg["layers"][0]["mlp"]["kind"] = "other"
    with pytest.raises(NotImplementedError):
        ModelSpec.from_hf_config(cfg)


def test_checkpoints_that_do_not_fit_are_refused(tmp_path):
    cfg = oracle.make_config(layers=[oracle.attention_layer()])
    w = oracle.make_weights(cfg)
    lost = {k: v for k, v in w.items() if k != "l0.shift"}
    with pytest.raises(KeyError):
        make_engine(oracle.save_model(tmp_path / "a", cfg, lost))
    wrong = dict(w, **{"l0.mix.k.conv": w["l0.mix.k.conv"][:, 1:]})
    with pytest.raises(ValueError):
        make_engine(oracle.save_model(tmp_path / "b", cfg, wrong))


def test_state_models_refuse_prefix_caching_and_speculation(tmp_path):
    """Even a stack without a recurrence carries rows between steps."""
    cfg = oracle.make_config(layers=[oracle.chunk_layer()])
    d = oracle.save_model(tmp_path, cfg, oracle.make_weights(cfg))
    with pytest.raises(ValueError):
        make_engine(d, enable_prefix_caching=True)
    with pytest.raises(ValueError):
        make_engine(d, speculative={"method": "ngram", "num_draft_tokens": 2})


def test_registry():
    from gpustack_amd.models import model_class_for
    from gpustack_amd.utils.model_registry import categories_for_architecture

    assert model_class_for("Fuvuvik").__name__ == "FuvuvikForCausalLM"
    assert categories_for_architecture("Fuvuvik") == ["llm"]


def test_random_weights_keep_the_streams_in_range():
    from gpustack_amd.bench.layer_bench import _engine, fuvuvik_spec

    spec = fuvuvik_spec(dict(width=64, heads=4, ff=48, layers=8))
    eng = _engine(spec, "cpu", 2, 64)
    toks = torch.randint(0, spec.vocab_size, (40,),
                         generator=torch.Generator().manual_seed(0)).tolist()
    out = eng.replay_step([("a", toks, [0, 39])], ["a"])
    assert out.shape == (2, spec.vocab_size) and bool(torch.isfinite(out).all())
    assert 0.2 < float(out.float().std()) < 5.0


# ---- each mechanism alone -----------------------------------------------------

i32 = lambda v: torch.tensor(v, dtype=torch.int32)


@pytest.mark.parametrize("S", [1, 2, 3, 5])
@pytest.mark.parametrize("gated", [True, False])
def test_stream_step_alone(S, gated):
    g = torch.Generator().manual_seed(S)
    T, W, eps = 6, 14, 1e-5
    x, a = torch.randn(T, S, W, generator=g), torch.randn(T, W, generator=g)
    r = torch.randn(T, W + 3, generator=g)[:, 2:2 + W] if gated else None
    rb = torch.randn(W, generator=g) if gated else None
    mix, b = torch.randn(S, S, generator=g), torch.randn(S, generator=g)
    rd, nw = torch.randn(S, generator=g), torch.rand(W, generator=g) + 0.5
    xs = x.double().transpose(0, 1)
    y = a.double()
    if gated:
        y = y * torch.sigmoid(r.double() + rb.double())
    new = oracle.stream_out(xs, mix, b, y)
    h = torch.zeros(T, W)
    ops.stream_step(x, a, r, rb, mix, b, rd, nw, eps, h)
    assert (x.double().transpose(0, 1) - new).abs().max() < 1e-5
    ref = oracle.rms_norm(oracle.stream_in(new, rd), nw, eps)
    assert (h.double() - ref).abs().max() < 1e-5
    # opening alone leaves the streams; closing alone asks for no norm
    before = x.clone()
    ops.stream_step(x, None, None, None, None, None, rd, nw, eps, h)
    assert torch.equal(x, before) and (h.double() - ref).abs().max() < 1e-5
    ops.stream_step(x, a, None, None, mix, b, None, None, eps, None)
    assert (x.double().transpose(0, 1)
            - oracle.stream_out(new, mix, b, a.double())).abs().max() < 1e-4


def test_token_shift_alone():
    """Two new sequences and one that goes on, slots out of order."""
    g = torch.Generator().manual_seed(1)
    W = 9
    mu = torch.rand(W, generator=g) * 2 - 0.5
    a, b, c = (torch.randn(n, W, generator=g) for n in (5, 7, 1))
    state = torch.randn(4, W, generator=g)            # junk to be ignored
    h = torch.cat([a, b[:4], c])
    hs = torch.zeros_like(h)
    ops.token_shift(hs, h, mu, state, i32([0, 5, 9]), i32([5, 4, 1]),
                    i32([3, 0, 2]), i32([0] * 5 + [1] * 4 + [2]),
                    i32([0, 1, 2, 3, 4, 0, 1, 2, 3, 0]))
    ref = [oracle.token_shift(t.double(), mu) for t in (a, b, c)]
    assert (hs[:5].double() - ref[0]).abs().max() < 1e-6
    assert (hs[5:9].double() - ref[1][:4]).abs().max() < 1e-6
    assert (hs[9:].double() - ref[2]).abs().max() < 1e-6
    hs2 = torch.zeros(3, W)
    ops.token_shift(hs2, b[4:], mu, state, i32([0]), i32([3]), i32([0]),
                    i32([0, 0, 0]), i32([4, 5, 6]))
    assert (hs2.double() - ref[1][4:]).abs().max() < 1e-6


@pytest.mark.parametrize("N", [1, 5, 16])
def test_gated_recurrence_alone(N):
    g = torch.Generator().manual_seed(N)
    rows = torch.randn(15, 3 * N + 2, generator=g) * 2
    zb, ub = torch.randn(N, generator=g), torch.randn(N, generator=g)
    state = torch.randn(3, 1, 1, N, generator=g)      # junk to be ignored

    def run(src, first, news, slots, pos):
        y = torch.zeros(src.shape[0], N)
        ops.gru_scan(y, src, 1, 1 + N, 2 + 2 * N, zb, ub, state, i32(first),
                     i32(news), i32(slots), i32(pos))
        return y.double()

    def ref(x):
        x = x.double()
        z = torch.sigmoid(x[:, 1:1 + N] + zb.double())
        c = oracle.mingru_candidate(x[:, 1 + N:1 + 2 * N] + ub.double())
        return oracle.mingru_recurrence(z, c) * oracle.silu(x[:, 2 + 2 * N:])

    y = run(rows[:11], [0, 6], [6, 5], [2, 0], [0, 1, 2, 3, 4, 5, 0, 1, 2, 3, 4])
    assert (y[:6] - ref(rows[:6])).abs().max() < 1e-5
    assert (y[6:] - ref(rows[6:])[:5]).abs().max() < 1e-5
    y = run(rows[11:], [0], [4], [0], [5, 6, 7, 8])
    assert (y - ref(rows[6:])[5:]).abs().max() < 1e-5


def test_candidate_is_continuous_at_zero():
    u = torch.tensor([-1e-9, 0.0, 1e-9], dtype=torch.float64)
    assert (oracle.mingru_candidate(u) - 0.5).abs().max() < 1e-8


@pytest.mark.parametrize("taps", [1, 2, 3, 6])
@pytest.mark.parametrize("silu,bias", [(False, False), (True, True)])
def test_short_convolution_alone(taps, silu, bias):
    g = torch.Generator().manual_seed(taps)
    C = 7
    src = torch.randn(17, C + 4, generator=g)
    w = torch.randn(C, taps, generator=g)
    b = torch.randn(C, generator=g) if bias else None
    st = torch.randn(3, taps - 1, C, generator=g)     # junk to be ignored
    full = oracle.causal_conv(src[:, 2:2 + C].double(), w)
    if bias:
        full = full + b.double()
    if silu:
        full = oracle.silu(full)
    at = 0
    for n in (1, 1, 2, 5, 1, 7):
        out = torch.zeros(n, C)
        ops.short_conv(out, src[at:at + n], 2, w, b, st, i32([0]), i32([n]),
                       i32([1]), i32([0] * n), i32(range(at, at + n)),
                       silu=silu)
        assert (out.double() - full[at:at + n]).abs().max() < 1e-5, at
        at += n


@pytest.mark.parametrize("rot_dims", [0, 4, 10])
@pytest.mark.parametrize("unit", [True, False])
def test_rotation_and_unit_heads_alone(rot_dims, unit):
    """The row kernel against: rotate, THEN divide by the root mean square."""
    g = torch.Generator().manual_seed(rot_dims)
    H, G, D, V, BS, T, eps = 3, 2, 10, 7, 4, 9, 1e-5
    src = torch.randn(T, (H + G) * D + G * V + 3, generator=g) * 0.01
    q = torch.zeros(T, H * D)
    kc, vc = torch.zeros(3, G, BS, D), torch.zeros(3, G, V, BS)
    slots = torch.randperm(3 * BS, generator=g)[:T]
    f = torch.tensor([30.0 ** (-2 * i / max(rot_dims, 1))
                      for i in range(rot_dims // 2)])
    nd = D if unit else 0
    rot0 = 0 if rot_dims else -1
    ops.head_rope_store(q, src, 0, H, D, None, nd, rot0, H * D, G, D, None, nd,
                        rot0, (H + G) * D, f, True, 1.0,
                        torch.arange(T, dtype=torch.int32), kc, vc, slots, eps)

    def ref(x, heads):
        x = x.double().view(T, heads, D).transpose(0, 1)
        if rot_dims:
            x = oracle.rotate(x, 30.0, rot_dims)
        return (oracle.rms_unit(x, eps) if unit else x).transpose(0, 1)

    assert (q.double().view(T, H, D) - ref(src[:, :H * D], H)).abs().max() < 1e-5
    k = kc[slots // BS, :, slots % BS]
    assert (k.double() - ref(src[:, H * D:(H + G) * D], G)).abs().max() < 1e-5
    v = src[:, (H + G) * D:(H + G) * D + G * V].view(T, G, V)
    assert torch.equal(vc[slots // BS, :, :, slots % BS], v)


@pytest.mark.parametrize("chunk,one,gated", [(0, False, True), (5, True, True),
                                             (5, False, False), (1, True, False),
                                             (100, True, True)])
def test_attention_alone(chunk, one, gated):
    g = torch.Generator().manual_seed(chunk + 7 * gated)
    T, H, G, D, V, BS = 23, 4, 2, 6, 5, 4
    q = torch.randn(T, H, D, generator=g)
    k, v = torch.randn(T, G, D, generator=g), torch.randn(T, G, V, generator=g)
    gate = torch.randn(T, H + 1, generator=g)[:, 1:] if gated else None
    bt = torch.randperm(8, generator=g)[:6].to(torch.int32)[None]
    kc, vc = torch.zeros(8, G, BS, D), torch.zeros(8, G, V, BS)
    t = torch.arange(T)
    kc[bt[0, t // BS].long(), :, t % BS] = k
    vc[bt[0, t // BS].long(), :, :, t % BS] = v
    out = torch.zeros(T, H, V)
    ops.paged_attention(out, q, kc, vc, bt, torch.zeros(T, dtype=torch.int32),
                        t.to(torch.int32), 0.7, chunk=chunk, gate=gate,
                        sinks=torch.zeros(H) if one else None)
    for a in range(H):
        ref = oracle.attend(q[:, a].double(), k[:, a // 2].double(),
                            v[:, a // 2].double(), 0.7, chunk, one)
        if gated:
            ref = ref * torch.sigmoid(gate[:, a:a + 1].double())
        assert (out[:, a].double() - ref).abs().max() < 1e-5


@pytest.mark.parametrize("layers", [
    [oracle.attention_layer(ff=0)], [oracle.attention_layer()],
    [oracle.chunk_layer(ff=0)], [oracle.chunk_layer()],
    [oracle.mingru_layer()], [oracle.mingru_layer(ff=10)],
])
def test_one_layer(tmp_path, layers):
    assert _one(tmp_path, layers) < TOL


def test_streams_mix_from_to_and_first_layer_sees_equal_streams(tmp_path):
    """A mixing matrix far from symmetric: transposing it changes the
    logits; so does forgetting that the update uses the old streams."""
    layers = [oracle.mingru_layer(ff=8), oracle.chunk_layer(ff=6)]
    cfg = oracle.make_config(layers=layers)
    w = oracle.make_weights(cfg, seed=6)
    for q in ("l0.hc1", "l0.hc2", "l1.hc1", "l1.hc2"):
        w[q + ".mix"] = torch.tensor([[0.5, 1.5, -0.5], [0.0, 0.25, 1.0],
                                      [-1.0, 0.0, 0.75]], dtype=torch.bfloat16)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, 20, 1)
    ref = oracle.forward(cfg, w, toks)
    assert err(replay(make_engine(d), {"a": toks}, [[("a", 20)]])["a"], ref) < TOL
    turned = {k: v.t() if k.endswith(".mix") else v for k, v in w.items()}
    assert err(oracle.forward(cfg, turned, toks), ref) > 0.05


def test_strong_gates_and_shifts(tmp_path):
    """Shifts past 1 and below 0, gates near their ends."""
    def change(w):
        g = torch.Generator().manual_seed(0)
        for k, v in w.items():
            if k.endswith(".shift"):
                w[k] = (torch.randn(v.shape, generator=g) * 1.5).bfloat16()
            if k.endswith(("rg1.b", "rg2.b")):
                w[k] = (torch.randn(v.shape, generator=g) * 4).bfloat16()

    assert _one(tmp_path, None, n=30, change=change,
                steps=[[("a", 9)]] + [[("a", 1)]] * 4 + [[("a", 17)]]) < TOL


def test_one_in_the_denominator_matters(tmp_path):
    cfg = oracle.make_config(layers=[oracle.chunk_layer()])
    w = oracle.make_weights(cfg, seed=2)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, 30, 2)
    ref = oracle.forward(cfg, w, toks)
    got = replay(make_engine(d), {"a": toks}, [[("a", 30)]])["a"]
    assert err(got, ref) < TOL
    plain = copy.deepcopy(cfg)
    plain["layers"][0]["mixer"]["mask"]["no_one"] = True
    assert err(oracle.forward(plain, w, toks), ref) > 0.02


@pytest.mark.parametrize("streams,width,layers", [
    # one stream, one head, one tap, chunks of one position, no feed-forward
    (1, 10, [oracle.attention_layer(heads=1, kv_heads=1, dim=4, vdim=3, conv=1,
                                    rot_dims=2, ff=0),
             oracle.chunk_layer(heads=1, kv_heads=1, dim=2, vdim=7, size=1,
                                rot_dims=2, ff=0),
             oracle.mingru_layer(width=1, ff=3)]),
    # kv heads == heads, value size == key size, full rotation
    (2, 18, [oracle.attention_layer(heads=2, kv_heads=2, dim=6, vdim=6, conv=2,
                                    rot_dims=6, ff=9),
             oracle.mingru_layer(width=18),
             oracle.chunk_layer(heads=3, kv_heads=3, dim=4, vdim=4, size=16,
                                rot_dims=4, ff=7)]),
    # no rotation, chunk wider than the sequence, more streams, many heads
    (7, 13, [oracle.chunk_layer(heads=18, kv_heads=1, dim=3, vdim=2, size=500,
                                rot_dims=0, ff=5),
             oracle.mingru_layer(width=31, ff=4),
             oracle.attention_layer(heads=6, kv_heads=3, dim=5, vdim=8, conv=7,
                                    rot_dims=4, ff=0)]),
])
def test_other_sizes(tmp_path, streams, width, layers):
    steps = [[("a", 11)], [("a", 2)], [("a", 19)]] + [[("a", 1)]] * 5
    assert _one(tmp_path, layers, n=37, width=width, streams=streams,
                steps=steps) < TOL


def test_other_constants(tmp_path):
    cfg = oracle.make_config(eps=0.05, embed_scale=1.0)
    w = oracle.make_weights(cfg, seed=8)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, 25, 3)
    ref = oracle.forward(cfg, w, toks)
    got = replay(make_engine(d), {"a": toks}, [[("a", 25)]])["a"]
    assert err(got, ref) < TOL
    other = dict(cfg, norm={"eps": 1e-5})
    assert err(oracle.forward(other, w, toks), ref) > 0.01


# ---- schedules ------------------------------------------------------------------

def test_whole_prompts_and_first_tokens(model):
    cfg, w, d = model
    eng = make_engine(d)
    for n in (1, 2, 3, 17, 64):
        toks = tokens_for(cfg, n, n)
        got = replay(eng, {"a": toks}, [[("a", n)]])["a"]
        assert err(got, oracle.forward(cfg, w, toks)) < TOL, n


def test_prefill_equals_token_by_token(model):
    cfg, w, d = model
    toks = tokens_for(cfg, 50, 7)
    ref = oracle.forward(cfg, w, toks)
    eng = make_engine(d)
    whole = replay(eng, {"a": toks}, [[("a", 50)]])["a"]
    single = replay(eng, {"a": toks}, [[("a", 1)]] * 50)["a"]
    late = replay(eng, {"a": toks}, [[("a", 18)]] + [[("a", 1)]] * 32)["a"]
    for got in (whole, single, late):
        assert err(got, ref) < TOL
    assert err(single, whole) < 1e-5 and err(late, whole) < 1e-5


@pytest.mark.parametrize("sizes", [[2] * 20, [16, 16, 8], [15, 2, 17, 1, 5],
                                   [1, 2, 3, 31, 3], [33, 7], [9, 31]])
def test_portions(model, sizes):
    """Portions cut inside pages, chunks and the convolution's reach."""
    cfg, w, d = model
    toks = tokens_for(cfg, sum(sizes), 3)
    got = replay(make_engine(d), {"a": toks}, [[("a", n)] for n in sizes])["a"]
    assert err(got, oracle.forward(cfg, w, toks)) < TOL


def test_unequal_batch_equals_each_alone(model):
    cfg, w, d = model
    prompts = {"a": tokens_for(cfg, 40, 1), "b": tokens_for(cfg, 9, 2),
               "c": tokens_for(cfg, 23, 3), "d": tokens_for(cfg, 30, 4)}
    schedule = [
        [("a", 20), ("b", 2)],
        [("b", 1), ("a", 1), ("c", 12)],
        [("c", 1), ("a", 1), ("b", 1)],                    # single rows only
        [("c", 1), ("d", 30), ("a", 1)],
        [("a", 17), ("b", 5), ("c", 9)],
    ]
    eng = make_engine(d)
    got = replay(eng, prompts, schedule)
    for r, toks in prompts.items():
        assert err(got[r], oracle.forward(cfg, w, toks)) < TOL, r
        alone = replay(eng, {r: toks}, [[(r, len(toks))]])[r]
        assert err(got[r], alone) < 1e-5, r


def test_blocks_and_slots_are_used_again(model):
    """A pool of 7 usable blocks and 2 state slots: every request takes
    blocks and a slot that an ended one has just given back."""
    cfg, w, d = model
    eng = make_engine(d, blocks=8, max_seqs=2)
    kv = eng.scheduler.kv
    free0, slots0 = kv.allocator.num_free, kv.state_allocator.num_free
    prompts = {f"r{i}": tokens_for(cfg, n, 20 + i)
               for i, n in enumerate([50, 33, 17, 60, 40, 31])}
    schedule = [
        [("r0", 30), ("r1", 2)], [("r0", 20), ("r1", 31)],      # r0, r1 end
        [("r2", 16), ("r3", 40)], [("r2", 1), ("r3", 20)],      # r2, r3 end
        [("r4", 1), ("r5", 1)],                       # new ones, single rows
        [("r4", 37), ("r5", 2)], [("r4", 2), ("r5", 28)],
    ]
    got = replay(eng, prompts, schedule)
    for r, toks in prompts.items():
        assert err(got[r], oracle.forward(cfg, w, toks)) < TOL, r
    assert kv.allocator.num_free == free0
    assert kv.state_allocator.num_free == slots0


def test_long_decoding_across_pages_and_chunks(model):
    cfg, w, d = model
    toks = tokens_for(cfg, 5 + 140, 13)
    got = replay(make_engine(d), {"a": toks},
                 [[("a", 5)]] + [[("a", 1)]] * 140)["a"]
    assert err(got, oracle.forward(cfg, w, toks)) < TOL


def test_bf16_engine_is_close(model):
    cfg, w, d = model
    toks = tokens_for(cfg, 40, 5)
    eng = make_engine(d, dtype="bfloat16")
    got = replay(eng, {"a": toks}, [[("a", 23)], [("a", 16)], [("a", 1)]])["a"]
    assert err(got, oracle.forward(cfg, w, toks)) < 0.15


# ---- faults that random weights would hide ------------------------------------------

@functools.lru_cache(maxsize=None)
def standout_tokens(kind):
    """(one-layer configuration, weights, far token, last token) such that,
    behind a prompt of filler token 0, the LAST token's scores single out the
    far token: of a few last tokens and all far ones the pair whose presence
    changes the last row most (a search with the oracle that sees every key).
    The score scale is large, so the softmax is nearly one-hot: losing that
    key, or wrongly admitting it, changes the row wholly. Nothing is rotated,
    and the shift and all taps but the current one are zero, so a key depends
    on its own token only, wherever it stands."""
    if kind == "chunk":
        L = oracle.chunk_layer(heads=2, kv_heads=2, dim=8, vdim=6, size=10 ** 6,
                               scale=4.0, rot_dims=0, ff=0)
    else:
        L = oracle.attention_layer(heads=2, kv_heads=1, dim=12, vdim=6, conv=3,
                                   scale=3.0, rot_dims=0, ff=0)
    cfg = oracle.make_config(width=16, vocab=40, layers=[L])
    w = oracle.make_weights(cfg, seed=9)
    w["l0.shift"] = torch.zeros(16, dtype=torch.bfloat16)
    for nm in "qkv":
        c = f"l0.mix.{nm}.conv"
        if c in w:
            w[c][:, :-1] = 0
    best, pair = -1.0, None
    for last in (39, 38, 37):
        base = oracle.forward(cfg, w, [0] * 23 + [last])[-1:]
        for t in range(1, 37):
            e = err(oracle.forward(cfg, w, [0] * 11 + [t] + [0] * 11 + [last])
                    [-1:], base)
            if e > best:
                best, pair = e, (t, last)
    return cfg, w, *pair


def standout_model(tmp_path, kind, far_pos, n, chunk=1000):
    cfg, w, far, last = standout_tokens(kind)
    cfg = copy.deepcopy(cfg)
    if kind == "chunk":
        cfg["layers"][0]["mixer"]["mask"]["size"] = chunk
    toks = [0] * n
    toks[far_pos] = far
    toks[-1] = last
    return cfg, w, oracle.save_model(tmp_path, cfg, w), toks


@pytest.mark.parametrize("kind", ["causal", "chunk"])
@pytest.mark.parametrize("far_pos", [0, 15, 16, 31, 200])
@pytest.mark.parametrize("decode", [False, True])
def test_far_key_among_hundreds(tmp_path, kind, far_pos, decode):
    cfg, w, d, toks = standout_model(tmp_path, kind, far_pos, 300)
    ref = oracle.forward(cfg, w, toks)[-1:]
    other = list(toks)
    other[far_pos] = 0
    assert err(oracle.forward(cfg, w, other)[-1:], ref) > 0.05
    eng = make_engine(d)
    n = len(toks)
    steps = [[("a", n - 1)], [("a", 1)]] if decode else [[("a", n)]]
    got = replay(eng, {"a": toks}, steps)["a"][-1:]
    assert err(got, ref) < TOL


# last row 82 in chunks of 19: its chunk starts at 76. In chunks of 16 it
# starts on a page border (80), and with 83 tokens in chunks of 82 it is the
# first of its chunk
@pytest.mark.parametrize("chunk,far_pos,seen", [
    (19, 75, False), (19, 76, True), (19, 77, True), (16, 79, False),
    (16, 80, True), (82, 81, False), (82, 0, False), (83, 0, True)])
@pytest.mark.parametrize("steps", [
    [[("a", 83)]], [[("a", 40)], [("a", 43)]], [[("a", 76)], [("a", 7)]],
    [[("a", 75)], [("a", 2)], [("a", 6)]], [[("a", 82)], [("a", 1)]],
    [[("a", 70)]] + [[("a", 1)]] * 13])
def test_chunk_border(tmp_path, chunk, far_pos, seen, steps):
    cfg, w, d, toks = standout_model(tmp_path, "chunk", far_pos, 83, chunk)
    ref = oracle.forward(cfg, w, toks)[-1:]
    got = replay(make_engine(d), {"a": toks}, steps)["a"][-1:]
    assert err(got, ref) < TOL
    # the key decides the row exactly if it is inside
    other = list(toks)
    other[far_pos] = 0
    moved = err(oracle.forward(cfg, w, other)[-1:], ref)
    assert moved > 0.05 if seen else moved < 1e-9
    # and a border one position off would show
    if far_pos in (75, 76, 79, 80):
        bad = copy.deepcopy(cfg)
        bad["layers"][0]["mixer"]["mask"]["misplaced"] = 1 if not seen else -1
        shifted = oracle.forward(bad, w, toks)[-1:]
        assert err(shifted, ref) > 0.05


def test_state_carries_the_first_token_to_the_last_row(tmp_path):
    """A recurrence that hardly forgets: the first token still shapes the
    last row, through a prompt cut into portions and decoded tokens."""
    cfg = oracle.make_config(width=16, layers=[oracle.mingru_layer(width=12)])
    w = oracle.make_weights(cfg, seed=4)
    w["l0.mix.z"] *= 0.2
    w["l0.mix.z.b"] = torch.full((12,), -5.0, dtype=torch.bfloat16)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, 60, 8)
    ref = oracle.forward(cfg, w, toks)
    # the shift and the recurrence hand the first token on; only the
    # recurrence reaches the last row
    other = [(toks[0] + 1) % cfg["vocab"]] + toks[1:]
    assert err(oracle.forward(cfg, w, other)[-1:], ref[-1:]) > 1e-3
    steps = [[("a", 3)], [("a", 20)], [("a", 2)], [("a", 20)]] + [[("a", 1)]] * 15
    got = replay(make_engine(d), {"a": toks}, steps)["a"]
    assert err(got, ref) < 2e-5


def test_shift_and_convolution_across_portion_starts(tmp_path):
    """Portions shorter than the convolution's reach; every portion's first
    row reads the previous step's last row."""
    layers = [oracle.attention_layer(conv=6), oracle.chunk_layer(size=4),
              oracle.attention_layer(conv=5, heads=2, ff=0)]
    steps = [[("a", 1)], [("a", 2)], [("a", 1)], [("a", 3)], [("a", 2)],
             [("a", 12)], [("a", 1)], [("a", 1)], [("a", 4)]]

    def change(w):
        for i in range(3):
            w[f"l{i}.shift"] = torch.full((22,), 0.9, dtype=torch.bfloat16)

    assert _one(tmp_path, layers, n=27, steps=steps, change=change) < TOL


def test_interrupted_requests_keep_their_rows(model):
    """A request that is left out of some steps goes on from its own slot."""
    cfg, w, d = model
    prompts = {"a": tokens_for(cfg, 25, 31), "b": tokens_for(cfg, 25, 32)}
    schedule = [[("a", 7)], [("b", 9)], [("b", 1)], [("b", 1)], [("a", 1)],
                [("b", 2)], [("a", 2), ("b", 1)], [("a", 15)], [("b", 11)]]
    got = replay(make_engine(d), prompts, schedule)
    for r, toks in prompts.items():
        assert err(got[r], oracle.forward(cfg, w, toks)) < TOL, r


# ---- the framework's own entry points -------------------------------------------

def test_greedy_generation_through_the_scheduler(model):
    cfg, w, d = model
    eng = make_engine(d)
    prompts = [tokens_for(cfg, n, 40 + n) for n in (3, 21, 9)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=14, temperature=0.0,
                                                ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert o == oracle.greedy(cfg, w, p, 14)


def test_generation_with_chunked_prefill_and_small_pool(model):
    cfg, w, d = model
    eng = make_engine(d, blocks=14, max_prefill_tokens=16)
    prompts = [tokens_for(cfg, n, 60 + n) for n in (45, 7, 30)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=10, temperature=0.0,
                                                ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert o == oracle.greedy(cfg, w, p, 10)


def test_replay_command(model, tmp_path):
    """The replay driver writes the wanted rows, step by step."""
    import numpy as np

    from gpustack_amd.engine.replay import run_trace

    cfg, w, d = model
    toks = tokens_for(cfg, 30, 77)
    lines = [json.dumps({"step": 0, "entries": [
                {"id": "x", "tokens": toks[:20], "want": [0, 19]}], "end": []}),
             json.dumps({"step": 1, "entries": [
                 {"id": "x", "tokens": toks[20:29], "want": []}], "end": []}),
             json.dumps({"step": 2, "entries": [
                 {"id": "x", "tokens": toks[29:], "want": [0]}], "end": ["x"]})]
    out = io.StringIO()
    assert run_trace(d, "float32", str(tmp_path / "o"), 64, lines=lines,
                     out=out, device="cpu") == 0
    assert out.getvalue().split() == ["done", "0", "done", "1", "done", "2"]
    ref = oracle.forward(cfg, w, toks)
    a = torch.from_numpy(np.fromfile(tmp_path / "o" / "0.f32", dtype="<f4")
                         ).view(2, -1)
    b = torch.from_numpy(np.fromfile(tmp_path / "o" / "2.f32", dtype="<f4")
                         ).view(1, -1)
    assert not (tmp_path / "o" / "1.f32").exists()
    assert err(a, ref[[0, 19]]) < TOL and err(b, ref[[29]]) < TOL
