"""Sapatar through the engine (scheduler, paged pools, state slots, model
runner, ops) against the plain float64 oracle in tests/sapatar_oracle.py.

Every test writes its own small checkpoint (config.json + safetensors with
random bf16 weights) and loads it like a served model. The engine runs in
fp32 here so that a structural fault — a key on the wrong side of a window's
edge, a lost state or normaliser, a previous row taken from another request,
a running maximum that starts elsewhere, streams mixed the wrong way round,
a cache shared by two layers that share weights only — shows far above the
rounding floor; one test repeats the comparison in bf16. Windows are a few
tokens long, so every key inside one carries weight.
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
import sapatar_oracle as oracle  # noqa: E402
from test_fusipel import err, make_engine, replay, tokens_for  # noqa: E402

from gpustack_amd import ops  # noqa: E402
from gpustack_amd.engine import SamplingParams  # noqa: E402
from gpustack_amd.engine.config import (ModelSpec, ParallelMixerSpec,  # noqa: E402
                                        ScanMixerSpec)

TOL = 2e-4      # fp32 engine against the float64 oracle

i32 = lambda v: torch.tensor(list(v), dtype=torch.int32)


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    cfg = oracle.make_config()
    w = oracle.make_weights(cfg, seed=3)
    d = oracle.save_model(tmp_path_factory.mktemp("sapatar"), cfg, w)
    return cfg, w, d


def _one(tmp_path, layers, n=41, seed=0, width=22, streams=3, steps=None,
         dtype="float32", change=None, eps=1e-5, rank=3):
    """A model of the given layers: whole prompt (or `steps`) vs oracle."""
    cfg = oracle.make_config(width=width, streams=streams, layers=layers,
                             eps=eps)
    w = oracle.make_weights(cfg, seed=seed, rank=rank)
    if change is not None:
        change(w)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, n, seed + 11)
    got = replay(make_engine(d, dtype=dtype), {"a": toks},
                 steps or [[("a", n)]])["a"]
    return err(got, oracle.forward(cfg, w, toks))


# ---- configuration ------------------------------------------------------------

def test_config_is_read_from_the_file(model):
    cfg, w, d = model
    spec = ModelSpec.from_dir(d)
    assert spec.architecture == "Sapatar" and spec.fp32_residual
    assert spec.vocab_size == cfg["vocab"] and spec.hidden_size == cfg["width"]
    assert spec.rms_norm_eps == cfg["norm"]["eps"]
    assert spec.streams == cfg["streams"] and spec.has_state
    assert not spec.token_shift and not spec.residual_gate
    assert not spec.tie_word_embeddings
    assert [ls.weights_of for ls in spec.layers] == [
        ent.get("weights_of", -1) for ent in cfg["layers"]]
    pools, shapes, extra = (spec.kv_pool_widths(), spec.state_pool_shapes(),
                            spec.extra_state_shapes())
    for i, (ls, ent) in enumerate(zip(spec.layers, cfg["layers"])):
        m, c = ls.mixer, ent["mixer"]
        if ent["type"] == "parallel":
            assert isinstance(m, ParallelMixerSpec)
            a, b = c["left"], c["right"]
            assert (m.left.heads, m.left.kv_heads, m.left.qk_dim, m.left.v_dim,
                    m.left.scale, m.left.window, m.left.bias, m.left.rot.dims,
                    m.left.rot.base, m.left.rot.layout) == (
                a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["scale"],
                a["mask"]["size"], True, a["rot"]["dims"], a["rot"]["base"],
                "half")
            assert (m.right.kind, m.right.heads, m.right.state, m.right.vdim,
                    m.right.gate_cap) == ("mlstm", b["heads"], b["dim"],
                                          b["vdim"], b["gate_cap"])
            assert m.scales == (c["left_scale"], c["right_scale"])
            assert pools[i] == ("kv", a["kv_heads"], a["dim"], a["vdim"])
            assert shapes[i] == (b["heads"], b["dim"], b["vdim"], 0, 0)
            assert extra[i] == (b["heads"], b["dim"] + 1)
        elif ent["type"] == "retention":
            assert isinstance(m, ScanMixerSpec) and m.kind == "retention"
            assert (m.heads, m.state, m.vdim, m.rot.dims, m.rot.base,
                    m.rot.layout, list(m.decay)) == (
                c["heads"], c["dim"], c["vdim"], c["rot"]["dims"],
                c["rot"]["base"], "half", c["decay"])
            assert pools[i] == ("state",) and extra[i] is None
            assert shapes[i] == (c["heads"], c["dim"], c["vdim"], 0, 0)
        else:
            assert (m.kind, m.heads, m.state, m.vdim, m.decay_rank) == (
                "wkv", c["heads"], c["dim"], c["dim"], 3)
            assert pools[i] == ("state",) and extra[i] is None
        f = ent.get("mlp")
        if f is None:
            assert ls.mlp is None
        else:
            assert (ls.mlp.kind, ls.mlp.ff, ls.mlp.experts, ls.mlp.top,
                    ls.mlp.shared_ff, ls.mlp.act, ls.mlp.gated, ls.mlp.renorm,
                    ls.mlp.route_bias, ls.mlp.shared_gated) == (
                "moe", f["expert"]["ff"], f["router"]["experts"],
                f["router"]["top"], f["shared"]["ff"], "silu", True, True,
                True, True)
    assert spec.shifted_runs() == [e["type"] == "wkv" for e in cfg["layers"]]
    # fp32 states and normalisers, a previous row per wkv run
    n = sum(4 * s[0] * s[1] * s[2] for s in shapes)
    n += sum(4 * e[0] * e[1] for e in extra if e)
    assert spec.state_bytes_per_slot(2) == n + 2 * cfg["width"] * sum(
        spec.shifted_runs())


def test_weight_count_matches_the_checkpoint(model):
    cfg, w, d = model
    n = sum(t.numel() for t in w.values())
    assert ModelSpec.from_dir(d).weight_bytes(2) == 2 * n


def test_bad_configurations_are_refused():
    ret, par, wkv = (oracle.retention_layer, oracle.parallel_layer,
                     oracle.wkv_layer)
    bad = [
        [par(heads=3, kv_heads=2)], [par(rot_dims=8, dim=6)],
        [par(rot_dims=3)], [par(size=0)], [par(cap=0.0)],
        [ret(decay=[0.5])], [ret(rot_dims=10, dim=8)], [ret(rot_dims=5)],
        [wkv(mlp=oracle.moe(3, 4))], [wkv(mlp=oracle.moe(3, 0))],
        # shared weights: no such layer, itself, a circle, other sizes
        [dict(wkv(), weights_of=4)], [dict(wkv(), weights_of=0)],
        [dict(wkv(), weights_of=1), dict(wkv(), weights_of=0)],
        [wkv(), dict(wkv(heads=3), weights_of=0)],
        [wkv(), dict(wkv(mlp=None), weights_of=0)],
    ]
    for layers in bad:
        with pytest.raises(ValueError):
            ModelSpec.from_hf_config(oracle.make_config(layers=layers))
    with pytest.raises(ValueError):
        ModelSpec.from_hf_config(oracle.make_config(streams=0))
    for key, where in (("type", ()), ("kind", ("mlp",))):
        cfg = oracle.make_config(layers=[oracle.wkv_layer()])
        at = cfg["layers"][0]
        for k in where:
            at = at[k]
        at[key] = "other"
        with pytest.raises(NotImplementedError):
            ModelSpec.from_hf_config(cfg)


def test_checkpoints_that_do_not_fit_are_refused(tmp_path):
    cfg = oracle.make_config(layers=[oracle.wkv_layer()])
    w = oracle.make_weights(cfg)
    lost = {k: v for k, v in w.items() if k != "l0.mix.mu.g"}
    with pytest.raises(KeyError):
        make_engine(oracle.save_model(tmp_path / "a", cfg, lost))
    wrong = dict(w, **{"l0.mix.w2": w["l0.mix.w2"][:, 1:]})
    with pytest.raises(ValueError):
        make_engine(oracle.save_model(tmp_path / "b", cfg, wrong))


def test_state_models_refuse_prefix_caching_and_speculation(model):
    _, _, d = model
    with pytest.raises(ValueError):
        make_engine(d, enable_prefix_caching=True)
    with pytest.raises(ValueError):
        make_engine(d, speculative={"method": "ngram", "num_draft_tokens": 2})


def test_registry(model):
    from gpustack_amd.models import model_class_for
    from gpustack_amd.utils import model_registry as mr

    assert model_class_for("Sapatar").__name__ == "SapatarForCausalLM"
    assert mr.categories_for_architecture("Sapatar") == ["llm"]


def test_random_weights_keep_the_streams_in_range():
    from gpustack_amd.bench.layer_bench import _engine, sapatar_spec

    spec = sapatar_spec(dict(width=64, heads=2, ff=48, experts=4, eff=16,
                             layers=8))
    eng = _engine(spec, "cpu", 2, 64)
    toks = torch.randint(0, spec.vocab_size, (20,),
                         generator=torch.Generator().manual_seed(0)).tolist()
    out = eng.replay_step([("a", toks, [0, 19])], ["a"])
    assert out.shape == (2, spec.vocab_size) and bool(torch.isfinite(out).all())
    assert 0.2 < float(out.float().std()) < 5.0


# ---- each mechanism alone -----------------------------------------------------

def test_several_shifts_alone():
    """Two new sequences and one that goes on, slots out of order."""
    g = torch.Generator().manual_seed(1)
    W = 9
    mu = torch.rand(3, W, generator=g) * 2 - 0.5
    a, b, c = (torch.randn(n, W, generator=g) for n in (5, 7, 1))
    state = torch.randn(4, W, generator=g)            # junk to be ignored
    h = torch.cat([a, b[:4], c])
    hs = torch.zeros(3, *h.shape)
    ops.token_shift(hs, h, mu, state, i32([0, 5, 9]), i32([5, 4, 1]),
                    i32([3, 0, 2]), i32([0] * 5 + [1] * 4 + [2]),
                    i32([0, 1, 2, 3, 4, 0, 1, 2, 3, 0]))
    hs2 = torch.zeros(3, 3, W)
    ops.token_shift(hs2, b[4:], mu, state, i32([0]), i32([3]), i32([0]),
                    i32([0, 0, 0]), i32([4, 5, 6]))
    for j in range(3):
        ref = [oracle.shifted(t.double(), mu[j]) for t in (a, b, c)]
        assert (hs[j].double() - torch.cat([ref[0], ref[1][:4], ref[2]])
                ).abs().max() < 1e-6
        assert (hs2[j].double() - ref[1][4:]).abs().max() < 1e-6


def _scan(make, T, H, N, P, cuts):
    """A sequence through ops.memory_scan in portions, beside a second one
    in the same batch that starts anew each time; `make(T)` gives (operands,
    keyword operands per row, constants)."""
    g = torch.Generator().manual_seed(T + N)
    (q, k, v), rows, const = make(T, g)
    (q2, k2, v2), rows2, _ = make(3, g)
    state = torch.randn(4, H, N, P, generator=g)      # junk to be ignored
    extra = torch.randn(4, H, N + 1, generator=g)
    out, den, at = [], [], 0
    for n in cuts:
        cat = lambda a, b: torch.cat([b, a[at:at + n]])
        y, rden = torch.zeros(3 + n, H * P), torch.zeros(3 + n, H)
        ops.memory_scan(
            y, cat(q, q2), cat(k, k2), cat(v, v2), state, i32([0, 3]),
            i32([3, n]), i32([2, 1]), i32([0, 1, 2, *range(at, at + n)]),
            rden=rden, extra=extra,
            **{nm: cat(rows[nm], rows2[nm]) for nm in rows}, **const)
        out.append(y[3:])
        den.append(rden[3:])
        at += n
    assert at == T
    return (q, k, v), rows, torch.cat(out).double(), torch.cat(den).double()


CUTS = [[30], [1] * 30, [2, 3, 1, 17, 1, 6]]


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("rot", [0, 2, 3])
def test_retention_alone(cuts, rot):
    H, N, P = 3, 6, 5
    decay = [0.5, 0.97, 0.9995]
    f = [40.0 ** (-2.0 * i / (2 * rot)) for i in range(rot)] if rot else []

    def make(T, g):
        R = lambda c: torch.randn(T, c, generator=g)
        return (R(H * N), R(H * N), R(H * P)), {}, dict(
            decay=torch.tensor(decay), k_scale=0.3, inv_freq=torch.tensor(f))

    (q, k, v), _, y, _ = _scan(make, 30, H, N, P, cuts)
    q, k, v = (oracle.heads_of(t.double(), H) for t in (q, k, v))
    if rot:
        q, k = oracle.rotate(q, 40.0, 2 * rot), oracle.rotate(k, 40.0, 2 * rot)
    ref = [oracle.retention_recurrence(q[a], k[a] * 0.3, v[a], decay[a])
           for a in range(H)]
    assert (y - torch.cat(ref, -1)).abs().max() < 2e-5


@pytest.mark.parametrize("cuts", CUTS)
def test_wkv_alone(cuts):
    H, N = 2, 7
    g0 = torch.Generator().manual_seed(0)
    w0, u = torch.randn(H * N, generator=g0) - 1, torch.randn(H, N, generator=g0)

    def make(T, g):
        R = lambda: torch.randn(T, H * N, generator=g)
        return (R(), R(), R()), {"chan": R()}, dict(w0=w0, bonus=u)

    (q, k, v), rows, y, _ = _scan(make, 30, H, N, N, cuts)
    dec = torch.exp(-torch.exp(rows["chan"].double() + w0.double()))
    q, k, v, dec = (oracle.heads_of(t.double(), H) for t in (q, k, v, dec))
    ref = [oracle.wkv_recurrence(q[a], k[a], v[a], dec[a], u[a])
           for a in range(H)]
    assert (y - torch.cat(ref, -1)).abs().max() < 2e-5


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("cap", [0.7, 6.0])
@pytest.mark.parametrize("lift", [-4.0, 0.0, 4.0])
def test_mlstm_alone(cuts, cap, lift):
    """Input gates far below, around and far above the starting maximum."""
    H, N, P = 2, 5, 6
    g0 = torch.Generator().manual_seed(0)
    ib, fb = torch.randn(H, generator=g0) + lift, torch.randn(H, generator=g0) + 1

    def make(T, g):
        R = lambda c: torch.randn(T, c, generator=g)
        return (R(H * N), R(H * N), R(H * P)), {"gates": R(2 * H) * 3}, dict(
            q_scale=0.4, i_b=ib, f_b=fb, cap=cap)

    (q, k, v), rows, y, den = _scan(make, 30, H, N, P, cuts)
    z = rows["gates"].double()
    i = oracle.capped(z[:, :H] + ib.double(), cap)
    f = oracle.log_sigmoid(oracle.capped(z[:, H:] + fb.double(), cap))
    q, k, v = (oracle.heads_of(t.double(), H) for t in (q, k, v))
    ref = [oracle.mlstm_recurrence(q[a] * 0.4, k[a], v[a], i[:, a], f[:, a])
           for a in range(H)]
    y = (y.view(30, H, P) * den[:, :, None]).view(30, H * P)
    ref = torch.cat(ref, -1)
    assert (y - ref).abs().max() < 1e-4 * max(1.0, float(ref.abs().max()))


@pytest.mark.parametrize("mode", [0, 2])
def test_head_norm_with_a_row_factor_alone(mode):
    """Dividing the parts first matters: eps is inside the root."""
    g = torch.Generator().manual_seed(mode)
    T, H, P, eps = 4, 3, 5, 0.3
    y, gate = torch.randn(T, H * P, generator=g), torch.randn(T, H * P, generator=g)
    w, sc = torch.randn(H * P, generator=g), torch.rand(T, H, generator=g) + 0.1
    out = torch.zeros(T, H * P)
    ops.gated_group_norm(out, y, gate, w, H, eps, mode, sc)
    u = oracle.rms_unit(y.double().view(T, H, P) * sc.double()[:, :, None], eps)
    gt = torch.sigmoid(gate.double()) if mode == 0 else oracle.silu(gate.double())
    assert (out.double() - u.view(T, -1) * w.double() * gt).abs().max() < 1e-5


@pytest.mark.parametrize("window", [1, 2, 5, 100])
def test_windowed_attention_alone(window):
    g = torch.Generator().manual_seed(window)
    T, H, G, D, V, BS = 23, 4, 2, 6, 5, 4
    q = torch.randn(T, H, D, generator=g)
    k, v = torch.randn(T, G, D, generator=g), torch.randn(T, G, V, generator=g)
    bt = torch.randperm(8, generator=g)[:6].to(torch.int32)[None]
    kc, vc = torch.zeros(8, G, BS, D), torch.zeros(8, G, V, BS)
    t = torch.arange(T)
    kc[bt[0, t // BS].long(), :, t % BS] = k
    vc[bt[0, t // BS].long(), :, :, t % BS] = v
    out = torch.zeros(T, H, V)
    ops.paged_attention(out, q, kc, vc, bt, torch.zeros(T, dtype=torch.int32),
                        t.to(torch.int32), 0.7, window=window)
    for a in range(H):
        ref = oracle.attend(q[:, a].double(), k[:, a // 2].double(),
                            v[:, a // 2].double(), 0.7, window)
        assert (out[:, a].double() - ref).abs().max() < 1e-5


@pytest.mark.parametrize("experts,top", [(1, 1), (6, 1), (6, 3), (5, 5)])
def test_router_alone(experts, top):
    """Softmax over the chosen logits; the bias counts for choice and
    weight."""
    g = torch.Generator().manual_seed(top)
    T, W = 9, 8
    h = torch.randn(T, W, generator=g)
    w = {"router": torch.randn(experts, W, generator=g),
         "router.b": torch.randn(experts, generator=g)}
    idx, wt = oracle.route(h.double(), w, "", top)
    ex = torch.zeros(T, top, dtype=torch.int32)
    got = torch.zeros(T, top)
    ops.route_topk(ex, got, torch.nn.functional.linear(h, w["router"],
                                                       w["router.b"]),
                   None, experts, 1, 1, 1, False, True, 1.0)
    assert torch.equal(ex.long(), idx)
    assert (got.double() - wt).abs().max() < 1e-6


@pytest.mark.parametrize("layers", [
    [oracle.retention_layer(mlp=None)], [oracle.retention_layer()],
    [oracle.parallel_layer(mlp=None)], [oracle.parallel_layer()],
    [oracle.wkv_layer(mlp=None)], [oracle.wkv_layer()],
])
def test_one_layer(tmp_path, layers):
    assert _one(tmp_path, layers) < TOL


@pytest.mark.parametrize("left,right", [(1.0, 0.0), (0.0, 1.0), (1.7, -0.6)])
def test_parallel_scales(tmp_path, left, right):
    assert _one(tmp_path, [oracle.parallel_layer(
        left_scale=left, right_scale=right)]) < TOL


def test_projection_biases_and_the_router_bias_count(tmp_path):
    cfg = oracle.make_config(layers=[oracle.parallel_layer()])
    w = oracle.make_weights(cfg, seed=2)
    toks = tokens_for(cfg, 30, 2)
    ref = oracle.forward(cfg, w, toks)
    d = oracle.save_model(tmp_path, cfg, w)
    assert err(replay(make_engine(d), {"a": toks}, [[("a", 30)]])["a"], ref) < TOL
    for nm in ("mix.left.q.b", "mix.left.k.b", "mix.left.v.b", "mix.right.i.b",
               "mix.right.f.b", "mlp.router.b"):
        z = dict(w, **{"l0." + nm: torch.zeros_like(w["l0." + nm])})
        assert err(oracle.forward(cfg, z, toks), ref) > 0.01, nm


def test_denominator_has_a_floor(tmp_path):
    """Input gates far below 0: the first rows' normalisers are small, and
    without the bound the heads would come out at full size (eps keeps the
    norm behind from hiding it)."""
    cfg = oracle.make_config(layers=[oracle.parallel_layer(
        left_scale=0.0, mlp=None)], eps=0.01)
    w = oracle.make_weights(cfg, seed=4)
    w["l0.mix.right.i.b"] = torch.full((2,), -3.0, dtype=torch.bfloat16)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, 20, 4)
    ref = oracle.forward(cfg, w, toks)
    for steps in ([[("a", 20)]], [[("a", 1)]] * 20):
        got = replay(make_engine(d), {"a": toks}, steps)["a"]
        assert err(got, ref) < TOL
    bad = copy.deepcopy(cfg)
    bad["layers"][0]["mixer"]["right"]["no_floor"] = True
    assert err(oracle.forward(bad, w, toks)[:3], ref[:3]) > 0.02


def test_streams_mix_from_to_and_first_layer_sees_equal_streams(tmp_path):
    """A mixing matrix far from symmetric: transposing it changes the
    logits; so does forgetting that the update uses the old streams."""
    layers = [oracle.wkv_layer(), oracle.retention_layer()]
    cfg = oracle.make_config(layers=layers)
    w = oracle.make_weights(cfg, seed=6)
    for q in ("l0.hc1", "l0.hc2", "l1.hc1", "l1.hc2"):
        w[q + ".mix"] = torch.tensor([[0.5, 1.5, -0.5], [0.0, 0.25, 1.0],
                                      [-1.0, 0.0, 0.75]], dtype=torch.bfloat16)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, 20, 1)
    ref = oracle.forward(cfg, w, toks)
    assert err(replay(make_engine(d), {"a": toks}, [[("a", 20)]])["a"], ref) < TOL
    turned = {k: v.t() if k.endswith("hc1.mix") or k.endswith("hc2.mix") else v
              for k, v in w.items()}
    assert err(oracle.forward(cfg, turned, toks), ref) > 0.05


def test_strong_shifts_and_decays(tmp_path):
    """Shifts past 1 and below 0; decays from nearly everything to nearly
    nothing."""
    def change(w):
        g = torch.Generator().manual_seed(0)
        for k, v in w.items():
            if ".mu." in k:
                w[k] = (torch.randn(v.shape, generator=g) * 1.5).bfloat16()
            if k.endswith("w0"):
                w[k] = (torch.randn(v.shape, generator=g) * 5 - 2).bfloat16()

    assert _one(tmp_path, None, n=30, change=change,
                steps=[[("a", 9)]] + [[("a", 1)]] * 4 + [[("a", 17)]]) < TOL


def test_layers_that_share_weights_have_states_of_their_own(tmp_path):
    """Four runs of one layer of each kind (an owner in front, one behind
    its users), against the same model with the weights written out."""
    layers = [dict(oracle.wkv_layer(), weights_of=4), oracle.parallel_layer(),
              oracle.retention_layer()]
    layers += [oracle.again(layers, 1), oracle.wkv_layer(),
               oracle.again(layers, 2)]
    layers += [dict(layers[0]), oracle.again(layers, 3)]
    cfg = oracle.make_config(layers=layers)
    w = oracle.make_weights(cfg, seed=5)
    d = oracle.save_model(tmp_path / "s", cfg, w)
    toks = tokens_for(cfg, 33, 5)
    steps = [[("a", 14)], [("a", 2)], [("a", 12)]] + [[("a", 1)]] * 5
    eng = make_engine(d)
    got = replay(eng, {"a": toks}, steps)["a"]
    assert err(got, oracle.forward(cfg, w, toks)) < TOL
    model = eng.runner.model
    assert model.layers[0] is model.layers[4] is model.layers[6]
    assert model.layers[7] is model.layers[3] is model.layers[1]
    flat = copy.deepcopy(cfg)
    wide = dict(w)
    for i, ent in enumerate(flat["layers"]):
        o = oracle.owner(cfg, i)
        ent.pop("weights_of", None)
        wide.update({f"l{i}." + k.split(".", 1)[1]: v.clone() for k, v in w.items()
                     if k.startswith(f"l{o}.")})
    assert len(wide) > len(w)
    d2 = oracle.save_model(tmp_path / "f", flat, wide)
    assert err(replay(make_engine(d2), {"a": toks}, steps)["a"], got) < 1e-6


@pytest.mark.parametrize("streams,width,rank,layers", [
    # one stream, one head, heads of one channel, a window of one, no
    # rotation, one expert, no feed-forward
    (1, 10, 1, [
        oracle.retention_layer(heads=1, dim=1, vdim=3, rot_dims=0,
                               mlp=oracle.moe(1, 1, 3, 5)),
        oracle.wkv_layer(heads=1, dim=1, mlp=None),
        oracle.parallel_layer(heads=1, kv_heads=1, dim=2, vdim=7, size=1,
                              rot_dims=0, r_heads=1, r_dim=1, r_vdim=1,
                              cap=20.0, mlp=None)]),
    # kv heads == heads, equal sizes, full rotation, every expert chosen
    (2, 18, 5, [
        oracle.parallel_layer(heads=2, kv_heads=2, dim=6, vdim=6, size=16,
                              rot_dims=6, r_heads=2, r_dim=6, r_vdim=6,
                              left_scale=1.0, right_scale=1.0,
                              mlp=oracle.moe(3, 3, 9, 9)),
        oracle.retention_layer(heads=2, dim=6, vdim=6, rot_dims=6,
                               decay=[1.0, 0.25]),
        oracle.wkv_layer(heads=3, dim=6)]),
    # a window wider than the sequence, more streams, many heads
    (7, 13, 2, [
        oracle.wkv_layer(heads=5, dim=4),
        oracle.parallel_layer(heads=18, kv_heads=1, dim=3, vdim=2, size=500,
                              rot_dims=2, r_heads=5, r_dim=9, r_vdim=4),
        oracle.retention_layer(heads=7, dim=4, vdim=11, rot_dims=2,
                               mlp=None)]),
])
def test_other_sizes(tmp_path, streams, width, rank, layers):
    steps = [[("a", 11)], [("a", 2)], [("a", 19)]] + [[("a", 1)]] * 5
    assert _one(tmp_path, layers, n=37, width=width, streams=streams,
                rank=rank, steps=steps) < TOL


def test_other_constants(tmp_path):
    """eps large enough to matter, in the norms of the heads as well."""
    assert _one(tmp_path, None, n=25, seed=8, eps=0.05) < TOL
    cfg = oracle.make_config(eps=0.05)
    w = oracle.make_weights(cfg, seed=8)
    toks = tokens_for(cfg, 25, 3)
    other = dict(cfg, norm={"eps": 1e-5})
    assert err(oracle.forward(other, w, toks), oracle.forward(cfg, w, toks)) > 0.01


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
    assert err(single, whole) < 2e-5 and err(late, whole) < 2e-5


@pytest.mark.parametrize("sizes", [[2] * 20, [16, 16, 8], [15, 2, 17, 1, 5],
                                   [1, 2, 3, 31, 3], [33, 7], [9, 31]])
def test_portions(model, sizes):
    """Portions cut inside pages and windows."""
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
        assert err(got[r], alone) < 2e-5, r


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


def test_long_decoding_across_pages_and_windows(model):
    cfg, w, d = model
    toks = tokens_for(cfg, 5 + 140, 13)
    got = replay(make_engine(d), {"a": toks},
                 [[("a", 5)]] + [[("a", 1)]] * 140)["a"]
    assert err(got, oracle.forward(cfg, w, toks)) < TOL


def test_interrupted_requests_keep_their_rows(model):
    """A request that is left out of some steps goes on from its own slot."""
    cfg, w, d = model
    prompts = {"a": tokens_for(cfg, 25, 31), "b": tokens_for(cfg, 25, 32)}
    schedule = [[("a", 7)], [("b", 9)], [("b", 1)], [("b", 1)], [("a", 1)],
                [("b", 2)], [("a", 2), ("b", 1)], [("a", 15)], [("b", 11)]]
    got = replay(make_engine(d), prompts, schedule)
    for r, toks in prompts.items():
        assert err(got[r], oracle.forward(cfg, w, toks)) < TOL, r


def test_a_stack_without_attention(tmp_path):
    """Nothing per token is cached: only the state slots carry a request."""
    layers = [oracle.wkv_layer(), oracle.retention_layer()]
    steps = [[("a", 12)], [("a", 2)]] + [[("a", 1)]] * 6
    assert _one(tmp_path, layers, n=20, steps=steps) < TOL
    # blocks without bytes are counted by what sequences can name, however
    # much memory there is
    eng = make_engine(str(tmp_path))
    n = type(eng.runner.kv).compute_num_blocks(eng.cfg, 1 << 40)
    assert n == 4 * (4096 // eng.cfg.block_size) + 1


def test_bf16_engine_is_close(model):
    cfg, w, d = model
    toks = tokens_for(cfg, 40, 5)
    eng = make_engine(d, dtype="bfloat16")
    got = replay(eng, {"a": toks}, [[("a", 23)], [("a", 16)], [("a", 1)]])["a"]
    ref = oracle.forward(cfg, w, toks)
    # a close call of a router may send a row elsewhere
    e = torch.tensor([err(got[t:t + 1], ref[t:t + 1]) for t in range(40)])
    assert float((e > 0.15).double().mean()) <= 0.1


# ---- faults that random weights would hide ------------------------------------------

@functools.lru_cache(maxsize=None)
def standout_tokens():
    """(one-layer configuration, weights, far token, last token) such that,
    behind a prompt of filler token 0, the LAST token's scores single out the
    far token: of a few last tokens and all far ones the pair whose presence
    changes the last row most (a search with the oracle that sees every key).
    The score scale is large, so the softmax is nearly one-hot: losing that
    key, or wrongly admitting it, changes the row wholly. Nothing is rotated
    and the memory beside is silent, so a key depends on its own token only,
    wherever it stands."""
    L = oracle.parallel_layer(heads=2, kv_heads=2, dim=8, vdim=6,
                              size=10 ** 6, scale=4.0, rot_dims=0,
                              right_scale=0.0, mlp=None)
    cfg = oracle.make_config(width=16, vocab=40, layers=[L])
    w = oracle.make_weights(cfg, seed=9)
    best, pair = -1.0, None
    for last in (39, 38, 37):
        base = oracle.forward(cfg, w, [0] * 23 + [last])[-1:]
        for t in range(1, 37):
            e = err(oracle.forward(cfg, w, [0] * 11 + [t] + [0] * 11 + [last])
                    [-1:], base)
            if e > best:
                best, pair = e, (t, last)
    return cfg, w, *pair


def standout_model(tmp_path, far_pos, n, window):
    cfg, w, far, last = standout_tokens()
    cfg = copy.deepcopy(cfg)
    cfg["layers"][0]["mixer"]["left"]["mask"]["size"] = window
    toks = [0] * n
    toks[far_pos] = far
    toks[-1] = last
    return cfg, w, oracle.save_model(tmp_path, cfg, w), toks


@pytest.mark.parametrize("far_pos", [0, 15, 16, 31, 200])
@pytest.mark.parametrize("decode", [False, True])
def test_far_key_among_hundreds(tmp_path, far_pos, decode):
    cfg, w, d, toks = standout_model(tmp_path, far_pos, 300, 300)
    ref = oracle.forward(cfg, w, toks)[-1:]
    other = list(toks)
    other[far_pos] = 0
    assert err(oracle.forward(cfg, w, other)[-1:], ref) > 0.05
    n = len(toks)
    steps = [[("a", n - 1)], [("a", 1)]] if decode else [[("a", n)]]
    got = replay(make_engine(d), {"a": toks}, steps)["a"][-1:]
    assert err(got, ref) < TOL


# the last row, 82, sees keys from 83 - window on: inside and outside of a
# window that starts within a page, on a page border (80, 64) and one before
@pytest.mark.parametrize("window,far_pos,seen", [
    (7, 75, False), (7, 76, True), (3, 79, False), (3, 80, True),
    (19, 63, False), (19, 64, True), (20, 63, True), (82, 0, False),
    (83, 0, True), (2, 80, False), (2, 81, True), (1, 81, False)])
@pytest.mark.parametrize("steps", [
    [[("a", 83)]], [[("a", 40)], [("a", 43)]], [[("a", 76)], [("a", 7)]],
    [[("a", 75)], [("a", 2)], [("a", 6)]], [[("a", 82)], [("a", 1)]],
    [[("a", 70)]] + [[("a", 1)]] * 13])
def test_window_edge(tmp_path, window, far_pos, seen, steps):
    cfg, w, d, toks = standout_model(tmp_path, far_pos, 83, window)
    ref = oracle.forward(cfg, w, toks)[-1:]
    got = replay(make_engine(d), {"a": toks}, steps)["a"][-1:]
    assert err(got, ref) < TOL
    # the key decides the row exactly if it is inside
    other = list(toks)
    other[far_pos] = 0
    moved = err(oracle.forward(cfg, w, other)[-1:], ref)
    assert moved > 0.05 if seen else moved < 1e-9
    # and an edge one position off would show
    bad = copy.deepcopy(cfg)
    bad["layers"][0]["mixer"]["left"]["mask"]["misplaced"] = -1 if seen else 1
    edge = far_pos == 83 - window if seen else far_pos == 82 - window
    if edge:
        assert err(oracle.forward(bad, w, toks)[-1:], ref) > 0.05


@pytest.mark.parametrize("kind", ["retention", "wkv", "mlstm"])
def test_state_carries_the_first_token_to_the_last_row(tmp_path, kind):
    """Memories that hardly forget: the first token still shapes the last
    row, through a prompt cut into portions and decoded tokens."""
    L = {"retention": lambda: oracle.retention_layer(
            decay=[0.999, 0.9995, 1.0], mlp=None),
         "wkv": lambda: oracle.wkv_layer(mlp=None),
         "mlstm": lambda: oracle.parallel_layer(size=1, mlp=None)}[kind]()
    cfg = oracle.make_config(width=16, layers=[L])
    w = oracle.make_weights(cfg, seed=4)
    if kind == "wkv":
        w["l0.mix.w0"] = torch.full((14,), -7.0, dtype=torch.bfloat16)
    if kind == "mlstm":
        w["l0.mix.right.f.b"] = torch.full((2,), 9.0, dtype=torch.bfloat16)
    d = oracle.save_model(tmp_path, cfg, w)
    toks = tokens_for(cfg, 60, 8)
    ref = oracle.forward(cfg, w, toks)
    other = [(toks[0] + 1) % cfg["vocab"]] + toks[1:]
    assert err(oracle.forward(cfg, w, other)[-1:], ref[-1:]) > 1e-3
    steps = [[("a", 3)], [("a", 20)], [("a", 2)], [("a", 20)]] + [[("a", 1)]] * 15
    got = replay(make_engine(d), {"a": toks}, steps)["a"]
    assert err(got, ref) < 5e-5


def test_shift_across_portion_starts(tmp_path):
    """Every portion's first row reads the previous step's last row."""
    layers = [oracle.wkv_layer(mlp=None), oracle.wkv_layer(heads=1, dim=5)]
    steps = [[("a", 1)], [("a", 2)], [("a", 1)], [("a", 3)], [("a", 2)],
             [("a", 12)], [("a", 1)], [("a", 1)], [("a", 4)]]

    def change(w):
        for k in w:
            if ".mu." in k:
                w[k] = torch.full((22,), 0.9, dtype=torch.bfloat16)

    assert _one(tmp_path, layers, n=27, steps=steps, change=change) < TOL


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
