"""The HIP kernels added for the Sapatar mechanisms against their fp32 torch
references (gpustack_amd/ops/torch_ref.py): matrix memories with constant,
per-channel and gated decay (prompt scan and decode step), rotation tables,
several token shifts of one row, gated grouped experts, expert sums in bf16,
tanh rows."""
import pytest
import torch

from gpustack_amd import ops
from gpustack_amd.ops import torch_ref
from test_fuvuvik_ops_gpu import close, ragged

pytestmark = pytest.mark.gpu

DT = [torch.float32, torch.bfloat16]

# heads, state rows, value channels: sizes the 16-byte staging takes and sizes
# no vector path divides; every lane split; more channels than a workgroup
SIZES = [(2, 32, 32), (3, 64, 64), (2, 48, 96), (1, 128, 128), (2, 256, 40),
         (1, 512, 24), (5, 7, 9), (2, 100, 33), (3, 20, 6), (1, 1, 1),
         (1, 16, 300)]


def operands(kind, H, N, P, T, dtype, seed, pad=8):
    """Operands of a mode: columns of one wide product where they share a
    row in the model, and the keyword arguments of the op."""
    g = torch.Generator().manual_seed(seed)
    R = lambda *s, k=1.0: torch.randn(*s, generator=g) * k
    n, v = H * N, H * P
    wide = R(T, 2 * n + v + 2 * H + pad).to(dtype)
    kw = {}
    if kind == "const":
        kw = dict(k_scale=N ** -0.5, decay=1.0 - 2.0 ** -(1 + 3 * torch.rand(
            H, generator=g)))
    elif kind == "rot":
        half = N // 2 - (N // 8 if N % 16 else 0)
        kw = dict(k_scale=N ** -0.5, decay=torch.full((H,), 0.97),
                  inv_freq=300.0 ** (-torch.arange(half) / half))
    elif kind == "chan":
        kw = dict(chan=(R(T, n) * 0.7).to(dtype), w0=R(n) - 1.0, bonus=R(n))
    else:
        kw = dict(q_scale=N ** -0.5, i_b=R(H) + 1.0, f_b=R(H) + 2.0, cap=5.0)
        wide[:, 2 * n + v:2 * n + v + 2 * H] *= 3
    return wide, kw


def split(wide, H, N, P, kind):
    n, v = H * N, H * P
    q, k, x = wide[:, :n], wide[:, n:2 * n], wide[:, 2 * n:2 * n + v]
    gates = {"gates": wide[:, 2 * n + v:2 * n + v + 2 * H]} \
        if kind == "gated" else {}
    return q, k, x, gates


def to_gpu(kw):
    return {k: v.cuda() if torch.is_tensor(v) else v for k, v in kw.items()}


def run_both(kind, H, N, P, dtype, news, hists, slots, single=False, seed=0):
    T = sum(news)
    wide, kw = operands(kind, H, N, P, T, dtype, seed + N * P)
    g = torch.Generator().manual_seed(seed + 5)
    state = torch.randn(7, H, N, P, generator=g)
    extra = torch.cat([torch.randn(7, H, N, generator=g),
                       torch.rand(7, H, 1, generator=g)], -1) \
        if kind == "gated" else None
    sf, sr, ss, rs, ps = ragged(news, hists, slots)
    ref, rd_r = torch.zeros(T, H * P), torch.zeros(T, H)
    st_r = state.clone()
    ex_r = extra.clone() if extra is not None else None
    q, k, v, gt = split(wide, H, N, P, kind)
    torch_ref.memory_scan(ref, q, k, v, st_r, sf, sr, ss, ps, extra=ex_r,
                          rden=rd_r, **gt, **kw)
    wg, kg = wide.cuda(), to_gpu(kw)
    q, k, v, gt = split(wg, H, N, P, kind)
    st_g = state.cuda()
    ex_g = extra.cuda() if extra is not None else None
    got = torch.zeros(T, H * P, device="cuda")
    rden = torch.zeros(T, H, device="cuda")
    psg = ps.cuda()
    if kind == "rot" and not single:
        kg["rot"] = ops.rope_table(psg, kg["inv_freq"])
    ops.memory_scan(got, q, k, v, st_g, sf.cuda(), sr.cuda(), ss.cuda(), psg,
                    extra=ex_g, rden=rden, single=single, **gt, **kg)
    what = f"{kind} {H} {N} {P} {dtype}"
    close(got, ref, torch.float32, what, tol=5e-5)
    close(st_g, st_r, torch.float32, what + " state", tol=5e-5)
    if extra is not None:
        close(ex_g, ex_r, torch.float32, what + " extra", tol=5e-5)
        # a sum close to zero loses its digits to its terms
        close(1 / rden, 1 / rd_r, torch.float32, what + " den", tol=5e-5)
        # slots of nobody in the batch are untouched
    idle = [i for i in range(7) if i not in slots]
    assert torch.equal(st_g.cpu()[idle], state[idle])


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("kind", ["const", "rot", "chan", "gated"])
@pytest.mark.parametrize("size", SIZES)
def test_memory_scan_prompts(dtype, kind, size):
    """Unequal portions, some continuing, lengths around the staged passes."""
    run_both(kind, *size, dtype, [17, 1, 70, 2, 16], [0, 4, 900, 1, 0],
             [3, 0, 5, 1, 6])


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("kind", ["const", "rot", "chan", "gated"])
@pytest.mark.parametrize("size", SIZES)
def test_memory_step_rows(dtype, kind, size):
    run_both(kind, *size, dtype, [1] * 5, [0, 4, 900, 1, 0], [3, 0, 5, 1, 6],
             single=True)


@pytest.mark.parametrize("kind", ["const", "chan", "gated"])
def test_memory_step_walks_more_rows_too(kind):
    """The single-row kernel is only a hint's choice: a batch that brings
    more rows after all is walked row by row."""
    run_both(kind, 2, 64, 32, torch.bfloat16, [3, 1, 5], [0, 2, 0], [4, 2, 0],
             single=True)


def test_memory_scan_fills_the_chip():
    """Enough workgroups for the narrow lane split."""
    run_both("chan", 40, 64, 64, torch.bfloat16, [3] * 7, [0, 1, 2, 3, 0, 1, 5],
             list(range(7)))
    run_both("gated", 72, 96, 64, torch.bfloat16, [5] * 7,
             [0, 1, 2, 3, 0, 1, 5], list(range(7)))


def test_gates_in_one_pass_or_many():
    """The running maximum over passes of 64 rows is the sequential one,
    whatever the portions, with gates that move it up and down."""
    for n in (63, 64, 65, 129):
        run_both("gated", 2, 16, 8, torch.float32, [n, 2], [0, 7], [2, 4],
                 seed=n)


def test_rope_table_matches():
    g = torch.Generator().manual_seed(0)
    pos = torch.randint(0, 100000, (77,), generator=g).to(torch.int32)
    f = 1e4 ** (-torch.arange(24) / 24.0)
    t = ops.rope_table(pos.cuda(), f.cuda()).cpu()
    ang = pos.float()[:, None] * f[None, :]
    assert (t[:, 0] - torch.cos(ang)).abs().max() < 2e-6
    assert (t[:, 1] - torch.sin(ang)).abs().max() < 2e-6


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("W", [22, 64, 2052, 5000])
def test_several_shifts_of_one_row(dtype, W):
    g = torch.Generator().manual_seed(W)
    mu = torch.randn(5, W, generator=g)
    st = torch.randn(6, W, generator=g).to(dtype)
    for news, hists in (([5, 1, 70, 2], [0, 4, 17, 0]),
                        ([1, 1, 1, 1], [0, 4, 17, 1])):
        T = sum(news)
        sf, sr, ss, rs, ps = ragged(news, hists, [3, 0, 5, 1])
        h = torch.randn(T, W, generator=g).to(dtype)
        st_r, ref = st.clone(), torch.zeros(5, T, W, dtype=dtype)
        torch_ref.token_shift(ref, h, mu, st_r, sf, sr, ss, ps)
        st_g, got = st.cuda(), torch.zeros(5, T, W, dtype=dtype).cuda()
        ops.token_shift(got, h.cuda(), mu.cuda(), st_g, *(
            t.cuda() for t in (sf, sr, ss, rs, ps)))
        close(got, ref, dtype)
        assert torch.equal(st_g.cpu(), st_r)
    # single rows, inside the stream kernel
    x = torch.randn(T, 3, W, generator=g).cuda()
    rd, nw = torch.randn(3, generator=g).cuda(), torch.rand(W, generator=g).cuda()
    st1, st2 = st.cuda(), st.cuda()
    h1, h2 = (torch.zeros(T, W, dtype=dtype, device="cuda") for _ in range(2))
    hs1, hs2 = (torch.zeros(5, T, W, dtype=dtype, device="cuda")
                for _ in range(2))
    sf, sr, ss, rs, ps = (t.cuda() for t in (sf, sr, ss, rs, ps))
    ops.stream_step(x, None, None, None, None, None, rd, nw, 1e-5, h1,
                    shift=(hs1, mu.cuda(), st1, rs, ss, ps))
    ops.stream_step(x, None, None, None, None, None, rd, nw, 1e-5, h2)
    ops.token_shift(hs2, h2, mu.cuda(), st2, sf, sr, ss, rs, ps)
    assert torch.equal(h1, h2) and torch.equal(st1, st2)
    close(hs1, hs2, torch.float32, tol=1e-6 if dtype == torch.float32 else 1e-2)


@pytest.mark.parametrize("E,W,F_", [(3, 64, 64), (9, 192, 128)])
def test_grouped_gated_experts(E, W, F_):
    g = torch.Generator().manual_seed(E)
    T, top, bf = 13, 2, torch.bfloat16
    x = torch.randn(T, W, generator=g).to(bf)
    up = (torch.randn(E, 2 * F_, W, generator=g) / W ** 0.5).to(bf)
    ex = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)])
    flat = ex.reshape(-1)
    order = torch.argsort(flat, stable=True)
    counts = torch.bincount(flat, minlength=E).to(torch.int32)
    offs = (counts.cumsum(0) - counts).to(torch.int32)
    tok = (order // top).to(torch.int32)
    u = torch.zeros(T * top, F_, dtype=bf, device="cuda")
    ops.grouped_up_act(u, x.cuda(), up.cuda(), tok.cuda(), offs.cuda(),
                       counts.cuda(), "silu")
    z = torch.einsum("tw,tfw->tf", x[tok.long()].float(),
                     up[flat[order]].float())
    ref = torch.nn.functional.silu(z[:, :F_]) * z[:, F_:]
    close(u, ref, bf)


@pytest.mark.parametrize("W", [7, 64, 4104])
def test_expert_sums_in_bf16(W):
    g = torch.Generator().manual_seed(W)
    T, top, bf = 9, 3, torch.bfloat16
    y = torch.randn(T * top, W, generator=g).to(bf)
    inv = torch.randperm(T * top, generator=g).to(torch.int32).view(T, top)
    wt, sh = torch.rand(T, top, generator=g), torch.randn(T, W, generator=g).to(bf)
    gl = torch.randn(T, 5, generator=g)
    for shared, gate in ((sh, gl), (sh, None), (None, None)):
        ref = torch.zeros(T, W)
        torch_ref.moe_combine(ref, y, inv, wt, shared, gate, 4)
        out = torch.zeros(T, W, dtype=bf, device="cuda")
        ops.moe_combine(out, y.cuda(), inv.cuda(), wt.cuda(),
                        shared.cuda() if shared is not None else None,
                        gate.cuda() if gate is not None else None, 4)
        close(out, ref, bf)


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("n", [5, 64])
def test_tanh_rows(dtype, n):
    x = (torch.randn(6, n, generator=torch.Generator().manual_seed(n)) * 2
         ).to(dtype)
    got = x.cuda()
    ops.act_inplace(got, "tanh")
    close(got, torch.tanh(x.float()), dtype, tol=1e-2 if dtype != torch.float32
          else 1e-6)
