"""The HIP kernels added for the Fuvuvik mechanisms against their fp32 torch
references (gpustack_amd/ops/torch_ref.py): stream rows with gate and token
shift, token shift over portions, gated recurrence in runs, short convolution
without activation, unit heads, chunked paged attention with a constant sink
and head gates, strided gate/up rows."""
import pytest
import torch

from gpustack_amd import ops
from gpustack_amd.ops import torch_ref

pytestmark = pytest.mark.gpu

DT = [torch.float32, torch.bfloat16]
i32 = lambda v: torch.tensor(v, dtype=torch.int32)


def close(a, b, dtype, what="", tol=None):
    tol = tol or (2e-5 if dtype == torch.float32 else 2e-2)
    a, b = a.float().cpu(), b.float().cpu()
    scale = b.abs().max().clamp(min=1.0)
    assert (a - b).abs().max() / scale < tol, what


def ragged(news, hists, slots):
    """seq_first, seq_rows, slots, row_seq, positions of a batch."""
    first, rs, pos, at = [], [], [], 0
    for i, (n, h) in enumerate(zip(news, hists)):
        first.append(at)
        rs += [i] * n
        pos += list(range(h, h + n))
        at += n
    return i32(first), i32(news), i32(slots), i32(rs), i32(pos)


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 6, 9])
@pytest.mark.parametrize("W,T", [(22, 5), (64, 7), (1300, 3), (2052, 600),
                                 (5000, 4), (9000, 2)])
def test_stream_step(dtype, S, W, T):
    g = torch.Generator().manual_seed(S * W)
    x = torch.randn(T, S, W, generator=g)
    a = torch.randn(T, W, generator=g).to(dtype)
    wide = torch.randn(T, W + 8, generator=g).to(dtype)
    gb, nw = torch.randn(W, generator=g), torch.rand(W, generator=g) + 0.5
    mix = torch.randn(S, S, generator=g) / S ** 0.5
    b, rd = torch.randn(S, generator=g), torch.randn(S, generator=g)
    eps = 1e-5
    # gate rows of a wider product, at an aligned and an unaligned column
    for col in (8, 3):
        gate = wide[:, col:col + W]
        xr, hr = x.clone(), torch.zeros(T, W, dtype=dtype)
        torch_ref.stream_step(xr, a, gate, gb, mix, b, rd, nw, eps, hr)
        xg, hg = x.cuda(), torch.zeros(T, W, dtype=dtype, device="cuda")
        gg = wide.cuda()[:, col:col + W]
        ops.stream_step(xg, a.cuda(), gg, gb.cuda(), mix.cuda(), b.cuda(),
                        rd.cuda(), nw.cuda(), eps, hg)
        close(xg, xr, torch.float32, "streams")
        close(hg, hr, dtype, "h")
    # closing alone, without a gate
    xr = x.clone()
    torch_ref.stream_step(xr, a, None, None, mix, b, None, None, eps, None)
    xg = x.cuda()
    ops.stream_step(xg, a.cuda(), None, None, mix.cuda(), b.cuda(), None, None,
                    eps, None)
    close(xg, xr, torch.float32)
    # opening alone leaves the streams as they are
    hr = torch.zeros(T, W, dtype=dtype)
    torch_ref.stream_step(x.clone(), None, None, None, None, None, rd, nw, eps, hr)
    xg, hg = x.cuda(), torch.zeros(T, W, dtype=dtype, device="cuda")
    ops.stream_step(xg, None, None, None, None, None, rd.cuda(), nw.cuda(), eps,
                    hg)
    assert torch.equal(xg.cpu(), x)
    close(hg, hr, dtype)


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("W", [22, 64, 2052, 5000])
def test_stream_step_with_shift_equals_two_steps(dtype, W):
    """Single rows: the shift inside the row kernel gives what the shift
    kernel gives, and leaves the same row behind."""
    g = torch.Generator().manual_seed(W)
    T, S, eps = 5, 3, 1e-5
    x = torch.randn(T, S, W, generator=g).cuda()
    rd, nw = torch.randn(S, generator=g).cuda(), torch.rand(W, generator=g).cuda()
    mu = torch.randn(W, generator=g).cuda()
    state = torch.randn(8, W, generator=g).to(dtype).cuda()
    sf, sr, ss, rs, ps = (t.cuda() for t in ragged(
        [1] * T, [0, 3, 9, 0, 1], [6, 2, 0, 7, 4]))
    st2 = state.clone()
    h, hs, h2, hs2 = (torch.zeros(T, W, dtype=dtype, device="cuda")
                      for _ in range(4))
    ops.stream_step(x, None, None, None, None, None, rd, nw, eps, h,
                    shift=(hs, mu, state, rs, ss, ps))
    ops.stream_step(x, None, None, None, None, None, rd, nw, eps, h2)
    ops.token_shift(hs2, h2, mu, st2, sf, sr, ss, rs, ps)
    assert torch.equal(h, h2) and torch.equal(state, st2)
    close(hs, hs2, torch.float32, tol=1e-6 if dtype == torch.float32 else 1e-2)


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("W", [7, 64, 2056, 4100])
def test_token_shift(dtype, W):
    g = torch.Generator().manual_seed(W)
    meta = ragged([5, 1, 300, 2], [0, 4, 17, 0], [3, 0, 5, 1])
    T = 308
    h = torch.randn(T, W, generator=g).to(dtype)
    mu = torch.randn(W, generator=g)
    st = torch.randn(6, W, generator=g).to(dtype)
    st_r, ref = st.clone(), torch.zeros_like(h)
    sf, sr, ss, rs, ps = meta
    torch_ref.token_shift(ref, h, mu, st_r, sf, sr, ss, ps)
    st_g, got = st.cuda(), torch.zeros_like(h).cuda()
    ops.token_shift(got, h.cuda(), mu.cuda(), st_g, *(t.cuda() for t in
                                                      (sf, sr, ss, rs, ps)))
    close(got, ref, dtype)
    assert torch.equal(st_g.cpu(), st_r)


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("N,off", [(5, 1), (64, 0), (130, 2), (2048, 0)])
@pytest.mark.parametrize("size", [None, 3, 16, 64])
def test_gru_scan(dtype, N, off, size):
    """Runs of several sizes, unequal sequences, some continuing; the state
    a portion starts from is overwritten in the same launch."""
    g = torch.Generator().manual_seed(N)
    news = [65, 1, 130, 2, 16]
    T = sum(news)
    src = torch.randn(T, 3 * N + 2 * off + 6, generator=g).to(dtype)
    zb, ub = torch.randn(N, generator=g) - 1, torch.randn(N, generator=g)
    st = torch.randn(7, 1, 1, N, generator=g)
    sf, sr, ss, rs, ps = ragged(news, [0, 9, 31, 0, 64], [4, 0, 6, 2, 1])
    cols = (off, off + N, off + 2 * N)
    st_r, ref = st.clone(), torch.zeros(T, N, dtype=dtype)
    torch_ref.gru_scan(ref, src, *cols, zb, ub, st_r, sf, sr, ss, ps)
    st_g, got = st.cuda(), torch.zeros(T, N, dtype=dtype, device="cuda")
    runs = None
    if size is not None:
        first = sf.tolist()
        runs = ops.build_scan_chunks(first, news, size, "cuda")
    ops.gru_scan(got, src.cuda(), *cols, zb.cuda(), ub.cuda(), st_g,
                 *(t.cuda() for t in (sf, sr, ss, ps)), chunks=runs)
    close(got, ref, dtype)
    close(st_g, st_r, torch.float32)


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 9])
@pytest.mark.parametrize("C,col0,big", [(300, 17, 1), (304, 16, 1), (1024, 8, 8)])
@pytest.mark.parametrize("silu,bias", [(False, False), (True, True)])
def test_short_conv(dtype, taps, C, col0, big, silu, bias):
    g = torch.Generator().manual_seed(C + taps)
    w = torch.randn(C, taps, generator=g)
    b = torch.randn(C, generator=g) if bias else None
    st = torch.randn(6, taps - 1, C, generator=g).to(dtype)
    cases = [([5, 1, 150 * big, 2], [0, 1, 17, 0], [3, 0, 5, 1], False),
             ([1] * 6, [0, 1, 2, 8, 0, 3], [5, 0, 3, 1, 2, 4], True)]
    for news, hists, slots, single in cases:
        sf, sr, ss, rs, ps = ragged(news, hists, slots)
        T = sum(news)
        src = torch.randn(T, col0 + C + 8, generator=g).to(dtype)
        st_r, ref = st.clone(), torch.zeros(T, C, dtype=dtype)
        torch_ref.short_conv(ref, src, col0, w, b, st_r, sf, sr, ss, ps, silu)
        st_g, got = st.cuda(), torch.zeros(T, C, dtype=dtype, device="cuda")
        ops.short_conv(got, src.cuda(), col0, w.cuda(),
                       b.cuda() if bias else None, st_g,
                       *(t.cuda() for t in (sf, sr, ss, rs, ps)), silu=silu,
                       single=single)
        close(got, ref, dtype, f"single={single}")
        assert torch.equal(st_g.cpu(), st_r), f"single={single}"


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("H,G,d,dv,rd", [(3, 2, 10, 7, 6), (8, 2, 64, 48, 16),
                                         (4, 4, 128, 64, 128), (6, 3, 96, 32, 0),
                                         (5, 1, 32, 24, 32)])
def test_unit_heads(dtype, H, G, d, dv, rd):
    g = torch.Generator().manual_seed(d)
    T, BS, eps = 37, 16, 1e-5
    src = torch.randn(T, (H + G) * d + G * dv + 8, generator=g).to(dtype)
    invf = torch.rand(rd // 2, generator=g)
    pos = torch.randint(0, 3000, (T,), generator=g).to(torch.int32)
    slots = torch.randperm(5 * BS, generator=g)[:T]
    rot0 = 0 if rd else -1

    def run(dev):
        to = lambda t: t.to(dev)
        q = torch.zeros(T, H * d, dtype=dtype, device=dev)
        kc = torch.zeros(5, G, BS, d, dtype=dtype, device=dev)
        vc = torch.zeros(5, G, dv, BS, dtype=dtype, device=dev)
        fn = ops.head_rope_store if dev == "cuda" else torch_ref.head_rope_store
        fn(q, to(src), 0, H, d, None, d, rot0, H * d, G, d, None, d, rot0,
           (H + G) * d, to(invf), True, 1.0, to(pos), kc, vc, to(slots), eps)
        return q, kc, vc

    for a, b, nm in zip(run("cuda"), run("cpu"), "qkv"):
        close(a, b, dtype, nm)


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("exact", [False, True])
@pytest.mark.parametrize("D,VW,H,G", [(64, 48, 4, 2), (32, 16, 6, 1),
                                      (10, 7, 3, 3)])
@pytest.mark.parametrize("chunk", [0, 1, 19, 64, 600])
def test_paged_attention_chunks_sink_gates(dtype, exact, D, VW, H, G, chunk):
    """Prompt portions beside decode rows, long enough for the key split;
    chunk borders inside pages and key tiles, and on them."""
    g = torch.Generator().manual_seed(D + chunk)
    BS = 16
    seqs = [(0, 40), (700, 1), (1279, 1), (75, 3), (599, 2), (300, 33)]
    maxb = 82
    nb = maxb * len(seqs)
    bt = torch.randperm(nb, generator=g).view(len(seqs), maxb).to(torch.int32)
    kc = torch.randn(nb, G, BS, D, generator=g).to(dtype)
    vc = torch.randn(nb, G, VW, BS, generator=g).to(dtype)
    starts, at = [], 0
    for _, n in seqs:
        starts.append(at)
        at += n
    T = at
    rs = i32([i for i, (_, n) in enumerate(seqs) for _ in range(n)])
    pos = i32([h + j for h, n in seqs for j in range(n)])
    q = torch.randn(T, H, D, generator=g).to(dtype)
    wide = torch.randn(T, H + 5, generator=g).to(dtype)
    sinks = torch.zeros(H)
    kw = dict(chunk=chunk, sinks=sinks if chunk else None)
    ref = torch.zeros(T, H, VW, dtype=dtype)
    torch_ref.paged_attention(ref, q, kc, vc, bt, rs, pos, 0.3,
                              gate=wide[:, 3:3 + H], **kw)
    tiles = ops.build_attn_tiles(starts, [h for h, _ in seqs],
                                 [n for _, n in seqs], H, G, 1, "cuda")
    if kw["sinks"] is not None:
        kw["sinks"] = sinks.cuda()
    for max_ctx in (0, 1280):
        out = torch.zeros(T, H, VW, dtype=dtype, device="cuda")
        ops.paged_attention(out, q.cuda(), kc.cuda(), vc.cuda(), bt.cuda(),
                            rs.cuda(), pos.cuda(), 0.3, tiles=tiles,
                            exact=exact, max_ctx=max_ctx,
                            gate=wide.cuda()[:, 3:3 + H], **kw)
        close(out, ref, dtype, f"max_ctx={max_ctx}")


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("F,extra", [(40, 24), (13, 5), (64, 0)])
@pytest.mark.parametrize("mode", ["gelu_tanh", "silu"])
def test_act_and_mul_of_strided_rows(dtype, F, extra, mode):
    g = torch.Generator().manual_seed(F)
    gu = torch.randn(9, 2 * F + extra, generator=g).to(dtype)
    ref, out = torch.zeros(9, F, dtype=dtype), torch.zeros(9, F, dtype=dtype)
    torch_ref.act_and_mul(ref, gu[:, :2 * F], mode)
    out = out.cuda()
    ops.act_and_mul(out, gu.cuda()[:, :2 * F], mode)
    close(out, ref, dtype)


def test_embed_streams():
    g = torch.Generator().manual_seed(0)
    e = torch.randn(11, 30, generator=g).bfloat16()
    tok = torch.tensor([3, 10, 0, 3])
    ref, x = torch.zeros(4, 5, 30), torch.zeros(4, 5, 30, device="cuda")
    torch_ref.embed_streams(ref, tok, e, 0.3)
    ops.embed_streams(x, tok.cuda(), e.cuda(), 0.3)
    close(x, ref, torch.float32)
