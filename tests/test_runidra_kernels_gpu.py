"""GPU numerics of the kernels Runidra adds to the extension _mix (residual
streams, matrix LSTM, router, gated unit, soft cap) and of the switches it adds
to the latent attention: each against the eager fp32 torch version of the same
op (ops/reference.py), for bf16 and float32 activations, on sizes that are not
multiples of the kernels' tiles."""

import pytest
import torch

from parallax_amd import ops
from parallax_amd.ops import reference as ref

pytestmark = pytest.mark.gpu

DEV = "cuda"
BOTH = [torch.bfloat16, torch.float32]


def _rand(*shape, dtype=torch.float32, scale=1.0, seed=0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def _close(got, want, dtype, scale=1.0):
    tol = (1e-2 if dtype == torch.bfloat16 else 2e-5) * scale
    torch.testing.assert_close(got.float().cpu(), want.float(), rtol=tol, atol=tol)


def _close_heads(got, want, dtype):
    """Each head's result is divided by its RMS, which magnifies rounding where
    the sum before it cancels."""
    tol = 2e-2 if dtype == torch.bfloat16 else 5e-4
    torch.testing.assert_close(got.float().cpu(), want.float(), rtol=tol, atol=tol)


# -- residual streams --------------------------------------------------------------


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("S,W", [(1, 48), (2, 1024), (3, 1000), (4, 4096), (2, 4100),
                                 (5, 64), (2, 33), (8, 260)])
def test_hyper_rmsnorm(dtype, S, W):
    T = 7
    x = _rand(T, S * W, seed=1)
    mix, wr, rd = _rand(S, S, seed=2), _rand(S, seed=3), _rand(S, seed=4)
    w = _rand(W, dtype=dtype, seed=5)
    bias = _rand(W, dtype=dtype, seed=6)
    y2, gate = _rand(T, W, dtype=dtype, seed=7), _rand(T, seed=8)
    wide = _rand(T, 2 * W, dtype=dtype, seed=9)
    cases = [
        (_rand(T, W, dtype=dtype, seed=10), None, None, None, True, True),
        (_rand(T, W, seed=11), bias, y2, gate, True, True),     # fp32 result
        (wide[:, W:], bias, None, None, True, True),            # strided
        (None, None, None, None, False, True),                  # read only
        (_rand(T, W, dtype=dtype, seed=12), None, y2, gate, True, False),
    ]
    for y, b, z2, g, update, read in cases:
        a = [y, b, z2, g, mix if update else None, wr if update else None,
             rd if read else None, w if read else None]
        xr, xg = x.clone(), x.to(DEV)
        want = ref.hyper_rmsnorm(xr, *a, 1e-5, torch.float32)
        da = [None if t is None else t.to(DEV) for t in a]
        if y is wide or (y is not None and not y.is_contiguous()):
            da[0] = wide.to(DEV)[:, W:]
        got = ops.hyper_rmsnorm(xg, *da, 1e-5, dtype)
        torch.testing.assert_close(xg.cpu(), xr, rtol=1e-5, atol=1e-5)
        if read:
            assert got.dtype == dtype
            _close(got, want, dtype)
        else:
            assert got is None


@pytest.mark.parametrize("dtype", BOTH)
def test_embed_streams(dtype):
    table = _rand(37, 100, dtype=dtype)
    ids = torch.tensor([0, 36, 5, 5, 12])
    got = ops.embed_streams(ids.to(DEV), table.to(DEV), 3).cpu()
    assert torch.equal(got, ref.embed_streams(ids, table, 3))


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("act", ["silu", "gelu_tanh"])
@pytest.mark.parametrize("I,bias", [(96, True), (37, True), (256, False)])
def test_biased_glu(dtype, act, I, bias):
    x = _rand(9, 2 * I + 8, dtype=dtype, scale=3.0, seed=1)
    b = _rand(2 * I, dtype=dtype, seed=2) if bias else None
    want = ref.biased_glu(x[:, : 2 * I].float(), b, act)
    got = ops.biased_glu(x.to(DEV)[:, : 2 * I], None if b is None else b.to(DEV), act)
    _close(got, want, dtype)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("n,scale,cap", [(520, 1.7, 11.0), (77, 0.25, 0.0), (33, 9.0, 1.5)])
def test_softcap_logits(dtype, n, scale, cap):
    x = _rand(3, n, dtype=dtype, scale=20.0)
    got = ops.softcap_logits(x.to(DEV), scale, cap)
    assert got.dtype == torch.float32
    torch.testing.assert_close(got.cpu(), ref.softcap_logits(x, scale, cap),
                               rtol=1e-5, atol=1e-5)


# -- small projections and the router ------------------------------------------------


@pytest.mark.parametrize("T,N,K", [(1, 3, 48), (8, 32, 2048), (33, 12, 100), (70, 130, 512)])
def test_linear_f32(T, N, K):
    x, w = _rand(T, K, dtype=torch.bfloat16, seed=1), _rand(N, K, dtype=torch.bfloat16, seed=2)
    got = ops.linear_f32(x.to(DEV), w.to(DEV))
    assert got.dtype == torch.float32
    torch.testing.assert_close(got.cpu(), ref.linear_f32(x, w), rtol=1e-4, atol=1e-3)
    xs = _rand(T, K + 8, dtype=torch.bfloat16, seed=3)
    torch.testing.assert_close(ops.linear_f32(xs.to(DEV)[:, 8:], w.to(DEV)).cpu(),
                               ref.linear_f32(xs[:, 8:], w), rtol=1e-4, atol=1e-3)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("E,top,extra,bias", [(20, 5, 1, True), (6, 6, 0, True), (1, 1, 1, True),
                                              (130, 9, 1, False), (239, 3, 1, True),
                                              (300, 5, 1, True)])
def test_route_softmax(dtype, E, top, extra, bias):
    T, K = 37, 256
    x = _rand(T, K, dtype=dtype, seed=1)
    w = _rand(E + extra, K, dtype=dtype, scale=0.1, seed=2)
    b = _rand(E, seed=3) if bias else None
    ids, wts, rest = ops.route_softmax(x.to(DEV), w.to(DEV), None if b is None else b.to(DEV),
                                       E, top)
    rid, rw, rr = ref.route_softmax(x, w, b, E, top)
    assert ids.dtype == torch.int64 and wts.dtype == torch.float32
    assert torch.equal(ids.cpu(), rid)
    torch.testing.assert_close(wts.cpu(), rw, rtol=1e-4, atol=1e-5)
    torch.testing.assert_close(rest.cpu(), rr, rtol=1e-4, atol=1e-3)


# -- matrix LSTM ---------------------------------------------------------------------


def _mlstm_inputs(T, H, d, dv, dtype, seed=0, scale=1.0):
    qkvg = _rand(T, H * (2 * d + 2 * dv), dtype=dtype, seed=seed)
    gates = _rand(T, 2 * H, scale=3.0 * scale, seed=seed + 1)
    gates[:, H:] += 2.0
    bias = _rand(2 * H, seed=seed + 2)
    w = _rand(H * dv, dtype=dtype, seed=seed + 3)
    return qkvg, gates, bias, w


def _run_mlstm(fn, dev, qkvg, gates, bias, w, state, slots, cu, pos, H, d, dv, cap, dtype):
    q, k, v, g = torch.split(qkvg.to(dev), [H * d, H * d, H * dv, H * dv], dim=1)
    return fn(q, k, v, g, gates.to(dev), bias.to(dev), w.to(dev), cap, 1e-5, state,
              torch.tensor(slots, device=dev),
              None if cu is None else torch.tensor(cu, dtype=torch.int32, device=dev),
              torch.tensor(pos, dtype=torch.int32, device=dev), dtype)


def _pad(d, dv):
    return (d * dv + d + 1 + 3) // 4 * 4


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("H,d,dv,cap", [(2, 40, 56, 10.0), (3, 64, 40, 5.0), (1, 128, 128, 15.0),
                                        (2, 24, 136, 8.0), (2, 20, 17, 1.0), (1, 8, 8, 30.0),
                                        (1, 200, 24, 12.0)])
def test_mlstm_portions_and_steps(dtype, H, d, dv, cap):
    """Portions of several sequences, one of them continued twice and then
    decoded, against the serial reference; dirty slots at the start."""
    lens = [150, 3, 64, 65]
    slots = [3, 0, 2, 4]
    st_r = torch.full((5, H, _pad(d, dv)), 7.0)
    st_g = st_r.to(DEV)
    start = [0] * len(lens)
    for rnd, ns in enumerate([lens, [2, 70, 1, 128]]):
        T = sum(ns)
        cu = [0]
        pos = []
        for n, s in zip(ns, start):
            cu.append(cu[-1] + n)
            pos += list(range(s, s + n))
        ins = _mlstm_inputs(T, H, d, dv, dtype, seed=10 * rnd)
        args = (slots, cu, pos, H, d, dv, cap)
        want = _run_mlstm(ref.mlstm, "cpu", *ins, st_r, *args, torch.float32)
        got = _run_mlstm(ops.mlstm, DEV, *ins, st_g, *args, dtype)
        _close_heads(got, want, dtype)
        used = d * dv + d + 1
        torch.testing.assert_close(st_g.cpu()[..., :used], st_r[..., :used],
                                   rtol=2e-4, atol=2e-4)
        start = [s + n for s, n in zip(start, ns)]
    for step in range(3):
        ins = _mlstm_inputs(len(lens), H, d, dv, dtype, seed=100 + step)
        args = (slots, None, [s + step for s in start], H, d, dv, cap)
        want = _run_mlstm(ref.mlstm, "cpu", *ins, st_r, *args, torch.float32)
        got = _run_mlstm(ops.mlstm, DEV, *ins, st_g, *args, dtype)
        _close_heads(got, want, dtype)
    used = d * dv + d + 1
    torch.testing.assert_close(st_g.cpu()[..., :used], st_r[..., :used], rtol=3e-4, atol=3e-4)
    assert float(st_g[1].min()) == 7.0 == float(st_g[1].max())   # a slot of nobody


def test_mlstm_chunks_match_the_serial_order_with_extreme_gates():
    """Chunked bf16 against float64 arithmetic where forget gates swing between
    keeping everything and dropping everything: sums over a chunk reach
    hundreds while neighbours differ by a fraction."""
    H, d, dv, cap, T = 2, 64, 64, 20.0, 300
    ins = list(_mlstm_inputs(T, H, d, dv, torch.bfloat16, seed=5))
    ins[1][:, H:] = torch.where(torch.arange(T).view(-1, 1) % 7 < 5,
                                torch.tensor(-25.0), torch.tensor(9.0))
    ins[1][40, :H] = 40.0     # one token that takes over the memory
    st_r, st_g = torch.zeros(1, H, _pad(d, dv)), torch.zeros(1, H, _pad(d, dv), device=DEV)
    args = ([0], [0, T], list(range(T)), H, d, dv, cap)
    want = _run_mlstm(ref.mlstm, "cpu", *ins, st_r, *args, torch.float32)
    got = _run_mlstm(ops.mlstm, DEV, *ins, st_g, *args, torch.bfloat16)
    _close_heads(got, want, torch.bfloat16)
    used = d * dv + d + 1
    torch.testing.assert_close(st_g.cpu()[..., :used], st_r[..., :used], rtol=1e-4, atol=1e-4)


# -- latent attention switches -------------------------------------------------------


def _freq(dims, base=10000.0):
    return torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)])


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("rank,rot_w,q_rank", [(72, 32, 120), (40, 24, 50), (300, 8, 1)])
def test_latent_kv_store_interleaved_with_query_latent(dtype, rank, rot_w, q_rank):
    T, bs = 6, 4
    both = _rand(T, q_rank + rank + rot_w, dtype=dtype, seed=1)
    nw, qw = _rand(rank, dtype=dtype, seed=2), _rand(q_rank, dtype=dtype, seed=3)
    pos = torch.tensor([0, 3, 17, 255, 1000, 5], dtype=torch.int32)
    slots = torch.tensor([3, 0, 7, 11, 6, -1])
    freq = _freq(rot_w)
    c_r = torch.zeros(3, bs, rank + rot_w)
    c_g = torch.zeros(3, bs, rank + rot_w, dtype=dtype, device=DEV)
    want = ref.latent_kv_store(both[:, q_rank:], nw, 1e-5, freq, 1.0, rot_w, pos, slots,
                               c_r, rank, True, both[:, :q_rank].float(), qw)
    bg = both.to(DEV)
    got = ops.latent_kv_store(bg[:, q_rank:], nw.to(DEV), 1e-5, freq.to(DEV), 1.0, rot_w,
                              pos.to(DEV), slots.to(DEV), c_g, rank, True,
                              bg[:, :q_rank], qw.to(DEV))
    _close(got, want, dtype)
    _close(c_g, c_r, dtype)


@pytest.mark.parametrize("dtype", BOTH)
def test_rope_rows_interleaved(dtype):
    q = _rand(5, 3, 40, dtype=dtype)
    pos = torch.tensor([0, 1, 9, 500, 4000], dtype=torch.int32)
    freq = _freq(16)
    want = ref.rope_rows(q, 24, 16, freq, 1.0, 16, pos, True)
    got = ops.rope_rows(q.to(DEV), 24, 16, freq.to(DEV), 1.0, 16, pos.to(DEV), True)
    torch.testing.assert_close(got.cpu(), want, rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("H,rank,rot_w,window,ctx", [(8, 72, 24, 90, 300), (3, 40, 16, 9, 50),
                                                     (16, 512, 64, 1024, 1500), (1, 24, 8, 1, 7)])
@pytest.mark.parametrize("decode", [False, True])
def test_latent_window_attention_sink(dtype, H, rank, rot_w, window, ctx, decode):
    bs = 16
    pages = (ctx + bs - 1) // bs
    cache = _rand(pages + 2, bs, rank + rot_w, dtype=dtype, seed=1)
    table = torch.randperm(pages + 2, generator=torch.Generator().manual_seed(2))[:pages]
    n = 1 if decode else min(ctx, 21)
    pos = torch.arange(ctx - n, ctx, dtype=torch.int32)
    q_lat, q_rot = _rand(n, H, rank, seed=3), _rand(n, H, rot_w, seed=4)
    bt = table.int().view(1, -1)
    seq = None if decode else torch.zeros(n, dtype=torch.int32)
    for sink in (_rand(H, seed=5), torch.full((H,), 6.0), torch.full((H,), -50.0), None):
        want = ref.latent_window_attention(q_lat, q_rot, cache, bt, seq, pos, window, 0.1, sink)
        got = ops.latent_window_attention(
            q_lat.to(DEV), q_rot.to(DEV), cache.to(DEV), bt.to(DEV),
            None if seq is None else seq.to(DEV), pos.to(DEV), window, 0.1, ctx,
            None if sink is None else sink.to(DEV))
        torch.testing.assert_close(got.cpu(), want, rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("H,dn,dr,dv,rank,window", [
    (8, 56, 24, 40, 72, 90), (3, 24, 8, 72, 40, 33), (16, 128, 64, 128, 512, 1024),
    (1, 8, 64, 8, 24, 1), (2, 104, 40, 120, 64, 500)])
def test_latent_expanded_attention(H, dn, dr, dv, rank, window):
    """Gathered contexts and tiled portions: sequences of unequal length, one
    that starts inside its context, one of a single token, tiles that end
    ragged; a planted key at the window's edge."""
    from parallax_amd.models.forward_meta import ForwardMeta

    bf = torch.bfloat16
    portions = [(0, 300), (700, 150), (41, 1), (0, 2), (5, 128)]
    bs, n_pages = 16, 400
    cache = _rand(n_pages, bs, rank + dr, dtype=bf, seed=1)
    perm = torch.randperm(n_pages, generator=torch.Generator().manual_seed(2)).int()
    bt = perm[: 5 * 60].view(5, 60).contiguous()
    pos = torch.cat([torch.arange(s, s + n) for s, n in portions]).int()
    lens = torch.tensor([n for _, n in portions], dtype=torch.int32)
    T = pos.numel()

    def meta(dev):
        return ForwardMeta(is_prefill=True, positions=pos.to(dev), slot_mapping=None,
                           block_tables=bt.to(dev), seq_lens=None, query_lens=lens.to(dev),
                           portions=portions)

    mr, mg = meta("cpu"), meta(DEV)
    plan, rows = mr.window_contexts(window)
    assert rows == sum(s + n - max(0, s - window + 1) for s, n in portions)
    lat_r, rot_r = ref.latent_gather(cache, bt, plan, rows, rank)
    lat_g, rot_g = ops.latent_gather(cache.to(DEV), bt.to(DEV), mg.window_contexts(window)[0],
                                     rows, rank)
    assert torch.equal(lat_g[:rows].cpu(), lat_r) and torch.equal(rot_g[:rows].cpu(), rot_r)
    kv = _rand(rows, H * (dn + dv), dtype=bf, seed=3)
    q = _rand(T, H, dn + dr, dtype=bf, seed=4)
    q_rot = _rand(T, H, dr, seed=5)
    # one key of the second sequence stands out for every head: seen up to
    # the window's edge and not beyond
    kv[int(plan[1]) + min(20, window - 1), : H * dn] = 3.0
    for sink in (None, _rand(H, seed=6), torch.full((H,), 5.0)):
        want = ref.latent_expanded_attention(q.float(), q_rot, kv, rot_r, plan, mr.query_bounds(),
                                             pos, window, 0.15, sink)
        kv_pad = torch.full((rot_g.shape[0], kv.shape[1]), float("nan"), dtype=bf)
        kv_pad[:rows] = kv
        got = ops.latent_expanded_attention(
            q.to(DEV), q_rot.to(DEV), kv_pad.to(DEV), rot_g, mg.window_contexts(window)[0],
            mg.query_bounds(), pos.to(DEV), window, 0.15,
            None if sink is None else sink.to(DEV))
        _close(got, want, bf)
