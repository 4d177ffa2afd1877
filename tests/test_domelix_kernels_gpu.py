"""GPU numerics of the kernels Domelix adds to the extension _mix (parallel
residual with two norms, short convolution, rotation table, fixed-decay linear
attention, gated delta rule) and of the switches it adds to the row attention,
the gated norm and the router: each against the eager fp32 torch version of the
same op (ops/reference.py), for bf16 and float32 activations, on sizes that are
not multiples of the kernels' tiles."""

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


def _dev(t):
    return None if t is None else t.to(DEV)


# -- residual step ---------------------------------------------------------------


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("W", [48, 1024, 1000, 4096, 4100, 33])
def test_parallel_rmsnorm_add(dtype, W):
    T = 7
    wa, wb, w1, w2 = (_rand(W, dtype=dtype, seed=s, scale=0.5) for s in range(4))
    wide = _rand(T, 2 * W, dtype=dtype, seed=5, scale=3.0)
    b = _rand(T, W, dtype=dtype, seed=6, scale=0.1)
    f32, fT = _rand(T, W, seed=7), _rand(T, W, dtype=dtype, seed=8)
    for a, bb, f, n1, n2 in [
        (wide[:, W:], b, f32, w1, w2), (wide[:, W:], None, fT, w1, w2),
        (wide[:, W:], b, None, w1, None), (None, None, None, w1, w2),
        (None, None, f32, None, w2), (wide[:, W:], b, f32, None, None),
    ]:
        x = _rand(T, W, seed=9)
        xr, xg = x.clone(), x.to(DEV)
        want = ref.parallel_rmsnorm_add(xr, a, bb, wa, wb, 0.5, f, n1, n2, 1e-5, 1.0,
                                        torch.float32)
        ag = None if a is None else wide.to(DEV)[:, W:]
        got = ops.parallel_rmsnorm_add(xg, ag, _dev(bb), wa.to(DEV), wb.to(DEV), 0.5,
                                       _dev(f), _dev(n1), _dev(n2), 1e-5, 1.0, dtype)
        torch.testing.assert_close(xg.cpu(), xr, rtol=1e-5, atol=1e-5)
        for g, r in zip(got, want):
            assert (g is None) == (r is None)
            if g is not None:
                assert g.dtype == dtype
                _close(g, r, dtype)


# -- gated norm --------------------------------------------------------------------


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("H,dv", [(3, 20), (2, 33), (6, 40), (4, 128), (1, 256), (2, 300),
                                  (32, 128), (33, 128), (5, 1)])
@pytest.mark.parametrize("act", ["silu", "sigmoid"])
def test_gated_rmsnorm(dtype, H, dv, act):
    T = 5
    o = _rand(T, H, dv, seed=1, scale=2.0)
    gate = _rand(T, H * dv + 8, dtype=dtype, seed=2)
    for whole, w in [(False, None), (False, _rand(dv, dtype=dtype, seed=3)), (True, None),
                     (True, _rand(H * dv, dtype=dtype, seed=4))]:
        want = ref.gated_rmsnorm(o, gate[:, 8:], w, 1e-5, torch.float32, whole, act)
        got = ops.gated_rmsnorm(o.to(DEV), gate.to(DEV)[:, 8:], _dev(w), 1e-5, dtype, whole, act)
        assert got.dtype == dtype
        _close(got, want, dtype)


# -- short convolution --------------------------------------------------------------


LENS = [1, 2, 3, 17, 8, 40, 5]


def _bounds(lens):
    return torch.tensor([0] + lens).cumsum(0).int()


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("C,taps", [(64, 4), (36, 3), (33, 4), (20, 2), (12, 1), (24, 6), (7, 9)])
def test_short_conv(dtype, C, taps):
    cu, T = _bounds(LENS), sum(LENS)
    B = len(LENS)
    x = _rand(T, C + 4, dtype=dtype, seed=1)
    w = _rand(C, taps, dtype=dtype, seed=2)
    state = _rand(B + 2, C, taps - 1, dtype=dtype, seed=3)
    slots = torch.tensor([3, 0, 7, 1, 5, 2, 4])
    # every other sequence begins at 0, whatever its slot holds
    pos = torch.cat([torch.arange(n) + (0 if b % 2 else 11) for b, n in enumerate(LENS)]).int()
    sr, sg = state.clone(), state.to(DEV)
    want = ref.short_conv(x[:, :C], w, sr, slots, cu, pos, torch.float32)
    got = ops.short_conv(x.to(DEV)[:, :C], w.to(DEV), sg, slots.to(DEV), cu.to(DEV),
                         pos.to(DEV), dtype)
    _close(got, want, dtype)
    assert torch.equal(sg.cpu(), sr)
    # one token per sequence
    x1, p1 = _rand(B, C, dtype=dtype, seed=4), torch.tensor([5, 0, 9, 1, 0, 30, 2]).int()
    want = ref.short_conv(x1, w, sr, slots, None, p1, torch.float32)
    got = ops.short_conv(x1.to(DEV), w.to(DEV), sg, slots.to(DEV), None, p1.to(DEV), dtype)
    _close(got, want, dtype)
    assert torch.equal(sg.cpu(), sr)


def test_rope_table():
    pos = torch.tensor([0, 1, 2, 77, 5000]).int()
    freq = 500.0 ** (-torch.arange(0, 10, 2).float() / 10)
    got = ops.rope_table(pos.to(DEV), freq.to(DEV)).cpu()
    torch.testing.assert_close(got, ref.rope_table(pos, freq), rtol=1e-5, atol=1e-5)


# -- linear attention with a fixed decay, gated delta rule ---------------------------


# (q/k heads, heads, key width, value width)
SIZES = [(2, 2, 64, 64), (3, 3, 32, 40), (2, 4, 128, 128), (1, 3, 128, 72), (2, 2, 20, 12),
         (1, 2, 13, 7), (1, 1, 256, 96), (2, 2, 1, 1), (1, 1, 300, 20), (1, 1, 600, 8)]
DECAYS = [0.9995, 0.55, 0.0, 1.0]


def _sequences(short):
    lens = [1, 2, 5, 3] if short else [70, 33, 1, 160, 32, 2]
    pos = torch.cat([torch.arange(n) + (0 if b % 2 else 9) for b, n in enumerate(lens)]).int()
    return lens, _bounds(lens), pos


def _decay_case(G, H, d, dv, dtype, lens, seed):
    T = sum(lens)
    y = _rand(T, 2 * G * d + H * dv, dtype=dtype, seed=seed)
    q, k, v = torch.split(y, [G * d, G * d, H * dv], -1)
    view = lambda t, n: t.unflatten(-1, (n, -1))
    return y, view(q, G), view(k, G), view(v, H)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("short", [False, True])
@pytest.mark.parametrize("H,d,dv", sorted({(H, d, dv) for _, H, d, dv in SIZES}))
@pytest.mark.parametrize("form", ["plain", "silu", "rotated"])
def test_decay_attention(dtype, short, H, d, dv, form):
    lens, cu, pos = _sequences(short)
    B = len(lens)
    y, q, k, v = _decay_case(H, H, d, dv, dtype, lens, 1)
    powers = ops.decay_powers((DECAYS * H)[:H])
    cs = None
    if form == "rotated":
        n = d // 2 - (3 if d > 64 else 0)    # all of the head, or part of it
        if n:
            cs = ref.rope_table(pos, 100.0 ** (-torch.arange(n).float() / n))
    scale = d ** -0.5 if form != "silu" else 1.0
    state = _rand(B + 1, H, d, dv, seed=2)
    slots = torch.tensor([2, 0, 4, 1, 6, 3][:B])
    sr, sg = state.clone(), state.to(DEV)
    want = ref.decay_attention(q, k, v, powers[:, 1], scale, form == "silu", cs, sr, slots, cu, pos)
    yg = y.to(DEV)
    qg, kg, vg = (t.unflatten(-1, (H, -1)) for t in torch.split(yg, [H * d, H * d, H * dv], -1))
    got = ops.decay_attention(qg, kg, vg, powers.to(DEV), scale, form == "silu", _dev(cs), sg,
                              slots.to(DEV), cu.to(DEV), pos.to(DEV))
    tol = 2e-5 * max(1.0, float(want.abs().max()))
    torch.testing.assert_close(got.cpu(), want, rtol=1e-4, atol=tol)
    torch.testing.assert_close(sg.cpu(), sr, rtol=1e-4, atol=2e-5 * max(1.0, float(sr.abs().max())))
    # decode: one token per sequence
    y, q, k, v = _decay_case(H, H, d, dv, dtype, [1] * B, 3)
    p1 = torch.tensor([70, 0, 8, 160, 33, 4][:B]).int()
    if cs is not None:
        cs = ref.rope_table(p1, 100.0 ** (-torch.arange(cs.shape[1] // 2).float()
                                          / (cs.shape[1] // 2)))
    want = ref.decay_attention(q, k, v, powers[:, 1], scale, form == "silu", cs, sr, slots, None, p1)
    got = ops.decay_attention(q.to(DEV), k.to(DEV), v.to(DEV), powers.to(DEV), scale,
                              form == "silu", _dev(cs), sg, slots.to(DEV), None, p1.to(DEV))
    torch.testing.assert_close(got.cpu(), want, rtol=1e-4,
                               atol=2e-5 * max(1.0, float(want.abs().max())))
    torch.testing.assert_close(sg.cpu(), sr, rtol=1e-4, atol=2e-5 * max(1.0, float(sr.abs().max())))


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("short", [False, True])
@pytest.mark.parametrize("G,H,d,dv", SIZES)
@pytest.mark.parametrize("keys", ["random", "alike"])
def test_gated_delta_rule(dtype, short, G, H, d, dv, keys):
    """keys alike: one direction written over and over with step sizes near 1,
    where the triangular system of a chunk is far from the identity."""
    lens, cu, pos = _sequences(short)
    B, T = len(lens), sum(lens)
    y, q, k, v = _decay_case(G, H, d, dv, dtype, lens, 5)
    gates = _rand(T, 2 * H, seed=6, scale=2.0)
    if keys == "alike":
        k.copy_((k.float() * 0.02 + 1.0).to(dtype))
        gates[:, :H] = 4.0
        gates[:, H:] -= 6.0
    a_log, dt = _rand(H, seed=7), _rand(H, seed=8)
    state = _rand(B + 1, H, d, dv, seed=9)
    slots = torch.tensor([2, 0, 4, 1, 6, 3][:B])
    sr, sg = state.clone(), state.to(DEV)
    want = ref.gated_delta_rule(q, k, v, gates, a_log, dt, sr, slots, cu, pos)
    yg = y.to(DEV)
    qg, kg, vg = torch.split(yg, [G * d, G * d, H * dv], -1)
    got = ops.gated_delta_rule(qg.unflatten(-1, (G, -1)), kg.unflatten(-1, (G, -1)),
                               vg.unflatten(-1, (H, -1)), gates.to(DEV), a_log.to(DEV),
                               dt.to(DEV), sg, slots.to(DEV), cu.to(DEV), pos.to(DEV))
    tol = 5e-5 * max(1.0, float(want.abs().max()))
    torch.testing.assert_close(got.cpu(), want, rtol=2e-4, atol=tol)
    torch.testing.assert_close(sg.cpu(), sr, rtol=2e-4, atol=5e-5 * max(1.0, float(sr.abs().max())))
    y, q, k, v = _decay_case(G, H, d, dv, dtype, [1] * B, 10)
    g1, p1 = _rand(B, 2 * H, seed=11), torch.tensor([70, 0, 8, 160, 33, 4][:B]).int()
    want = ref.gated_delta_rule(q, k, v, g1, a_log, dt, sr, slots, None, p1)
    got = ops.gated_delta_rule(q.to(DEV), k.to(DEV), v.to(DEV), g1.to(DEV), a_log.to(DEV),
                               dt.to(DEV), sg, slots.to(DEV), None, p1.to(DEV))
    torch.testing.assert_close(got.cpu(), want, rtol=2e-4,
                               atol=5e-5 * max(1.0, float(want.abs().max())))
    torch.testing.assert_close(sg.cpu(), sr, rtol=2e-4, atol=5e-5 * max(1.0, float(sr.abs().max())))


def test_chunks_agree_with_single_tokens():
    """The chunked kernels against the token-serial one on the same portion."""
    H, d, dv, T = 3, 64, 48, 200
    q, k, v = (_rand(T, H, n, dtype=torch.bfloat16, seed=s).to(DEV)
               for s, n in ((1, d), (2, d), (3, dv)))
    gates, a_log, dt = _rand(T, 2 * H, seed=4).to(DEV), torch.zeros(H).to(DEV), torch.zeros(H).to(DEV)
    powers = ops.decay_powers([0.99, 0.5, 1.0]).to(DEV)
    slots = torch.zeros(1, dtype=torch.long, device=DEV)
    pos = torch.arange(T, dtype=torch.int32, device=DEV)
    for fn, extra in ((ops.gated_delta_rule, (gates, a_log, dt)),
                      (ops.decay_attention, (powers, 0.125, False, None))):
        s1, s2 = torch.zeros(1, H, d, dv, device=DEV), torch.zeros(1, H, d, dv, device=DEV)
        cu = torch.tensor([0, T], dtype=torch.int32, device=DEV)
        whole = fn(q, k, v, *extra, s1, slots, cu, pos)
        cut = lambda t, i: t[i:i + 1] if torch.is_tensor(t) and t.shape[:1] == (T,) else t
        one = torch.cat([fn(q[i:i + 1], k[i:i + 1], v[i:i + 1], *[cut(e, i) for e in extra], s2,
                            slots, None, pos[i:i + 1]) for i in range(T)])
        torch.testing.assert_close(whole, one, rtol=1e-4, atol=1e-4)
        torch.testing.assert_close(s1, s2, rtol=1e-4, atol=1e-4)


# -- row attention: distance bias, sinks, element-wise gate ----------------------------


def _row_case(dtype, H, G, d, dv, lens, bs=16, seed=0):
    """Random paged rows of every sequence and the portion of its last tokens."""
    ctx = [c for c, _ in lens]
    pages = [(c + bs - 1) // bs for c in ctx]
    perm = torch.randperm(sum(pages) + 2, generator=torch.Generator().manual_seed(seed))
    bt = torch.zeros(len(lens), max(pages), dtype=torch.int32)
    at = 0
    for b, n in enumerate(pages):
        bt[b, :n] = perm[at:at + n].int()
        at += n
    cache = _rand(sum(pages) + 2, bs, G * (d + dv), dtype=dtype, seed=seed + 1)
    T = sum(n for _, n in lens)
    q = _rand(T, H * d, dtype=dtype, seed=seed + 2).float()
    pos = torch.cat([torch.arange(c - n, c) for c, n in lens]).int()
    seq = torch.cat([torch.full((n,), b) for b, (_, n) in enumerate(lens)]).int()
    return q, cache, bt, seq, pos, _bounds([n for _, n in lens])


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("H,G,d,dv", [(8, 2, 64, 64), (6, 2, 32, 48), (3, 3, 20, 12), (8, 2, 128, 128),
                                      (5, 1, 7, 9), (2, 2, 64, 200)])
@pytest.mark.parametrize("n_bias", [1, 9, 60, 1000])
def test_row_attention_with_bias_sink_and_gate(dtype, H, G, d, dv, n_bias):
    for lens in ([(150, 150), (33, 2), (200, 40), (1, 1)], [(90, 1), (300, 1), (1, 1)]):
        decode = all(n == 1 for _, n in lens)
        q, cache, bt, seq, pos, cu = _row_case(dtype, H, G, d, dv, lens, seed=n_bias)
        bias = _rand(H, n_bias, seed=3, scale=2.0)
        sink = _rand(H, seed=4, scale=3.0)
        gate = _rand(q.shape[0], H * dv + 8, dtype=dtype, seed=5)
        one = _rand(q.shape[0], H, dtype=dtype, seed=6)
        for kw in (dict(dist_bias=bias, sink=sink, gate=gate), dict(dist_bias=bias, gate=one),
                   dict(sink=sink), dict(gate=gate)):
            wide = kw.get("gate") is gate
            args = (H, G, 1, d, dv, 0, 0, d ** -0.5, 0.0, 0.0, None, 1.0)
            rk = dict(kw, gate=gate[:, 8:]) if wide else kw
            want = ref.row_attention(q, cache, None, bt, None if decode else seq, pos, *args,
                                     torch.float32, **rk)
            gk = {n: t.to(DEV) for n, t in kw.items()}
            if wide:
                gk["gate"] = gk["gate"][:, 8:]
            got = ops.row_attention(q.to(DEV), cache.to(DEV), None, bt.to(DEV),
                                    None if decode else seq.to(DEV), pos.to(DEV), *args, dtype,
                                    max_seq_len=300, query_bounds=None if decode else cu.to(DEV),
                                    bf16_queries=dtype == torch.bfloat16, **gk)
            _close(got, want, dtype)


def test_row_attention_queries_that_are_no_bf16_numbers():
    """Without the flag all of an fp32 query counts over bf16 rows."""
    q, cache, bt, seq, pos, cu = _row_case(torch.bfloat16, 4, 2, 64, 64, [(120, 120), (70, 9)])
    q = q + _rand(*q.shape, seed=8, scale=1e-3)
    bias = _rand(4, 30, seed=3)
    args = (4, 2, 1, 64, 64, 0, 0, 0.5, 0.0, 0.0, None, 1.0, torch.float32)
    want = ref.row_attention(q, cache, None, bt, seq, pos, *args, dist_bias=bias)
    got = ops.row_attention(q.to(DEV), cache.to(DEV), None, bt.to(DEV), seq.to(DEV), pos.to(DEV),
                            *args, max_seq_len=120, query_bounds=cu.to(DEV), dist_bias=bias.to(DEV))
    torch.testing.assert_close(got.cpu(), want, rtol=2e-5, atol=2e-5)


# -- router -----------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("E,top,groups,keep", [(14, 3, 2, 1), (15, 4, 5, 2), (64, 8, 8, 3), (8, 8, 4, 4),
                                               (6, 1, 6, 1), (128, 6, 16, 4), (200, 5, 20, 7),
                                               (10, 4, 1, 1), (260, 4, 4, 2)])
def test_route_softmax_in_groups(dtype, E, top, groups, keep):
    T, W = 37, 72
    x, w = _rand(T, W, dtype=dtype, seed=1), _rand(E, W, dtype=dtype, seed=2, scale=0.3)
    ids, wts, _ = ref.route_softmax(x, w, None, E, top, groups, keep)
    gi, gw, _ = ops.route_softmax(x.to(DEV), w.to(DEV), None, E, top, groups, keep)
    assert torch.equal(gi.cpu(), ids)
    torch.testing.assert_close(gw.cpu(), wts, rtol=1e-5, atol=1e-6)
