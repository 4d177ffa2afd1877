"""Runidra on the CPU engine (fp32) against the plain reference in
runidra_oracle.py: each mechanism alone, then the engine's step function,
cache manager, state slots and scheduler under many ways of cutting and
batching the same sequences. Configurations are small and deliberately
irregular (see runidra_util.small_config)."""

import math

import pytest
import torch

import runidra_oracle as oracle
import runidra_util as U
from parallax_amd import ops
from parallax_amd.models.config import ModelConfig, mlstm_state_width
from parallax_amd.models.forward_meta import ForwardMeta
from parallax_amd.models.latent_attention import LatentWindowAttention
from parallax_amd.models.linear_attention import MLSTM
from parallax_amd.models.runidra import RunidraLayer, RunidraShardModel
from parallax_amd.server.kv_cache import LinearStateCache, MLAKVCache
from parallax_amd.server.sampling_params import SamplingParams

D = oracle.F64
# fp32 rounding: the matrix LSTM divides every head's result by its RMS, which
# magnifies it where the sum before cancels (about 6e-5 on single rows here)
TOL = 2e-4
WIDTH = 40
EPS = 1e-5


@pytest.fixture(scope="module")
def ckpt(tmp_path_factory):
    cfg = U.small_config()
    w = oracle.random_weights(cfg, seed=3)
    path = U.write_checkpoint(str(tmp_path_factory.mktemp("rn")), cfg, w)
    return cfg, w, path


def _rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


# -- mechanisms alone --------------------------------------------------------------


def test_config_reader():
    cfg = U.small_config()
    mc = ModelConfig.from_hf_config(cfg)
    assert mc.architecture == "Runidra" and mc.streams == 3
    # runs, not layers: 0, (1, 2, 3) twice, 4
    assert mc.layer_weights == [0, 1, 2, 3, 1, 2, 3, 4] == oracle.layer_order(cfg)
    assert mc.num_layers == 8 == len(mc.layer_specs)
    assert mc.layer_types[:3] == ["linear_attention", "latent_attention", "linear_attention"]
    # every pass has a cache entry or a state of its own
    assert mc.latent_cache_dims(0, 8) == [(24, 12), (40, 4)] * 2
    assert mc.latent_cache_dims(2, 5) == [(40, 4), (24, 12)]
    assert [r for _, r in mc.linear_state_shapes(0, 8)] == [
        (3, mlstm_state_width(12, 20)), (2, mlstm_state_width(20, 8)),
        (2, mlstm_state_width(20, 8)), (1, mlstm_state_width(16, 16))]
    assert mc.has_linear_layers and mc.logit_softcap == 6.0 and mc.logit_scale == 1.4
    assert mc.num_experts == 5 and mc.shared_expert_intermediate_size == 36
    assert mlstm_state_width(3, 5) == 20 and mlstm_state_width(4, 4) == 24
    plain = ModelConfig.from_hf_config(U.small_config(loop=None))
    assert plain.layer_weights == [0, 1, 2, 3, 4]
    with pytest.raises(ValueError):
        ModelConfig.from_hf_config(U.small_config([{"type": "gla", "mixer": {}, "mlp": None}],
                                                  loop=None))
    with pytest.raises(ValueError):
        ModelConfig.from_hf_config(U.small_config(loop=(1, 6, 2)))


@pytest.mark.parametrize("S", [1, 2, 4])
def test_hyper_connections(S):
    """Write, then read and norm, with the mix matrix indexed [from, to]; a
    matrix taken the other way round would show (it is not symmetric)."""
    T, W = 5, 12
    x = _rand(T, S * W, seed=1)
    mix, wr, rd = _rand(S, S, seed=2), _rand(S, seed=3), _rand(S, seed=4)
    y, bias, y2 = _rand(T, W, seed=5), _rand(W, seed=6), _rand(T, W, seed=7)
    gate, w = _rand(T, 1, seed=8), _rand(W, seed=9)
    X = x.view(T, S, W).permute(1, 0, 2).double()
    z = y.double() + bias.double() + torch.sigmoid(gate.double()) * y2.double()
    want = oracle.hyper_write(X, mix.double(), wr.double(), z)
    got = x.clone()
    h = ops.hyper_rmsnorm(got, y, bias, y2, gate, mix, wr, rd, w, EPS, torch.float32)
    torch.testing.assert_close(got.view(T, S, W).permute(1, 0, 2).double(), want,
                               rtol=1e-5, atol=1e-5)
    torch.testing.assert_close(
        h.double(), oracle.rms_norm(oracle.hyper_read(want, rd.double()), w.double(), EPS),
        rtol=1e-5, atol=1e-5)
    if S > 1:
        other = oracle.hyper_write(X, mix.double().T, wr.double(), z)
        assert (other - want).abs().max() > 0.1
    # reading alone leaves the streams as they are
    keep = got.clone()
    ops.hyper_rmsnorm(got, None, None, None, None, None, None, rd, w, EPS, torch.float32)
    assert torch.equal(got, keep)


def test_feed_forwards_and_router():
    cfg = U.small_config([U.mlstm_layer(mlp=U.dense(28)), U.mlstm_layer(mlp=U.experts(6, 3)),
                          U.mlstm_layer(mlp=U.experts(4, 4, 8, 0))], loop=None)
    w = oracle.random_weights(cfg, seed=5)
    mc = ModelConfig.from_hf_config(cfg)
    m = RunidraShardModel(mc).float()
    for k, v in w.items():
        assert m.load_hf_weight(k, v), k
    m.finalize_weights()
    m = m.float()
    h = _rand(17, WIDTH, seed=2)
    d = m.layers[0].mlp
    torch.testing.assert_close((d(h) + d.down_bias).double(), oracle.dense_ff(h.double(), w, "l0.mlp."),
                               rtol=1e-4, atol=1e-4)
    for n in (1, 2):
        mlp = cfg["layers"][n]["mlp"]
        y, y2, gate = m.layers[n].mlp(h)
        assert (y2 is None) == (not mlp.get("shared"))
        if y2 is not None:
            y = y + torch.sigmoid(gate) * y2
        torch.testing.assert_close(y.double(), oracle.moe(h.double(), w, "l%d.mlp." % n, mlp),
                                   rtol=1e-4, atol=1e-4)
        ids, wts, _ = m.layers[n].mlp.experts.router.route(h)
        want = oracle.route(h.double(), w, "l%d.mlp." % n, mlp["router"]["top"])
        for t in range(17):
            assert ids[t].tolist() == [e for e, _ in want[t]]
            assert all(abs(float(a) - b) < 1e-5 for a, (_, b) in zip(wts[t], want[t]))
        # the bias moves the choice, not only the weights
        free = dict(w, **{"l%d.mlp.router.b" % n: torch.zeros(mlp["router"]["experts"], dtype=D)})
        if mlp["router"]["top"] < mlp["router"]["experts"]:
            other = oracle.route(h.double(), free, "l%d.mlp." % n, mlp["router"]["top"])
            assert any([e for e, _ in a] != [e for e, _ in b] for a, b in zip(want, other))


def test_logits_scale_and_cap():
    x = _rand(4, 9, scale=20.0)
    z = x.double() * 0.3
    torch.testing.assert_close(ops.softcap_logits(x, 0.3, 2.0).double(), 2.0 * torch.tanh(z / 2.0),
                               rtol=1e-5, atol=1e-6)
    torch.testing.assert_close(ops.softcap_logits(x, 0.3, 0.0).double(), z, rtol=1e-6, atol=1e-6)


def _meta(start, n, cache=None, table=None, bs=8, linear=None, slot=0):
    pos = torch.arange(start, start + n)
    bt = torch.tensor(table if table is not None else [0])
    prefill = not (n == 1 and start > 0)
    return ForwardMeta(
        is_prefill=prefill, positions=pos.int(),
        slot_mapping=bt[pos // bs] * bs + pos % bs if table is not None
        else torch.zeros(n, dtype=torch.long),
        block_tables=bt.int().unsqueeze(0),
        seq_lens=torch.tensor([start + n], dtype=torch.int32),
        query_lens=torch.tensor([n], dtype=torch.int32), mla_cache=cache,
        linear_cache=linear, linear_slots=torch.tensor([slot]))


def _mixer(spec, w, width=WIDTH):
    cfg = U.small_config([spec], width=width, loop=None)
    m = RunidraShardModel(ModelConfig.from_hf_config(cfg)).float()
    for k, v in w.items():
        m.load_hf_weight(k, v)
    m.finalize_weights()
    return m.float().layers[0].mixer


def _run_latent(m, spec, h, cuts, entry=0, bs=8):
    mx = spec["mixer"]
    pages = (h.shape[0] + bs - 1) // bs
    cache = MLAKVCache(2, [mx["kv_rank"]] * 2, [mx["rot_dim"]] * 2, bs, pages + 3,
                       torch.device("cpu"), torch.float32)
    for c in cache.caches:
        c.fill_(5.0)   # leftovers of earlier requests
    table = torch.randperm(pages + 3, generator=torch.Generator().manual_seed(9))[:pages].tolist()
    outs, at = [], 0
    for n in cuts:
        outs.append(m(h[at:at + n], _meta(at, n, cache, table, bs), entry))
        at += n
    assert at == h.shape[0]
    assert torch.all(cache.caches[1 - entry] == 5.0)   # the other pass's entry
    return torch.cat(outs)


def _run_mlstm(m, spec, h, cuts, entry=0):
    mx = spec["mixer"]
    lin = LinearStateCache(2, [(0,)] * 2,
                           [(mx["heads"], mlstm_state_width(mx["dim"], mx["vdim"]))] * 2, 3,
                           torch.device("cpu"), torch.float32)
    for s in lin.recurrent_states:
        s.fill_(9.0)
    outs, at = [], 0
    for n in cuts:
        outs.append(m(h[at:at + n], _meta(at, n, linear=lin, slot=2), entry))
        at += n
    assert at == h.shape[0]
    assert torch.all(lin.recurrent_states[entry][:2] == 9.0)
    assert torch.all(lin.recurrent_states[1 - entry] == 9.0)
    return torch.cat(outs), lin.recurrent_states[entry][2]


CUTS = [[150], [2, 5, 1, 1, 64, 3, 1, 40, 2, 31], [7] + [1] * 143]


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("heads,dim,vdim,cap", [(3, 12, 20, 6.0), (1, 8, 8, 1.0), (2, 5, 33, 20.0)])
def test_mlstm_alone_portions_and_slots(cuts, heads, dim, vdim, cap):
    spec = U.mlstm_layer(heads, dim, vdim, cap, None)
    w = oracle.random_weights(U.small_config([spec], loop=None), seed=7)
    m = _mixer(spec, w)
    assert isinstance(m, MLSTM)
    h = _rand(150, WIDTH, seed=3)
    want, ends = oracle.mlstm(h.double(), w, "l0.mix.", spec["mixer"], EPS, True)
    got, state = _run_mlstm(m, spec, h, cuts, entry=1)
    torch.testing.assert_close(got.double(), want, rtol=1e-3, atol=1e-3)
    for a, (S, n, mmax) in enumerate(ends):
        torch.testing.assert_close(state[a][: dim * vdim].view(dim, vdim).double(), S,
                                   rtol=1e-4, atol=1e-4)
        torch.testing.assert_close(state[a][dim * vdim:dim * vdim + dim].double(), n,
                                   rtol=1e-4, atol=1e-4)
        assert abs(float(state[a][dim * vdim + dim]) - mmax) < 1e-4


@pytest.mark.parametrize("cuts", CUTS)
def test_mlstm_keeps_a_far_token_and_its_maximum_starts_at_zero(cuts):
    """One early token with a wide-open input gate and forget gates near 1:
    140 tokens later it still fills the memory, so a lost state shows. With
    every input gate far below zero the denominator is exp(-m) of a maximum
    that started at 0: one that started at minus infinity would give unit-size
    results instead of none."""
    spec = U.mlstm_layer(2, 12, 8, 12.0, None)
    w = oracle.random_weights(U.small_config([spec], loop=None), seed=8)
    w["l0.mix.f.b"] = torch.full((2,), 9.0, dtype=D)
    w["l0.mix.f"] *= 0.0
    w["l0.mix.i"] *= 0.0
    w["l0.mix.i"][:, 0] = 6.0
    w["l0.mix.i.b"] = torch.full((2,), -6.0, dtype=D)
    h = _rand(150, WIDTH, seed=4)
    h[:, 0] = 0.0
    h[6, 0] = 3.0
    m = _mixer(spec, w)
    want = oracle.mlstm(h.double(), w, "l0.mix.", spec["mixer"], EPS)
    got, _ = _run_mlstm(m, spec, h, cuts)
    torch.testing.assert_close(got.double(), want, rtol=1e-3, atol=1e-3)
    lost = oracle.mlstm(h[20:].double(), w, "l0.mix.", spec["mixer"], EPS)
    assert (lost - want[20:]).abs().max() > 0.1
    # all gates shut: o is e^-6 small before the head norm's eps
    q, i, f = _rand(9, 12, seed=5).double(), torch.full((9,), -6.0, dtype=D), \
        torch.full((9,), -0.01, dtype=D)
    small = oracle.mlstm_cell(q, q, q, i, f)[0]
    assert small.abs().max() < 0.2
    st = torch.zeros(1, 1, mlstm_state_width(12, 12))
    zi, zf = 12 * math.atanh(-0.5), 12 * math.atanh(
        (-math.log(math.expm1(0.01))) / 12)
    gates = torch.tensor([[zi, zf]]).repeat(9, 1)
    got = ops.mlstm((q * 12 ** 0.5).float(), q.float(), q.float(), torch.full((9, 12), 60.0), gates,
                    torch.zeros(2), torch.ones(12), 12.0, 1.0, st, torch.tensor([0]),
                    torch.tensor([0, 9], dtype=torch.int32), torch.arange(9, dtype=torch.int32),
                    torch.float32)
    torch.testing.assert_close(got.double(), oracle.rms_norm(small, None, 1.0), rtol=1e-3, atol=1e-5)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("window,rank,rot_dim", [(9, 24, 12), (1, 8, 2), (64, 40, 16), (500, 20, 6)])
def test_latent_attention_alone_portions_and_pages(cuts, window, rank, rot_dim):
    spec = U.latent_layer(window=window, rank=rank, rot_dim=rot_dim, mlp=None)
    w = oracle.random_weights(U.small_config([spec], loop=None), seed=9)
    m = _mixer(spec, w)
    assert isinstance(m, LatentWindowAttention)
    h = _rand(150, WIDTH, seed=5)
    want = oracle.latent_attention(h.double(), w, "l0.mix.", spec["mixer"], EPS)
    got = _run_latent(m, spec, h, cuts, entry=1)
    torch.testing.assert_close(got.double(), want, rtol=1e-4, atol=1e-4)


def test_rotation_pairs_neighbours():
    x = _rand(6, 2, 8, seed=1)
    pos = torch.tensor([0, 1, 2, 50, 1000, 7])
    freq = torch.tensor([500.0 ** (-2.0 * i / 8) for i in range(4)])
    got = ops.rope_rows(x, 0, 8, freq, 1.0, 8, pos.int(), True)
    want = oracle.rotate_pairs(x.double(), pos, 500.0)
    torch.testing.assert_close(got.double(), want, rtol=1e-4, atol=1e-4)


def _planted(spec, at, n, seed):
    """Weights and inputs under which every query's score with the token `at`
    stands far above all others (through the unrotated part): returns (w, h)."""
    mx = spec["mixer"]
    w = oracle.random_weights(U.small_config([spec], loop=None), seed=seed)
    g = torch.Generator().manual_seed(seed)
    h = torch.randn(n, WIDTH, generator=g) * 0.3
    h[:, 0] = 0.0
    h[:, 1] = 2.0                   # what every query latent reads
    h[at, 0] = 6.0                  # what makes the planted key
    for name in ("dq", "dkv"):
        w["l0.mix." + name] *= 0.2
    w["l0.mix.dq"][0, :] = 0.0
    w["l0.mix.dq"][0, 1] = 4.0      # latent 0 of every query is large
    R = mx["kv_rank"]
    w["l0.mix.dkv"][0, :] = 0.0
    w["l0.mix.dkv"][0, 0] = 4.0     # latent 0 of the planted key is large
    H, d, r = mx["heads"], mx["dim"], mx["rot_dim"]
    uq = w["l0.mix.uq"].view(H, d + r, -1)
    uk = w["l0.mix.uk"].view(H, d, R)
    uq[:, 0, :] = 0.0
    uq[:, 0, 0] = 4.0
    uk[:, 0, :] = 0.0
    uk[:, 0, 0] = 4.0
    return {k: v.bfloat16().to(D) for k, v in w.items()}, h   # as a checkpoint holds them


@pytest.mark.parametrize("at", [0, 3, 7, 8, 40, 63])
@pytest.mark.parametrize("cuts", [[120], [50, 70], [41] + [1] * 79])
def test_window_edges(at, cuts):
    """A planted key takes almost the whole softmax: the queries at distances
    0 .. window - 1 see it, the one at `window` does not; at page borders and
    inside pages, in prompts and in decoding."""
    window = 24
    spec = U.latent_layer(window=window, scale=0.2, mlp=None)
    w, h = _planted(spec, at, 120, 11)
    mx = spec["mixer"]
    s, _ = oracle.latent_scores(h.double(), w, "l0.mix.", mx, EPS)
    a = oracle.sink_softmax(s, w["l0.mix.sink"], window)
    last = at + window - 1
    assert float(a[:, at, at].min()) > 0.9 and float(a[:, last, at].min()) > 0.9
    assert float(a[:, last + 1, at].max()) == 0.0
    want = oracle.latent_attention(h.double(), w, "l0.mix.", mx, EPS)
    # one token more or less in the window is far outside the tolerance
    for other in (window - 1, window + 1):
        moved = oracle.latent_attention(h.double(), w, "l0.mix.",
                                        dict(mx, mask={"size": other}), EPS)
        assert (moved - want).abs().max() > 0.05
    got = _run_latent(_mixer(spec, w), spec, h, cuts)
    torch.testing.assert_close(got.double(), want, rtol=1e-3, atol=1e-3)


def test_sink_takes_its_share_once():
    spec = U.latent_layer(window=40, mlp=None)
    w = oracle.random_weights(U.small_config([spec], loop=None), seed=12)
    h = _rand(60, WIDTH, seed=6)
    outs = []
    for sink in (-40.0, 0.0, 4.0, 40.0):
        w["l0.mix.sink"] = torch.full((3,), sink, dtype=D)
        want = oracle.latent_attention(h.double(), w, "l0.mix.", spec["mixer"], EPS)
        got = _run_latent(_mixer(spec, w), spec, h, [20, 1, 1, 2, 36])
        torch.testing.assert_close(got.double(), want, rtol=1e-4, atol=1e-4)
        outs.append(want)
    assert outs[3].abs().max() < 1e-6          # a huge sink leaves nothing
    assert (outs[0] - outs[1]).abs().max() > 0.05


# -- the engine: step function, cache manager, scheduler ----------------------------


def test_whole_prompt_and_layers(ckpt):
    cfg, w, path = ckpt
    eng = U.make_engine(path)
    toks = U.tokens(70, cfg["vocab"], 1)
    streams = {}
    eng.model.tap = lambda i, x: streams.__setitem__(i, x.clone())
    got = U.run_schedule(eng, {"a": toks}, [[("a", 70)]])["a"]
    want, layers = oracle.forward(cfg, w, toks, return_layers=True)
    assert len(streams) == len(layers) == 8
    for i, x in enumerate(layers):
        torch.testing.assert_close(streams[i].double(), x, rtol=2e-4, atol=2e-4)
    assert U.rel_err(got, want) < TOL


def test_looped_layers_share_weights(ckpt):
    _, _, path = ckpt
    eng = U.make_engine(path)
    assert len(eng.model.layers) == 5 and eng.model.num_local_layers == 8
    assert len(eng.kv_cache.caches) == 4
    assert len(eng.linear_cache.recurrent_states) == 4


def test_first_tokens_and_single_token_prompt(ckpt):
    cfg, w, path = ckpt
    eng = U.make_engine(path)
    for n in (1, 2, 3):
        toks = U.tokens(n, cfg["vocab"], 20 + n)
        got = U.run_schedule(eng, {"a": toks}, [[("a", n)]])["a"]
        assert U.rel_err(got, oracle.forward(cfg, w, toks)) < TOL


def test_prefill_equals_token_by_token_decoding(ckpt):
    cfg, w, path = ckpt
    toks = U.tokens(60, cfg["vocab"], 2)
    want = oracle.forward(cfg, w, toks)
    eng = U.make_engine(path)
    whole = U.run_schedule(eng, {"a": toks}, [[("a", 60)]])["a"]
    one = U.run_schedule(eng, {"b": toks}, [[("b", 1)] for _ in toks])["b"]
    assert U.rel_err(whole, want) < TOL and U.rel_err(one, want) < TOL


@pytest.mark.parametrize("cuts", [[2] * 40, [3, 2, 7, 1, 1, 1, 33, 2, 5, 25], [79, 1],
                                  [8, 8, 8, 8, 8, 8, 8, 8, 8, 8], [5, 1, 1, 1, 9, 1, 62]])
def test_portions_of_several_sizes(ckpt, cuts):
    cfg, w, path = ckpt
    assert sum(cuts) == 80
    toks = U.tokens(80, cfg["vocab"], 3)
    eng = U.make_engine(path)
    got = U.run_schedule(eng, {"a": toks}, [[("a", n)] for n in cuts])["a"]
    assert U.rel_err(got, oracle.forward(cfg, w, toks)) < TOL


def test_mixed_batches_of_unequal_requests(ckpt):
    cfg, w, path = ckpt
    seqs = {"a": U.tokens(90, cfg["vocab"], 4), "b": U.tokens(7, cfg["vocab"], 5),
            "c": U.tokens(41, cfg["vocab"], 6), "d": U.tokens(1, cfg["vocab"], 7),
            "e": U.tokens(30, cfg["vocab"], 8)}
    schedule = [
        [("a", 16), ("b", 1)],
        [("b", 1), ("a", 31), ("c", 2)],
        [("c", 1), ("b", 1), ("a", 1), ("d", 1)],          # d ends: e takes its slot
        [("e", 9), ("a", 1), ("b", 4), ("c", 30)],          # b ends
        [("a", 40), ("c", 1), ("e", 1)],
        [("e", 20), ("a", 1), ("c", 7)],
    ]
    eng = U.make_engine(path, pages=24, block_size=8)  # 192 tokens: pages are tight
    got = U.run_schedule(eng, seqs, schedule)
    for name, toks in seqs.items():
        assert got[name].shape[0] == len(toks)
        assert U.rel_err(got[name], oracle.forward(cfg, w, toks)) < TOL, name
    assert eng.cache_manager.num_free_blocks == 24


def test_pages_and_slots_freed_and_used_again(ckpt):
    cfg, w, path = ckpt
    eng = U.make_engine(path, pages=8, block_size=8, max_requests=2)
    for k in range(5):   # 5 requests through 8 pages and 2 state slots
        toks = U.tokens(50 + k, cfg["vocab"], 30 + k)
        cuts = [20, 1, 1] + [len(toks) - 22]
        got = U.run_schedule(eng, {"r%d" % k: toks}, [[("r%d" % k, n)] for n in cuts])
        assert U.rel_err(got["r%d" % k], oracle.forward(cfg, w, toks)) < TOL
        assert eng.cache_manager.num_free_blocks == 8
        # what a request leaves in its slot is not zero: the next owner must
        # not start from it
        assert any(float(s.abs().max()) > 0 for s in eng.linear_cache.recurrent_states)


def test_long_decoding_past_every_window(ckpt):
    cfg, w, path = ckpt
    toks = U.tokens(150, cfg["vocab"], 9)
    eng = U.make_engine(path)
    got = U.run_schedule(eng, {"a": toks}, [[("a", 12)]] + [[("a", 1)]] * 138)["a"]
    assert U.rel_err(got, oracle.forward(cfg, w, toks)) < TOL


@pytest.mark.parametrize("layers,streams,loop", [
    # one head, one stream, every width alike, one expert, a window of one
    ([U.mlstm_layer(1, 8, 8, 1.0, U.experts(1, 1, 8, 8)),
      U.latent_layer(1, 8, 8, 8, 8, 8, 1, 1.0, 10.0, U.dense(8))], 1, None),
    # attention only; every expert used by every token; one layer looped
    # three times; no feed-forward at the end
    ([U.latent_layer(2, 4, 2, 30, 10, 50, 70, mlp=U.experts(3, 3, 8, 40)),
      U.latent_layer(5, 12, 8, 4, 33, 3, 6, mlp=None)], 4, (0, 1, 3)),
    # recurrence only; the whole stack twice; five streams
    ([U.mlstm_layer(4, 6, 10, 30.0, None), U.mlstm_layer(2, 40, 3, 0.5, U.experts(7, 2, 12, 0))],
     5, (0, 2, 2)),
    # a loop that runs once and an empty one
    ([U.mlstm_layer(), U.latent_layer()], 2, (0, 1, 1)),
    ([U.latent_layer(), U.mlstm_layer()], 2, (1, 1, 4)),
])
def test_other_sizes(tmp_path, layers, streams, loop):
    cfg = U.small_config(layers, width=24, vocab=53, eps=1e-6, streams=streams, loop=loop,
                         logit_scale=1.0, softcap=30.0)
    w = oracle.random_weights(cfg, seed=17)
    path = U.write_checkpoint(str(tmp_path), cfg, w)
    toks = U.tokens(60, 53, 10)
    eng = U.make_engine(path)
    got = U.run_schedule(eng, {"a": toks}, [[("a", n)] for n in [6, 1, 1, 30, 2, 20]])["a"]
    assert U.rel_err(got, oracle.forward(cfg, w, toks)) < TOL


@pytest.mark.parametrize("cut", [1, 3, 5, 7])
def test_layer_ranges_hand_the_streams_on(ckpt, cut):
    """Two shards of the stack, run one after the other, give the whole
    stack's result, also when the cut falls between two passes of the loop or
    inside one: the fp32 streams travel between them."""
    cfg, w, path = ckpt
    mc = ModelConfig.from_pretrained(path)
    from parallax_amd.server.shard_loader import load_shard_weights

    toks = U.tokens(20, cfg["vocab"], 50)
    hidden = None
    for lo, hi in ((0, cut), (cut, 8)):
        m = RunidraShardModel(mc, lo, hi)
        load_shard_weights(m, path)
        m.finalize_weights()
        m = m.float()
        if lo == 0:
            hidden = m.embed(torch.tensor(toks))
        assert hidden.shape == (20, m.hidden_width) == (20, 3 * WIDTH)
        dims, shapes = mc.latent_cache_dims(lo, hi), mc.linear_state_shapes(lo, hi)
        cache = MLAKVCache(len(dims), [a for a, _ in dims], [b for _, b in dims], 8, 8,
                           torch.device("cpu"), torch.float32)
        lin = LinearStateCache(len(shapes), [c for c, _ in shapes], [r for _, r in shapes], 2,
                               torch.device("cpu"), torch.float32) if shapes else None
        hidden = m(hidden, _meta(0, 20, cache, list(range(8)), 8, lin, 1))
    assert U.rel_err(m.compute_logits(hidden), oracle.forward(cfg, w, toks)) < TOL


def _greedy(cfg, w, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(oracle.forward(cfg, w, seq)[-1].argmax()))
    return seq[len(prompt):]


def test_greedy_generation_through_the_scheduler(ckpt):
    cfg, w, path = ckpt
    eng = U.make_engine(path, prefill_chunk_size=16)
    prompts = [U.tokens(37, cfg["vocab"], 11), U.tokens(5, cfg["vocab"], 12),
               U.tokens(18, cfg["vocab"], 13)]
    ns = (8, 12, 7)
    sp = [SamplingParams(temperature=0.0, max_new_tokens=n, ignore_eos=True) for n in ns]
    out = list(eng.generate(prompts, sp).values())
    for p, n, got in zip(prompts, ns, out):
        assert got == _greedy(cfg, w, p, n)
    assert eng.cache_manager.num_free_blocks == 64


def test_two_peer_pipeline_greedy(ckpt):
    """The packet-driven multi-host path: two peers split the layer runs inside
    the loop's second pass, the streams travel between them."""
    from parallax_amd.p2p.peer_executor import PeerExecutor
    from parallax_amd.p2p.transport import LoopbackTransport

    cfg, w, path = ckpt
    mc = ModelConfig.from_pretrained(path)
    registry, peers = {}, []
    for pid, (s, e) in zip(["p0", "p1"], [(0, 5), (5, 8)]):
        peers.append(PeerExecutor(mc, s, e, pid, LoopbackTransport(pid, registry),
                                  dtype=torch.float32, num_kv_blocks=64, block_size=8,
                                  model_path=path))
    head = peers[0]
    prompts = [U.tokens(19, cfg["vocab"], 70), U.tokens(4, cfg["vocab"], 71)]
    sp = SamplingParams(temperature=0.0, max_new_tokens=5, ignore_eos=True)
    rids = [head.submit(p, sp, ["p0", "p1"]) for p in prompts]
    outputs, done = {r: [] for r in rids}, set()
    for _ in range(2000):
        for px in peers:
            px.step(recv_timeout=0.001)
        for out in head.drain_outputs():
            outputs[out.rid].append(out.token_id)
            if out.finished:
                done.add(out.rid)
        if len(done) == len(rids):
            break
    for p, rid in zip(prompts, rids):
        assert outputs[rid] == _greedy(cfg, w, p, 5)


def _pp_worker(rank, world, port, path, prompts, out_file):
    import os

    os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT=str(port),
                      RANK=str(rank), WORLD_SIZE=str(world))
    import torch.distributed as dist

    from parallax_amd.parallel.comm import init_distributed
    from parallax_amd.server.engine import Engine, EngineArgs

    comm = init_distributed(pp_size=world, tp_size=1, backend="gloo",
                            device=torch.device("cpu"))
    eng = Engine(ModelConfig.from_pretrained(path),
                 EngineArgs(block_size=8, num_kv_blocks=64, max_batch_size=4,
                            dtype=torch.float32, micro_batches=2,
                            enable_prefix_cache=False, max_model_len=512),
                 comm=comm, model_path=path)
    sp = [SamplingParams(temperature=0.0, max_new_tokens=4, ignore_eos=True)] * len(prompts)
    outs = list(eng.generate(prompts, sp).values())
    if rank == 0:
        torch.save(outs, out_file)
    dist.barrier()
    dist.destroy_process_group()


def test_pipeline_stages_over_gloo(ckpt, tmp_path):
    """Two pipeline stages in two processes (gloo): all streams cross the
    stage boundary, greedy tokens equal the reference's."""
    import torch.multiprocessing as mp

    cfg, w, path = ckpt
    prompts = [U.tokens(13, cfg["vocab"], 80), U.tokens(3, cfg["vocab"], 81),
               U.tokens(26, cfg["vocab"], 82)]
    out_file = str(tmp_path / "pp2.pt")
    mp.spawn(_pp_worker, args=(2, 29685, path, prompts, out_file), nprocs=2, join=True)
    for p, toks in zip(prompts, torch.load(out_file)):
        assert toks == _greedy(cfg, w, p, 4)


def test_trace_replay_program(ckpt, tmp_path):
    """bin/trace_run picks the model class from config.json; ended requests
    give their pages and state slots back."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np

    cfg, w, path = ckpt
    a, b = U.tokens(21, cfg["vocab"], 60), U.tokens(9, cfg["vocab"], 61)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:16], "want": [0, 15]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[16:17], "want": []},
                                {"id": "b", "tokens": b[:8], "want": [7]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[8:], "want": [0]},
                                {"id": "a", "tokens": a[17:], "want": [3]}], "end": ["a", "b"]},
    ]
    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "logits"
    p = subprocess.run(
        [sys.executable, os.path.join(repo, "bin", "trace_run"), "--model", path,
         "--dtype", "float32", "--out", str(out), "--max-tokens", "64", "--device", "cpu"],
        input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True,
        text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == \
        ["done 0", "done 1", "done 2"]
    V = cfg["vocab"]
    la, lb = oracle.forward(cfg, w, a), oracle.forward(cfg, w, b)
    got = torch.from_numpy(np.concatenate(
        [np.fromfile(out / ("%d.f32" % i), dtype="<f4").reshape(-1, V) for i in range(3)]))
    want = torch.stack([la[0], la[15], lb[7], lb[8], la[20]])
    assert U.rel_err(got, want) < TOL


def test_a_layer_module_reads_every_size_from_its_entry():
    mc = ModelConfig.from_hf_config(U.small_config())
    layer = RunidraLayer(mc, U.latent_layer(2, 6, 4, 10, 14, 18, 5))
    m = layer.mixer
    assert (m.heads, m.dn, m.dr, m.dv, m.rank, m.q_rank, m.window) == (2, 6, 4, 10, 14, 18, 5)
    assert m.q_up.weight.shape == (20, 18) and m.sink.shape == (2,)
