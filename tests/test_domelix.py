"""Domelix on the CPU engine (fp32) against the plain reference in
domelix_oracle.py: each mechanism alone, then the engine's step function, cache
manager, state slots and scheduler under many ways of cutting and batching the
same sequences. Configurations are small and deliberately irregular (see
domelix_util.small_config)."""

import pytest
import torch

import domelix_oracle as oracle
import domelix_util as U
from parallax_amd import ops
from parallax_amd.models.config import ModelConfig
from parallax_amd.models.domelix import DomelixLayer, DomelixShardModel
from parallax_amd.models.forward_meta import ForwardMeta
from parallax_amd.models.linear_attention import DecayLinearAttention, GatedDeltaRule
from parallax_amd.models.row_attention import DistanceBiasAttention, distance_buckets
from parallax_amd.server.kv_cache import LinearStateCache, MLAKVCache
from parallax_amd.server.sampling_params import SamplingParams

D = oracle.F64
# fp32 rounding: head norms magnify it where the sum before them cancels
TOL = 2e-4
WIDTH = 40
EPS = 1e-5


@pytest.fixture(scope="module")
def ckpt(tmp_path_factory):
    cfg = U.small_config()
    w = oracle.random_weights(cfg, seed=3)
    path = U.write_checkpoint(str(tmp_path_factory.mktemp("dx")), cfg, w)
    return cfg, w, path


def _rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


# -- mechanisms alone --------------------------------------------------------------


def test_config_reader():
    cfg = U.small_config()
    mc = ModelConfig.from_hf_config(cfg)
    assert mc.architecture == "Domelix" and mc.num_layers == 5
    assert mc.layer_types == ["linear_attention", "parallel_attention_recurrent",
                              "linear_attention", "parallel_attention_recurrent",
                              "linear_attention"]
    # rows for the parallel layers only, a state for every layer
    assert mc.latent_cache_dims(0, 5) == [(12, 20), (16, 12)]
    assert mc.latent_cache_dims(2, 4) == [(16, 12)]
    assert mc.pooled_cache_blocks(0, 5) == [0, 0]
    assert mc.linear_state_shapes(0, 5) == [
        ((2 * 24 + 36, 3), (4, 12, 9)), ((0,), (2, 10, 14)), ((0,), (3, 14, 22)),
        ((0,), (3, 6, 5)), ((2 * 20 + 48, 2), (3, 20, 16))]
    assert mc.has_linear_layers
    assert (mc.num_experts, mc.num_experts_per_tok, mc.n_group, mc.topk_group) == (6, 2, 3, 2)
    with pytest.raises(ValueError):
        ModelConfig.from_hf_config(U.small_config([{"type": "gla", "mixer": {}, "mlp": None}]))
    bad = U.retention_layer(mlp={"kind": "dense", "ff": 8})
    with pytest.raises(ValueError):
        ModelConfig.from_hf_config(U.small_config([bad]))


def test_bad_sizes_are_refused():
    for spec in (U.retention_layer(mlp=U.experts(6, 3, 8, (3, 1))),    # 3 of 2 experts
                 U.retention_layer(mlp=U.experts(7, 2, 8, (3, 1))),    # unequal groups
                 U.retention_layer(heads=3, decay=[0.5, 0.5]),
                 U.retention_layer(dim=6, dims=8),
                 U.delta_layer(heads=5, kv_heads=2),
                 U.parallel_layer(U.left(heads=5, kv_heads=2))):
        with pytest.raises(ValueError):
            DomelixShardModel(ModelConfig.from_hf_config(U.small_config([spec])))


def test_residual_step():
    T, W = 5, 12
    x, a, b, f = (_rand(T, W, seed=s, scale=s) for s in (1, 2, 3, 4))
    wa, wb, w1, w2 = (_rand(W, seed=s) for s in (5, 6, 7, 8))
    d = lambda t: t.double()
    m = (oracle.unit_rms(d(a), EPS) * d(wa) + oracle.unit_rms(d(b), EPS) * d(wb)) / 2
    for args, add in (((a, b, wa, wb, 0.5, f), m + d(f)), ((a, None, None, None, 1.0, f), d(a) + d(f)),
                      ((a, b, wa, wb, 0.5, None), m), ((None, None, None, None, 1.0, None), 0 * m)):
        y = x.clone()
        h1, h2 = ops.parallel_rmsnorm_add(y, *args, w1, w2, EPS, 1.0, torch.float32)
        want = d(x) + add
        torch.testing.assert_close(d(y), want, rtol=1e-5, atol=1e-5)
        torch.testing.assert_close(d(h1), oracle.norm_about_one(want, d(w1), EPS), rtol=1e-5, atol=1e-5)
        torch.testing.assert_close(d(h2), oracle.norm_about_one(want, d(w2), EPS), rtol=1e-5, atol=1e-5)


@pytest.mark.parametrize("rows,limit", [(10, 50), (6, 17), (30, 128), (2, 2), (2, 9), (8, 64), (9, 30),
                                        (16, 9), (10, 160)])
def test_distance_buckets(rows, limit):
    got = distance_buckets(rows, limit).tolist()
    assert len(got) == limit + 1
    assert got == [oracle.bucket(n, rows, limit) for n in range(limit + 1)]
    assert got == sorted(got) and got[0] == 0 and got[-1] == rows - 1
    assert got[: rows // 2] == list(range(rows // 2))
    assert oracle.bucket(10 * limit, rows, limit) == rows - 1
    with pytest.raises(ValueError):
        distance_buckets(rows, rows // 2)


def test_feed_forward_and_grouped_router():
    cfg = U.small_config([U.retention_layer(mlp=U.experts(6, 2, 20, (3, 1))),
                          U.retention_layer(mlp=U.experts(8, 3, 12, (2, 1))),
                          U.retention_layer(mlp=U.experts(4, 4, 8, None)),
                          U.retention_layer(mlp=U.experts(5, 1, 8, (5, 3)))])
    w = oracle.random_weights(cfg, seed=5)
    m = _model(cfg, w)
    h = _rand(40, WIDTH, seed=2)
    for n in range(4):
        mlp, p = cfg["layers"][n]["mlp"], "l%d.mlp." % n
        torch.testing.assert_close(m.layers[n].mlp(h).double(), oracle.moe(h.double(), w, p, mlp),
                                   rtol=1e-4, atol=1e-4)
        ids, wts = m.layers[n].mlp.router(h)
        want = oracle.route(h.double(), w, p, mlp["router"])
        free = oracle.route(h.double(), w, p, dict(mlp["router"], groups=None))
        for t in range(40):
            assert ids[t].tolist() == [e for e, _ in want[t]]
            assert all(abs(float(a) - b) < 1e-5 for a, (_, b) in zip(wts[t], want[t]))
        if n < 2:    # the groups matter
            assert any([e for e, _ in a] != [e for e, _ in b] for a, b in zip(want, free))


def _as_stored(w):
    """Weights as a checkpoint holds them (bf16), after a test has changed some."""
    return {k: v.bfloat16().to(D) for k, v in w.items()}


def _model(cfg, w):
    m = DomelixShardModel(ModelConfig.from_hf_config(cfg)).float()
    for k, v in w.items():
        assert m.load_hf_weight(k, v), k
    m.finalize_weights()
    return m.float()


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


def _run(m, cfg, h, cuts, bs=8):
    """The first layer's mixer over h in portions: dirty slots and pages, a
    shuffled block table. Returns (its result; a pair for 'parallel', the state
    it leaves)."""
    mc = ModelConfig.from_hf_config(cfg)
    dims, shapes = mc.latent_cache_dims(0, 1), mc.linear_state_shapes(0, 1)
    pages = (h.shape[0] + bs - 1) // bs
    cache = MLAKVCache(len(dims), [a for a, _ in dims], [b for _, b in dims], bs, pages + 3,
                       torch.device("cpu"), torch.float32)
    for c in cache.caches:
        c.fill_(5.0)   # leftovers of earlier requests
    lin = LinearStateCache(1, [shapes[0][0]], [shapes[0][1]], 3, torch.device("cpu"), torch.float32)
    for s in lin.recurrent_states + lin.conv_states:
        s.fill_(9.0)
    table = torch.randperm(pages + 3, generator=torch.Generator().manual_seed(9))[:pages].tolist()
    outs, at = [], 0
    for n in cuts:
        y = m.layers[0].mixer(h[at:at + n], _meta(at, n, cache, table, bs, lin, 2))
        outs.append(y if isinstance(y, tuple) else (y,))
        at += n
    assert at == h.shape[0]
    assert torch.all(lin.recurrent_states[0][:2] == 9.0)
    assert torch.all(lin.conv_states[0][:2] == 9.0)
    return tuple(torch.cat(t) for t in zip(*outs)), lin.recurrent_states[0][2]


CUTS = [[150], [2, 5, 1, 1, 64, 3, 1, 40, 2, 31], [7] + [1] * 143]


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, dim=6, vdim=6, dims=6, decay=[1.0]),
                                dict(heads=2, dim=9, vdim=30, dims=0), dict(dim=16, dims=16, base=1e6)])
def test_retention_alone(cuts, kw):
    spec = U.retention_layer(mlp=None, **kw)
    cfg = U.small_config([spec])
    w = oracle.random_weights(cfg, seed=7)
    m, h = _model(cfg, w), _rand(150, WIDTH, seed=3)
    assert isinstance(m.layers[0].mixer, DecayLinearAttention)
    want, ends = oracle.retention(h.double(), w, "l0.mix.", spec["mixer"], EPS, True)
    (got,), state = _run(m, cfg, h, cuts)
    torch.testing.assert_close(got.double(), want, rtol=1e-3, atol=1e-3)
    for a, S in enumerate(ends):
        torch.testing.assert_close(state[a].double(), S, rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("lf,rt", [
    (U.left(), U.right()), (U.left(4, 4, 6, 6, 1.0, 3, 4), U.right(1, 5, 5, [0.9])),
    (U.left(6, 2, 9, 4, 0.1, 400, 32), U.right(3, 4, 12, [0.0, 1.0, 0.3]))])
def test_parallel_alone(cuts, lf, rt):
    spec = U.parallel_layer(lf, rt, None)
    cfg = U.small_config([spec])
    w = oracle.random_weights(cfg, seed=9)
    m, h = _model(cfg, w), _rand(150, WIDTH, seed=5)
    assert isinstance(m.layers[0].mixer.left, DistanceBiasAttention)
    (a, b), state = _run(m, cfg, h, cuts)
    torch.testing.assert_close(a.double(), oracle.bias_attention(h.double(), w, "l0.mix.left.", lf),
                               rtol=1e-4, atol=1e-4)
    want, ends = oracle.lightning(h.double(), w, "l0.mix.right.", rt, EPS, True)
    torch.testing.assert_close(b.double(), want, rtol=1e-3, atol=1e-3)
    for i, S in enumerate(ends):
        torch.testing.assert_close(state[i].double(), S, rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=5, vdim=5, conv=1),
                                dict(heads=6, kv_heads=2, dim=8, vdim=4, conv=2),
                                dict(heads=3, kv_heads=1, dim=7, vdim=30, conv=6)])
def test_delta_alone(cuts, kw):
    spec = U.delta_layer(mlp=None, **kw)
    cfg = U.small_config([spec])
    w = oracle.random_weights(cfg, seed=11)
    m, h = _model(cfg, w), _rand(150, WIDTH, seed=6)
    assert isinstance(m.layers[0].mixer, GatedDeltaRule)
    want, ends = oracle.delta(h.double(), w, "l0.mix.", spec["mixer"], EPS, True)
    (got,), state = _run(m, cfg, h, cuts)
    torch.testing.assert_close(got.double(), want, rtol=1e-3, atol=1e-3)
    for a, S in enumerate(ends):
        torch.testing.assert_close(state[a].double(), S, rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("kind", ["retention", "delta"])
def test_states_keep_a_far_token(cuts, kind):
    """One early token writes a key no later token comes near, decays stay next
    to 1, and only the last tokens ask for it: what they read has crossed every
    portion's border in the state."""
    if kind == "retention":
        spec = U.retention_layer(2, 12, 8, 0, decay=[1.0, 0.9999], mlp=None)
    else:
        spec = U.delta_layer(2, 2, 12, 8, 4, None)
    cfg = U.small_config([spec])
    w = oracle.random_weights(cfg, seed=8)
    p, d = "l0.mix.", 12
    for x in ("q", "k"):
        w[p + x] *= 0.1
        for a in range(2):
            w[p + x][a * d] = 0.0
            w[p + x][a * d, 0 if x == "k" else 1] = 8.0
    if kind == "delta":
        w[p + "a"] *= 0.0
        w[p + "dt_bias"] = torch.full((2,), -12.0, dtype=D)
        w[p + "b"] *= 0.0
        for x in "qkv":
            w[p + x + ".conv"] *= 0.0
            w[p + x + ".conv"][:, -1] = 1.0
    w = _as_stored(w)
    h = _rand(150, WIDTH, seed=4)
    h[:, :2] = 0.0
    h[6, 0] = 6.0
    h[100:, 1] = 6.0
    fn = getattr(oracle, kind)
    want = fn(h.double(), w, p, spec["mixer"], EPS)
    (got,), _ = _run(_model(cfg, w), cfg, h, cuts)
    torch.testing.assert_close(got.double(), want, rtol=1e-3, atol=1e-3)
    lost = fn(h[20:].double(), w, p, spec["mixer"], EPS)
    assert (lost[80:] - want[100:]).abs().max() > 0.1


@pytest.mark.parametrize("cut", [1, 2, 3, 5, 9])
def test_the_convolution_reads_across_portions(cut):
    """Taps that look 3 tokens back and nowhere else: the first tokens of a
    portion take their input from the one before (or several before, when a
    portion is shorter than the window)."""
    spec = U.delta_layer(2, 1, 8, 8, 4, None)
    cfg = U.small_config([spec])
    w = oracle.random_weights(cfg, seed=12)
    for x in "qkv":
        w["l0.mix." + x + ".conv"] *= 0.0
        w["l0.mix." + x + ".conv"][:, 0] = 1.5
    h = _rand(30, WIDTH, seed=7)
    want = oracle.delta(h.double(), w, "l0.mix.", spec["mixer"], EPS)
    cuts = [12] + [cut] * (18 // cut) + ([18 % cut] if 18 % cut else [])
    (got,), _ = _run(_model(cfg, w), cfg, h, cuts)
    torch.testing.assert_close(got.double(), want, rtol=1e-3, atol=1e-3)


def _planted(at, n, seed, bias_far):
    """A left mixer whose every query scores far above all others on the token
    `at`, and whose bias table adds `bias_far` to its last row only."""
    lf = U.left(2, 1, 8, 6, 0.25, 40, 8)
    spec = U.parallel_layer(lf, None, None)
    cfg = U.small_config([spec])
    w = oracle.random_weights(cfg, seed=seed)
    p = "l0.mix.left."
    h = _rand(n, WIDTH, seed=seed, scale=0.3)
    h[:, 0] = 0.0
    h[:, 1] = 2.0                # what every query reads
    h[at, 0] = 6.0               # what makes the planted key
    for x in ("q", "k"):
        w[p + x] *= 0.2
    for a in range(2):
        w[p + "q"][a * 8] = 0.0
        w[p + "q"][a * 8, 1] = 4.0
    w[p + "k"][0] = 0.0
    w[p + "k"][0, 0] = 4.0
    w[p + "rel"] = torch.zeros_like(w[p + "rel"])
    w[p + "rel"][-1] = bias_far
    w[p + "sink"] = torch.full((2,), 20.0, dtype=D)
    return cfg, lf, _as_stored(w), h


@pytest.mark.parametrize("at", [0, 3, 7, 8, 40, 63])
@pytest.mark.parametrize("cuts", [[150], [50, 70, 30], [41] + [1] * 109])
def test_far_keys_and_the_last_bucket(at, cuts):
    """The planted key (score about 48) stands against a sink of 20. With -56 on
    the last bucket it is seen up to the last distance before that bucket and
    not from there on: the bucket's first distance shows, in prompts and in
    decoding, at page borders and inside pages; with 0 it is seen to the end."""
    p = "l0.mix.left."
    for far in (0.0, -56.0):
        cfg, lf, w, h = _planted(at, 150, 13, far)
        a = oracle.sink_weights(oracle.bias_scores(h.double(), w, p, lf), w[p + "sink"])
        edge = min(n for n in range(200) if oracle.bucket(n, 8, 40) == 7)
        assert 20 < edge < 40
        assert float(a[:, at:min(150, at + edge), at].min() if at + edge <= 150 else 1.0) > 0.9
        beyond = a[:, at + edge:, at]
        assert float(beyond.max()) < 1e-3 if far else float(beyond.min()) > 0.9
        want = oracle.bias_attention(h.double(), w, p, lf)
        (got, _), _ = _run(_model(cfg, w), cfg, h, cuts)
        torch.testing.assert_close(got.double(), want, rtol=1e-3, atol=1e-3)
        if far:   # the table read with another limit gives something else
            moved = oracle.bias_attention(h.double(), w, p, dict(lf, bias_max=43))
            assert (moved - want).abs().max() > 0.05


def test_bias_is_not_scaled_and_every_head_has_its_own():
    lf = U.left(2, 1, 8, 6, 0.05, 12, 6)
    cfg = U.small_config([U.parallel_layer(lf, None, None)])
    w = oracle.random_weights(cfg, seed=14)
    w["l0.mix.left.rel"] *= 4.0     # exact in bf16
    h = _rand(40, WIDTH, seed=8)
    want = oracle.bias_attention(h.double(), w, "l0.mix.left.", lf)
    (got, _), _ = _run(_model(cfg, w), cfg, h, [20, 1, 1, 2, 16])
    torch.testing.assert_close(got.double(), want, rtol=1e-4, atol=1e-4)
    for k in (0.05, None):
        other = dict(w)
        other["l0.mix.left.rel"] = w["l0.mix.left.rel"] * k if k else w["l0.mix.left.rel"].flip(1)
        assert (oracle.bias_attention(h.double(), other, "l0.mix.left.", lf) - want).abs().max() > 0.05


def test_sink_takes_its_share_once():
    lf = U.left()
    cfg = U.small_config([U.parallel_layer(lf, None, None)])
    w = oracle.random_weights(cfg, seed=15)
    h = _rand(60, WIDTH, seed=9)
    outs = []
    for sink in (-40.0, 0.0, 4.0, 40.0):
        w["l0.mix.left.sink"] = torch.full((3,), sink, dtype=D)
        want = oracle.bias_attention(h.double(), w, "l0.mix.left.", lf)
        (got, _), _ = _run(_model(cfg, w), cfg, h, [20, 1, 1, 2, 36])
        torch.testing.assert_close(got.double(), want, rtol=1e-4, atol=1e-4)
        outs.append(want)
    assert outs[3].abs().max() < 1e-6          # a huge sink leaves nothing
    assert (outs[0] - outs[1]).abs().max() > 0.05


def test_rotation_pairs_halves():
    x = _rand(6, 2, 10, seed=1)
    pos = torch.tensor([0, 1, 2, 50, 1000, 7])
    freq = torch.tensor([500.0 ** (-2.0 * i / 8) for i in range(4)])
    cs = ops.rope_table(pos.int(), freq)
    st = torch.zeros(6, 2, 10, 10)
    # decay 0 and unit values: o = (q . k) v with k the rotated unit vectors
    want = oracle.rotate_halves(x.double(), pos, 500.0, 8)
    for i in range(10):
        k = torch.zeros(6, 2, 10)
        k[..., i] = 1.0
        kr = oracle.rotate_halves(k.double(), pos, 500.0, 8)
        got = ops.decay_attention(x, k, torch.ones(6, 2, 10), ops.decay_powers([0.0, 0.0]), 0.5,
                                  False, cs, st, torch.arange(6), None, pos.int())
        torch.testing.assert_close(got[..., 0].double(), (want * kr).sum(-1) / 2, rtol=1e-4, atol=1e-4)


# -- the engine: step function, cache manager, scheduler ----------------------------


def test_whole_prompt_and_layers(ckpt):
    cfg, w, path = ckpt
    eng = U.make_engine(path)
    toks = U.tokens(70, cfg["vocab"], 1)
    streams = {}
    eng.model.tap = lambda i, x: streams.__setitem__(i, x.clone())
    got = U.run_schedule(eng, {"a": toks}, [[("a", 70)]])["a"]
    want, layers = oracle.forward(cfg, w, toks, return_layers=True)
    assert len(streams) == len(layers) == 5
    for i, x in enumerate(layers):
        torch.testing.assert_close(streams[i].double(), x, rtol=2e-4, atol=2e-4)
    assert U.rel_err(got, want) < TOL
    assert len(eng.kv_cache.caches) == 2 and len(eng.linear_cache.recurrent_states) == 5


def test_first_tokens_and_single_token_prompt(ckpt):
    cfg, w, path = ckpt
    eng = U.make_engine(path)
    for n in (1, 2, 3, 4, 5):
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
        for kept in (eng.linear_cache.recurrent_states, eng.linear_cache.conv_states):
            assert any(s.numel() and float(s.abs().max()) > 0 for s in kept)


def test_long_decoding(ckpt):
    cfg, w, path = ckpt
    toks = U.tokens(150, cfg["vocab"], 9)
    eng = U.make_engine(path)
    got = U.run_schedule(eng, {"a": toks}, [[("a", 12)]] + [[("a", 1)]] * 138)["a"]
    assert U.rel_err(got, oracle.forward(cfg, w, toks)) < TOL


@pytest.mark.parametrize("layers", [
    # one head, every width alike, one expert, a convolution of one tap
    [U.parallel_layer(U.left(1, 1, 8, 8, 1.0, 2, 2), U.right(1, 8, 8, [1.0]), U.experts(1, 1, 8, None)),
     U.delta_layer(1, 1, 8, 8, 1, U.experts(1, 1, 8, (1, 1))),
     U.retention_layer(1, 8, 8, 8, 10.0, [0.5], U.experts(2, 2, 8, (2, 2)))],
    # recurrent layers only; every expert used by every token
    [U.retention_layer(5, 4, 30, 2, 10.0, mlp=U.experts(3, 3, 8, None)),
     U.delta_layer(6, 2, 3, 10, 7, None)],
    # parallel layers only, no feed-forward anywhere
    [U.parallel_layer(U.left(6, 3, 10, 4, 0.2, 200, 40), U.right(4, 3, 9), None),
     U.parallel_layer(U.left(2, 2, 4, 30, 2.0, 5, 8), U.right(1, 20, 2), None)],
    # one layer of each kind alone
    [U.delta_layer()], [U.retention_layer()], [U.parallel_layer()],
])
def test_other_sizes(tmp_path, layers):
    cfg = U.small_config(layers, width=24, vocab=53, eps=1e-6)
    w = oracle.random_weights(cfg, seed=17)
    path = U.write_checkpoint(str(tmp_path), cfg, w)
    toks = U.tokens(60, 53, 10)
    eng = U.make_engine(path)
    got = U.run_schedule(eng, {"a": toks}, [[("a", n)] for n in [6, 1, 1, 30, 2, 20]])["a"]
    assert U.rel_err(got, oracle.forward(cfg, w, toks)) < TOL


@pytest.mark.parametrize("cut", [1, 2, 4])
def test_layer_ranges_hand_the_stream_on(ckpt, cut):
    """Two shards of the stack, run one after the other, give the whole stack's
    result: the fp32 stream travels between them."""
    cfg, w, path = ckpt
    mc = ModelConfig.from_pretrained(path)
    from parallax_amd.server.shard_loader import load_shard_weights

    toks = U.tokens(20, cfg["vocab"], 50)
    hidden = None
    for lo, hi in ((0, cut), (cut, 5)):
        m = DomelixShardModel(mc, lo, hi)
        load_shard_weights(m, path)
        m.finalize_weights()
        m = m.float()
        if lo == 0:
            hidden = m.embed(torch.tensor(toks))
        dims, shapes = mc.latent_cache_dims(lo, hi), mc.linear_state_shapes(lo, hi)
        cache = MLAKVCache(len(dims), [a for a, _ in dims], [b for _, b in dims], 8, 8,
                           torch.device("cpu"), torch.float32)
        lin = LinearStateCache(len(shapes), [c for c, _ in shapes], [r for _, r in shapes], 2,
                               torch.device("cpu"), torch.float32)
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
    """The packet-driven multi-host path: two peers split the stack, the fp32
    stream travels between them."""
    from parallax_amd.p2p.peer_executor import PeerExecutor
    from parallax_amd.p2p.transport import LoopbackTransport

    cfg, w, path = ckpt
    mc = ModelConfig.from_pretrained(path)
    registry, peers = {}, []
    for pid, (s, e) in zip(["p0", "p1"], [(0, 2), (2, 5)]):
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
    """Two pipeline stages in two processes (gloo): the fp32 stream crosses the
    stage boundary, greedy tokens equal the reference's."""
    import torch.multiprocessing as mp

    cfg, w, path = ckpt
    prompts = [U.tokens(13, cfg["vocab"], 80), U.tokens(3, cfg["vocab"], 81),
               U.tokens(26, cfg["vocab"], 82)]
    out_file = str(tmp_path / "pp2.pt")
    mp.spawn(_pp_worker, args=(2, 29687, path, prompts, out_file), nprocs=2, join=True)
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
    m = DomelixLayer(mc, U.delta_layer(6, 2, 5, 7, 3, None), 0, 0).mixer
    assert (m.heads, m.kv_heads, m.dim, m.vdim) == (6, 2, 5, 7)
    assert m.conv_weight.shape == (20 + 42, 3) and m.gate_weight.shape == (12, WIDTH)
    m = DomelixLayer(mc, U.parallel_layer(U.left(6, 3, 4, 5), U.right(2, 7, 9)), 4, 2).mixer
    assert m.left.cache_layer_idx == 4 and m.right.state_layer_idx == 2
    assert m.in_proj.weight.shape == (24 + 12 + 15 + 30 + 14 + 14 + 18 + 18, WIDTH)
