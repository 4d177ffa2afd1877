"""Domelix on the GPU engine (HIP kernels, bf16 and float32) against the plain
reference in domelix_oracle.py: mixed batches, portions, decoding through
hipGraphs, pages and state slots used again, irregular sizes, greedy
generation."""

import pytest
import torch

import domelix_oracle as oracle
import domelix_util as U
from parallax_amd import ops
from parallax_amd.server.sampling_params import SamplingParams

pytestmark = pytest.mark.gpu

TOL = {torch.float32: 3e-4, torch.bfloat16: 0.08}
BOTH = [torch.float32, torch.bfloat16]


def close(got, want, dtype) -> bool:
    """float32: every row within rounding of the float64 reference. bfloat16:
    router near-ties and head norms over cancelling sums make single rows far
    more sensitive to rounding than the rest, and a flipped choice stays in the
    recurrent state: 85 rows in 100 within 0.08 and the median under 0.04;
    same() is the sharp bf16 check."""
    if dtype == torch.bfloat16:
        e = U.row_errs(got, want)
        few = e.numel() < 8          # a median of a handful of rows says little
        return bool((e < TOL[dtype]).double().mean() >= 0.85
                    and (few or e.median() < 0.04))
    return U.rel_err(got, want) < TOL[dtype]


def same(got, whole, dtype) -> bool:
    """A schedule against the same dtype's whole prompt: the same arithmetic up
    to the order of sums (bf16: nine rows in ten within 0.05, where a sum's
    order can move a rounding to bf16)."""
    if dtype == torch.float32:
        return U.same_as_whole(got, whole, 1e-3)
    return bool((U.row_errs(got, whole) < 0.05).double().mean() >= 0.9)


def _weights(cfg, seed):
    w = oracle.random_weights(cfg, seed=seed)
    for k in w:
        if k.endswith("router"):
            # well-separated experts: bf16 rounding seldom flips a choice (the
            # float32 runs and the kernel tests route by the inputs)
            w[k] = (w[k] * 3).bfloat16().to(oracle.F64)
    return w


@pytest.fixture(scope="module")
def ckpt(tmp_path_factory):
    # widths on the vector paths (multiples of 8) and off them, expert widths the
    # grouped-GEMM kernels tile (32, 96)
    layers = [
        U.delta_layer(mlp=U.experts(6, 2, 32)),
        U.parallel_layer(mlp=U.experts(4, 3, 96, None)),
        U.retention_layer(2, 40, 72, 24, mlp=None),
        U.parallel_layer(U.left(4, 2, 16, 24, 0.4, 33, 8), U.right(3, 8, 16), U.experts(8, 1, 64, (4, 1))),
        U.delta_layer(3, 1, 16, 16, 3, U.experts(6, 2, 32)),
    ]
    cfg = U.small_config(layers, width=64, vocab=136)
    w = _weights(cfg, 3)
    path = U.write_checkpoint(str(tmp_path_factory.mktemp("dxg")), cfg, w)
    return cfg, w, path


SEQS = {"a": (90, 4), "b": (7, 5), "c": (41, 6), "d": (1, 7), "e": (30, 8)}
SCHEDULE = [
    [("a", 16), ("b", 1)],
    [("b", 1), ("a", 31), ("c", 2)],
    [("c", 1), ("b", 1), ("a", 1), ("d", 1)],
    [("e", 9), ("a", 1), ("b", 4), ("c", 30)],
    [("a", 40), ("c", 1), ("e", 1)],
    [("e", 20), ("a", 1), ("c", 7)],
]


@pytest.mark.parametrize("dtype,graphs", [(torch.float32, False), (torch.bfloat16, False),
                                          (torch.bfloat16, True)])
def test_mixed_batches(ckpt, dtype, graphs):
    cfg, w, path = ckpt
    assert ops.has_mix_extension()
    seqs = {k: U.tokens(n, cfg["vocab"], s) for k, (n, s) in SEQS.items()}
    eng = U.make_engine(path, device="cuda", dtype=dtype, pages=24, graphs=graphs)
    assert (eng.graph_runner is not None) == graphs
    got = U.run_schedule(eng, seqs, SCHEDULE)
    alone = U.make_engine(path, device="cuda", dtype=dtype, pages=24)
    for name, toks in seqs.items():
        want = oracle.forward(cfg, w, toks)
        assert close(got[name], want, dtype), (name, U.describe(got[name], want, TOL[dtype]))
        whole = U.run_schedule(alone, {name: toks}, [[(name, len(toks))]])[name]
        assert same(got[name], whole, dtype), (name, U.describe(got[name], whole, 0.1))
    assert eng.cache_manager.num_free_blocks == 24


@pytest.mark.parametrize("dtype", BOTH)
def test_portions_decoding_and_reuse(ckpt, dtype):
    cfg, w, path = ckpt
    eng = U.make_engine(path, device="cuda", dtype=dtype, pages=20, max_requests=2,
                        graphs=dtype == torch.bfloat16)
    alone = U.make_engine(path, device="cuda", dtype=dtype, pages=20)
    for k, cuts in enumerate([[150], [2] * 20 + [1] * 60, [3, 2, 7, 1, 1, 1, 33, 2, 5, 45],
                              [12] + [1] * 128]):
        toks = U.tokens(sum(cuts), cfg["vocab"], 40 + k)
        got = U.run_schedule(eng, {"r": toks}, [[("r", n)] for n in cuts])["r"]
        want = oracle.forward(cfg, w, toks)
        assert close(got, want, dtype), (cuts[:3], U.describe(got, want, TOL[dtype]))
        whole = U.run_schedule(alone, {"w": toks}, [[("w", len(toks))]])["w"]
        assert same(got, whole, dtype), (cuts[:3], U.describe(got, whole, 0.1))
        assert eng.cache_manager.num_free_blocks == 20


def test_cutting_changes_nothing_beyond_rounding(ckpt):
    cfg, w, path = ckpt
    toks = U.tokens(100, cfg["vocab"], 50)
    eng = U.make_engine(path, device="cuda", dtype=torch.float32)
    whole = U.run_schedule(eng, {"a": toks}, [[("a", 100)]])["a"]
    cut = U.run_schedule(eng, {"b": toks}, [[("b", n)] for n in [37, 1, 1, 2, 59]])["b"]
    assert U.rel_err(cut, whole.double()) < 1e-4


@pytest.mark.parametrize("dtype", BOTH)
def test_sizes_outside_the_tuned_paths(tmp_path, dtype):
    """A width, vocabulary, head and expert sizes that are no multiples of 8:
    vendor's plain GEMM, scalar paths of the kernels, per-expert loop (decode
    then runs eagerly)."""
    layers = [U.delta_layer(5, 1, 10, 6, 5, U.experts(3, 2, 14, None)),
              U.parallel_layer(U.left(5, 5, 11, 10, 0.3, 7, 5), U.right(1, 21, 9), None),
              U.retention_layer(3, 9, 5, 6, 40.0, mlp=U.experts(6, 1, 20, (2, 1)))]
    cfg = U.small_config(layers, width=46, vocab=53)
    w = _weights(cfg, 17)
    path = U.write_checkpoint(str(tmp_path), cfg, w)
    eng = U.make_engine(path, device="cuda", dtype=dtype, graphs=dtype == torch.bfloat16)
    assert eng.graph_runner is None     # the per-expert loop reads the routing on the host
    toks = U.tokens(75, 53, 10)
    got = U.run_schedule(eng, {"a": toks},
                         [[("a", n)] for n in [6, 1, 1, 30, 2, 5] + [1] * 30])["a"]
    want = oracle.forward(cfg, w, toks)
    assert close(got, want, dtype), U.describe(got, want, TOL[dtype])


@pytest.mark.parametrize("dtype", BOTH)
def test_long_contexts_and_wide_heads(tmp_path, dtype):
    """Head widths of a real model's size, one above the chunked kernels' widest,
    contexts of many pages and chunks."""
    layers = [U.delta_layer(4, 2, 128, 128, 4, U.experts(6, 2, 96)),
              U.parallel_layer(U.left(8, 2, 64, 128, 0.12, 128, 32), U.right(2, 128, 64), None),
              U.retention_layer(2, 256, 136, 256, 10000.0, [0.999, 0.97], U.experts(8, 2, 64, (2, 1))),
              U.retention_layer(1, 264, 40, 100, 10000.0, [0.99], None)]
    cfg = U.small_config(layers, width=128, vocab=216)
    w = _weights(cfg, 23)
    path = U.write_checkpoint(str(tmp_path), cfg, w)
    eng = U.make_engine(path, device="cuda", dtype=dtype, pages=40, block_size=32,
                        graphs=dtype == torch.bfloat16)
    seqs = {"a": U.tokens(500, 216, 31), "b": U.tokens(135, 216, 32)}
    schedule = [[("a", 233)], [("a", 200), ("b", 100)], [("a", 1), ("b", 1)],
                [("a", 36), ("b", 4)]] + [[("a", 1), ("b", 1)]] * 30
    got = U.run_schedule(eng, seqs, schedule)
    for name, toks in seqs.items():
        want = oracle.forward(cfg, w, toks)
        assert close(got[name], want, dtype), (name, U.describe(got[name], want, TOL[dtype]))


def test_greedy_generation_fp32_matches_the_reference(ckpt):
    cfg, w, path = ckpt
    eng = U.make_engine(path, device="cuda", dtype=torch.float32, prefill_chunk_size=16)
    prompts = [U.tokens(37, cfg["vocab"], 11), U.tokens(5, cfg["vocab"], 12)]
    sp = [SamplingParams(temperature=0.0, max_new_tokens=n, ignore_eos=True) for n in (10, 16)]
    out = list(eng.generate(prompts, sp).values())
    for p, s, got in zip(prompts, sp, out):
        seq = list(p)
        for _ in range(s.max_new_tokens):
            seq.append(int(oracle.forward(cfg, w, seq)[-1].argmax()))
        assert got == seq[len(p):]


def test_greedy_generation_bf16_through_graphs(ckpt):
    """bf16 + captured decode graphs + async decode: every generated token is
    the reference's best token or within rounding of it (two in 24 may stand
    at a position that rounding moves further)."""
    cfg, w, path = ckpt
    eng = U.make_engine(path, device="cuda", dtype=torch.bfloat16, graphs=True)
    eng.warmup_serving()   # what `serve` does at start: GEMM picks, every decode graph
    prompts = [U.tokens(29, cfg["vocab"], 21), U.tokens(3, cfg["vocab"], 22),
               U.tokens(64, cfg["vocab"], 23)]
    sp = [SamplingParams(temperature=0.0, max_new_tokens=24, ignore_eos=True)] * 3
    out = list(eng.generate(prompts, sp).values())
    for p, got in zip(prompts, out):
        assert len(got) == 24
        logits = oracle.forward(cfg, w, list(p) + got)
        spread = float(logits.std())
        gaps = [float(logits[len(p) - 1 + i].max() - logits[len(p) - 1 + i][tok])
                for i, tok in enumerate(got)]
        assert sum(x < 0.25 * spread for x in gaps) >= 22, gaps
    assert eng.cache_manager.num_free_blocks == 64
