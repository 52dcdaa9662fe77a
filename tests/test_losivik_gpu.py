"""Losivik served on the GPU (HIP kernels, bf16 and fp32) against the plain
whole-sequence oracle: whole prompts, portions, decode, mixed batches with
page and slot reuse, greedy generation through the scheduler, captured
decode, long contexts (attention key splits, many state-space pieces), edges
of windows and kept tokens that show, long memory, and the matrix-core
attention paths at their head sizes."""
import pytest
import torch

from tests import losivik_oracle as O
from tests.losivik_util import (assert_logits, chunk_schedule, make_engine,
                                oracle_logits, planted_attention,
                                planted_latent, planted_memory, random_tokens,
                                replay, slow_decay)

pytestmark = pytest.mark.gpu

if not torch.cuda.is_available():
    pytest.skip("needs a GPU", allow_module_level=True)

from tests.test_losivik import VARIANTS, _cfg  # noqa: E402

DTYPES = [torch.float32, torch.bfloat16]


@pytest.mark.parametrize("dtype", DTYPES)
def test_whole_chunked_decode_match_oracle(tmp_path, dtype):
    cfg = _cfg("base")
    W = O.random_weights(cfg, seed=1)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=dtype)
    toks = random_tokens(61, cfg["vocab"], 5)
    want = oracle_logits(cfg, W, toks)
    for sched in ([[("a", 61)]],
                  chunk_schedule("a", 61, [2, 17, 3, 1, 1, 16]),
                  [[("a", 20)]] + [[("a", 1)]] * 41):
        got = replay(eng, {"a": toks}, sched)["a"]
        assert_logits(got, want, dtype)


def test_layer_residuals_match_oracle(tmp_path):
    cfg = _cfg("base")
    W = O.random_weights(cfg, seed=12)
    eng = make_engine(tmp_path, cfg, W, device="cuda")
    toks = random_tokens(90, cfg["vocab"], 2)
    layers, seen = [], []
    O.forward(cfg, W, toks, layers)
    eng.runner.layer_tap = lambda i, x: seen.append(x.clone())
    eng.feed([("a", toks, [89])], ["a"])
    for i, x in enumerate(seen):
        assert torch.allclose(x.double().cpu(), layers[i], atol=4e-4), i


@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_reuse_pages_and_slots(tmp_path, dtype):
    cfg = _cfg("base")
    W = slow_decay(O.random_weights(cfg, seed=2))
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=dtype,
                      kv_blocks=12, block_size=16)
    for t in eng.kv.k_cache + eng.kv.v_cache + eng.kv.rec_state + \
            eng.kv.conv_state:
        if t is not None:
            t.fill_(float("nan"))
    reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 10 + i)
            for i, n in enumerate([37, 9, 52, 18, 33, 5, 41])}
    sched = [
        [("r0", 20), ("r1", 2)],
        [("r0", 1), ("r1", 7), ("r2", 30)],
        [("r0", 16), ("r2", 1), ("r3", 18)],        # r0, r1, r3 end
        [("r2", 21), ("r4", 33), ("r5", 2), ("r6", 3)],
        [("r5", 3), ("r6", 38)],
    ]
    got = replay(eng, reqs, sched)
    for rid, toks in reqs.items():
        assert_logits(got[rid], oracle_logits(cfg, W, toks), dtype, rid)
    assert eng.kv.free_blocks == eng.kv.n_blocks - 1
    assert eng.kv.free_state_slots == eng.kv.n_state_slots - 1


@pytest.mark.parametrize("name", list(VARIANTS))
def test_variants_fp32(tmp_path, name):
    cfg = _cfg(name)
    W = O.random_weights(cfg, seed=21)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=torch.float32)
    toks = random_tokens(45, cfg["vocab"], 1)
    want = oracle_logits(cfg, W, toks)
    for sched in ([[("a", 45)]], chunk_schedule("a", 45, [2, 5, 1, 16, 3]),
                  [[("a", 9)]] + [[("a", 1)]] * 36):
        assert_logits(replay(eng, {"a": toks}, sched)["a"], want,
                      torch.float32, name)


def test_long_contexts_and_key_splits(tmp_path):
    """Decode rows over a context long enough for the attention key splits
    and portions of some hundred tokens (several state-space pieces), fp32
    against the oracle."""
    cfg = O.make_config(window=500, lat_window=200)
    W = slow_decay(O.random_weights(cfg, seed=24))
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=torch.float32,
                      kv_blocks=40)
    toks = random_tokens(330, cfg["vocab"], 9)
    want = oracle_logits(cfg, W, toks)
    for sched in ([[("a", 300)]] + [[("a", 1)]] * 30,
                  [[("a", 150)], [("a", 170)]] + [[("a", 1)]] * 10):
        got = replay(eng, {"a": toks}, sched)["a"]
        assert_logits(got, want, torch.float32)


def test_greedy_generation_through_scheduler(tmp_path):
    cfg = _cfg("base")
    W = O.random_weights(cfg, seed=3)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=torch.float32)
    try:
        prompt = random_tokens(11, cfg["vocab"], 3)
        req = eng.generate(prompt, max_new_tokens=12, temperature=0.0,
                           repetition_penalty=1.0)
        seq = list(prompt)
        for tok in req.output_ids:
            logits = oracle_logits(cfg, W, seq)[-1]
            top2 = torch.topk(logits, 2).values
            if float(top2[0] - top2[1]) > 1e-3:   # skip near-ties
                assert int(logits.argmax()) == tok
            seq.append(tok)
        assert len(req.output_ids) == 12
    finally:
        eng.shutdown()


def test_graph_decode_equals_eager(tmp_path):
    """Captured decode steps (hipGraph) replayed several times with eager
    prefill work between them must give the tokens of the eager engine."""
    cfg = _cfg("base")
    W = O.random_weights(cfg, seed=23)
    prompts = [random_tokens(n, cfg["vocab"], 40 + n) for n in (13, 5)]
    outs = {}
    for graphs in (False, True):
        eng = make_engine(tmp_path, cfg, W, device="cuda",
                          dtype=torch.float32, use_graphs=graphs)
        assert (eng.graphs is not None) == graphs
        try:
            outs[graphs] = [
                eng.generate(p, max_new_tokens=24, temperature=0.0,
                             repetition_penalty=1.0).output_ids
                for p in prompts]
        finally:
            eng.shutdown()
    assert outs[True] == outs[False]
    seq = list(prompts[0])
    for tok in outs[True][0]:
        logits = oracle_logits(cfg, W, seq)[-1]
        top2 = torch.topk(logits, 2).values
        if float(top2[0] - top2[1]) > 1e-3:
            assert int(logits.argmax()) == tok
        seq.append(tok)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kv,window,keep", [(2, 70, 3), (4, 64, 70), (1, 1, 1)])
def test_head_sizes_of_the_matrix_core_paths(tmp_path, dtype, kv, window,
                                             keep):
    """Attention heads and a latent row of 64: bf16 prompt portions of 16
    tokens or more run on the matrix cores, shorter portions and decode rows
    on the generic kernels with their key splits; fp32 takes the generic
    kernels throughout. All must agree with the oracle on one sequence cut
    in different ways."""
    cfg = O.make_config(width=64, vocab=90, heads=4, kv_heads=kv, dim=64,
                        vdim=64, scale=0.125, window=window, keep=keep,
                        lat_heads=4, lat_dim=16, lat_vdim=16, kv_rank=64,
                        lat_window=window, ssd_heads=4, ssd_vdim=16, state=32,
                        norm_groups=2, ff=48, expert_ff=24, shared_ff=24,
                        side=16)
    W = O.random_weights(cfg, seed=25)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=dtype,
                      kv_blocks=40)
    toks = random_tokens(210, cfg["vocab"], 11)
    want = oracle_logits(cfg, W, toks)
    for sched in ([[("a", 210)]],
                  chunk_schedule("a", 210, [100, 3, 60, 17, 1, 16]),
                  [[("a", 170)]] + [[("a", 1)]] * 40):
        got = replay(eng, {"a": toks}, sched)["a"]
        assert_logits(got, want, dtype)


@pytest.mark.parametrize("window", [1, 64, 90])
def test_whole_prompts_with_projected_keys(tmp_path, window):
    """bf16, a latent row wider than its keys and values: whole prompts
    project keys and values, portions and decode rows score latent rows; all
    equal the oracle, alone and as several whole prompts in one step"""
    cfg = O.make_config(width=64, vocab=90, lat_heads=3, lat_dim=64,
                        lat_vdim=64, kv_rank=96, lat_window=window,
                        lat_scale=0.125)
    W = O.random_weights(cfg, seed=27)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=torch.bfloat16,
                      kv_blocks=60)
    assert eng.weights.layers[1].mix[""].w_ukv is not None
    reqs = {r: random_tokens(n, cfg["vocab"], 30 + n)
            for r, n in (("a", 210), ("b", 5), ("c", 130))}
    want = {r: oracle_logits(cfg, W, t) for r, t in reqs.items()}
    for sched in ([[("a", 210), ("b", 5), ("c", 130)]],
                  [[("a", 100), ("c", 64)], [("a", 110), ("b", 5), ("c", 66)]],
                  [[("a", 200), ("b", 5), ("c", 129)]] +
                  [[("a", 1)]] * 10 + [[("c", 1)]]):
        got = replay(eng, reqs, sched)
        for r in reqs:
            assert_logits(got[r], want[r], torch.bfloat16, r)


def _edge_check(tmp_path, case, dtype, sched, window, far, stays):
    cfg, W, toks = case
    T = len(toks)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=dtype)
    edge = far + window - 1
    steps = {"whole": [[("a", T)]],
             "decode": [[("a", far + 1)]] + [[("a", 1)]] * (T - far - 1),
             "portions": chunk_schedule("a", T, [edge, 2, 18])}[sched]
    got = replay(eng, {"a": toks}, steps)["a"]
    want = oracle_logits(cfg, W, toks)
    for t in (far, edge - 1, edge, edge + 1, T - 1):
        torch.testing.assert_close(
            got[t].double().cpu(), want[t], rtol=0.03,
            atol=0.03 * float(want[t].abs().max()))
    seen = float(got[far, 3])
    assert float(got[edge, 3]) > 0.8 * seen > 0.0
    for t in (edge + 1, T - 1):
        if stays:
            assert float(got[t, 3]) > 0.8 * seen
        else:
            assert abs(float(got[t, 3])) < 0.05 * seen


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep,far,dim", [
    (64, 4, 3, 64), (64, 4, 4, 64), (64, 70, 69, 64), (64, 64, 64, 64),
    (100, 1, 0, 64), (72, 31, 31, 96), (72, 32, 31, 96), (17, 16, 15, 4)])
@pytest.mark.parametrize("sched", ["whole", "decode", "portions"])
def test_window_and_kept_edges_show(tmp_path, dtype, window, keep, far, dim,
                                    sched):
    """A planted key takes nearly all weight while it is visible: the row
    window - 1 after it still sees it, later ones only if it is one of the
    kept first tokens; matrix-core (64) and generic head sizes."""
    case = planted_attention(window, keep, far, far + window + 20, dim=dim)
    _edge_check(tmp_path, case, dtype, sched, window, far, far < keep)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,far,rank,dim", [
    (64, 3, 64, 4), (17, 15, 64, 4), (100, 0, 8, 4), (33, 31, 5, 4),
    (65, 2, 80, 64), (70, 63, 72, 64)])
@pytest.mark.parametrize("sched", ["whole", "decode", "portions"])
def test_latent_window_edge_shows(tmp_path, dtype, window, far, rank, dim,
                                  sched):
    case = planted_latent(window, far, far + window + 20, rank=rank, dim=dim)
    _edge_check(tmp_path, case, dtype, sched, window, far, False)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("far", [0, 63, 64])
@pytest.mark.parametrize("sched", [[400], [70] + [1] * 330,
                                   [64, 1, 63, 2, 270]])
def test_memory_lasts(tmp_path, dtype, far, sched):
    """one write into a state that forgets nothing is read by every later
    row, through pieces, portions and decoded tokens"""
    cfg, W, toks = planted_memory(far, 400)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=dtype,
                      kv_blocks=40)
    eng.kv.rec_state[0].fill_(float("nan"))
    got = replay(eng, {"a": toks}, [[("a", n)] for n in sched])["a"]
    assert_logits(got, oracle_logits(cfg, W, toks), dtype)
    for t in (far + 1, far + 65, 399):
        assert float(got[t, 3]) > 0.8 * float(got[far, 3]) > 0.4


@pytest.mark.parametrize("dtype", DTYPES)
def test_expert_execution_strategies(tmp_path, dtype):
    """Steps of 300 and 700 tokens at a width and expert size the
    grouped-GEMM kernel covers (bf16: sorted rows through the kernel; beyond
    its range and in fp32 sorted rows through plain products per expert),
    decode rows through the all-experts products: all equal the oracle."""
    cfg = O.make_config(width=128, vocab=80, expert_ff=128, experts=8, top=2,
                        shared_ff=64, kinds=("latent_attention", "parallel"),
                        mlps=("moe", "moe"))
    W = O.random_weights(cfg, seed=26)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=dtype,
                      kv_blocks=80)
    toks = random_tokens(1010, cfg["vocab"], 12)
    want = oracle_logits(cfg, W, toks)
    got = replay(eng, {"a": toks},
                 [[("a", 300)], [("a", 700)]] + [[("a", 1)]] * 10)["a"]
    assert_logits(got, want, dtype)
