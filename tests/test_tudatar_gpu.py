"""Tudatar served on the GPU (HIP kernels, bf16 and fp32) against the plain
whole-sequence oracle: whole prompts, portions, decode, mixed batches with
page and slot reuse, greedy generation through the scheduler, captured
decode, long contexts (the attention key splits), window edges that show,
and the matrix-core attention paths at their head sizes."""
import pytest
import torch

from tests import tudatar_oracle as O
from tests.tudatar_util import (assert_logits, chunk_schedule, make_engine,
                                 oracle_logits, planted_attention, random_tokens,
                                replay)

pytestmark = pytest.mark.gpu

if not torch.cuda.is_available():
    pytest.skip("needs a GPU", allow_module_level=True)

from tests.test_tudatar import VARIANTS, _cfg  # noqa: E402


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
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


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_mixed_batches_reuse_pages_and_slots(tmp_path, dtype):
    cfg = _cfg("base")
    W = O.random_weights(cfg, seed=2)
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
    and portions of some hundred tokens, fp32 against the oracle."""
    cfg = O.make_config(window=500)
    W = O.random_weights(cfg, seed=24)
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


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("kv,window", [(2, 70), (4, 64), (1, 1)])
def test_head_sizes_of_the_matrix_core_paths(tmp_path, dtype, kv, window):
    """Attention heads of 64 and a latent row of 64 + 32: bf16 prompt
    portions of 16 tokens or more run on the matrix cores, shorter portions
    and decode rows on the generic kernels with their key splits; fp32 takes
    the generic kernels throughout. All must agree with the oracle on one
    sequence cut in different ways."""
    cfg = O.make_config(width=64, vocab=90, ff=24, heads=4, kv_heads=kv,
                        dim=64, vdim=64, scale=0.125, window=window,
                        lat_heads=4, lat_dim=16, rot_dim=32, lat_vdim=16,
                        kv_rank=64, q_rank=24, delta_dim=32, delta_vdim=40)
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


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("window,far,dim", [(64, 3, 64), (64, 70, 64),
                                            (100, 0, 64), (72, 31, 96),
                                            (17, 15, 4)])
@pytest.mark.parametrize("sched", ["whole", "decode", "portions"])
def test_window_edge_shows(tmp_path, dtype, window, far, dim, sched):
    """A planted key takes nearly all weight while it is visible: the row
    window - 1 after it still sees it, the next one does not; matrix-core
    (64) and generic head sizes."""
    T = far + window + 20
    cfg, W, toks = planted_attention(window, far, T, dim=dim)
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
    assert float(got[edge, 0]) > 0.8 * float(got[far, 0])
    assert abs(float(got[edge + 1, 0])) < 0.05 * float(got[edge, 0])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_expert_execution_strategies(tmp_path, dtype):
    """Steps of 300 and 700 tokens at a width and expert size the
    grouped-GEMM kernel covers (bf16: sorted rows through the kernel; beyond
    its range and in fp32 sorted rows through plain products per expert),
    decode rows through the all-experts products: all equal the oracle."""
    cfg = O.make_config(width=128, vocab=80, ff=128, experts=8, top=2,
                        kinds=("attention", "channel_delta"))
    W = O.random_weights(cfg, seed=26)
    eng = make_engine(tmp_path, cfg, W, device="cuda", dtype=dtype,
                      kv_blocks=80)
    toks = random_tokens(1010, cfg["vocab"], 12)
    want = oracle_logits(cfg, W, toks)
    got = replay(eng, {"a": toks},
                 [[("a", 300)], [("a", 700)]] + [[("a", 1)]] * 10)["a"]
    assert_logits(got, want, dtype)
