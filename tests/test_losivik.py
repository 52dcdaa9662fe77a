"""Losivik on the CPU reference path against the plain oracle
(tests/losivik_oracle.py): each mechanism alone, then the served model —
whole prompts, decoding, portions, mixed batches with page and slot reuse,
planted keys at the edges of windows and kept tokens, long memory, the
scheduler's own greedy generation."""
import io
import json
import math
import sys

import pytest
import torch

from bee2bee_amd.models.spec import losivik_spec
from bee2bee_amd.ops import reference as ref
from tests import losivik_oracle as O
from tests.losivik_util import (assert_logits, chunk_schedule, make_engine,
                                oracle_logits, planted_attention,
                                planted_latent, planted_memory, random_tokens,
                                rel_err, replay, row_errs, slow_decay)
from tests.test_tudatar import i32, pages

F32, F64 = torch.float32, torch.float64
NAN = float("nan")


# ----------------------------------------------------------- mechanisms

@pytest.mark.parametrize("W", [1, 2, 7, 24])
def test_position_vectors(W):
    """scaled embedding plus sin/cos pairs; an odd width ends with a sine"""
    torch.manual_seed(0)
    table = torch.randn(9, W)
    ids = torch.tensor([3, 8, 0, 3])
    pos = i32([0, 1, 700, 31])
    got = ref.embed_sinusoid(ids, table, 2.5, pos, ref.sinusoid_freqs(W, "cpu"))
    pv = O.position_vectors(701, W)
    want = table.double()[ids] * 2.5 + pv[pos.long()]
    assert torch.allclose(got.double(), want, atol=1e-6)
    assert float(got[0, 0]) == float(table[3, 0] * 2.5)     # sin 0


@pytest.mark.parametrize("W", [1, 5, 24])
def test_residual_update_and_norm_pair(W):
    torch.manual_seed(1)
    x, ys = torch.randn(4, W) * 3, [torch.randn(4, W) for _ in range(3)]
    s1, s2, wp, wa, wb = (torch.randn(W) for _ in range(5))
    r = x.clone()
    out = ref.scaled_add(r, ys[0], s1, ys[1], s2, ys[2], F32)
    want = x + s1 * ys[0] + s2 * (ys[1] + ys[2])
    assert torch.allclose(r, want, atol=1e-5) and torch.equal(out, r)
    r = x.clone()
    ref.scaled_add(r, ys[0], s1, None, None, None, F32)
    assert torch.allclose(r, x + s1 * ys[0], atol=1e-5)
    r = x.clone()
    a, b = ref.add_norm_pair(r, ys[0], wp, 1.0 + wa, None, 1e-5, F32)
    want = x.double() + O.unit(ys[0].double(), 1e-5) * wp
    assert b is None and torch.allclose(r.double(), want, atol=1e-5)
    assert torch.allclose(a.double(), O.norm_around_zero(
        {"n": wa}, "n", want, 1e-5), atol=1e-5)


def test_side_gate_takes_the_layers_slice():
    torch.manual_seed(2)
    g, table = torch.randn(5, 3) * 2, torch.randn(7, 12)
    ids = torch.tensor([6, 0, 2, 2, 5])
    got = ref.side_gate(g, table, 6, ids)
    want = O.gelu_tanh(g.double()) * table.double()[ids][:, 6:9]
    assert torch.allclose(got.double(), want, atol=1e-6)


@pytest.mark.parametrize("groups", [1, 2, 6, 12])
def test_gate_comes_before_the_grouped_norm(groups):
    torch.manual_seed(3)
    y, z, w = torch.randn(4, 12) * 2, torch.randn(4, 12), torch.randn(12)
    out = torch.empty(4, 12)
    ref.gated_group_norm(y, z, w, groups, 1e-5, out, 0.3)
    v = (y.double() * O.silu(z.double())).view(4, groups, -1)
    want = O.unit(v, 1e-5).view(4, 12) * w * 0.3
    assert torch.allclose(out.double(), want, atol=1e-5)


@pytest.mark.parametrize("H,G,N,V", [(4, 2, 7, 6), (3, 3, 4, 5), (6, 1, 3, 1),
                                     (1, 1, 1, 1)])
@pytest.mark.parametrize("sched", [[150], [2] * 11 + [1], [1] * 23,
                                   [64, 65, 3], [63, 1, 64]])
@pytest.mark.parametrize("shift", [0.0, 3.0, -6.0])
def test_state_space_scan_portions(H, G, N, V, sched, shift):
    """the chunked evaluation against the token loop, from a NaN-filled
    slot, with decays from forgetting at once to forgetting nothing"""
    torch.manual_seed(4)
    T = sum(sched)
    xbc = torch.randn(T, H * V + 2 * G * N)
    dt = torch.randn(T, H) * 2
    bias, A_log, skip = torch.randn(H), torch.randn(H) + shift, torch.randn(H)
    x, B, C = xbc.double().split([H * V, G * N, G * N], -1)
    own = [n // (H // G) for n in range(H)]
    want = O.ssd_scan(x.view(T, H, V), B.view(T, G, N)[:, own],
                      C.view(T, G, N)[:, own],
                      O.softplus(dt.double() + bias.double()),
                      torch.exp(A_log.double()), skip.double())
    state = torch.full((3, H, N, V), NAN)
    got, at = [], 0
    for n in sched:
        got.append(ref.ssd_scan(xbc[at:at + n], dt[at:at + n], bias,
                                torch.exp(A_log), skip, G, state, i32([1]),
                                i32([0, n]), i32(list(range(at, at + n)))))
        at += n
    got = torch.cat(got).double().view(T, H, V)
    assert torch.allclose(got, want, atol=2e-4 * float(want.abs().max()))
    assert bool(state[0].isnan().all()) and bool(state[2].isnan().all())


def test_state_space_read_sees_own_write_and_fades():
    """closed form with one head, one row, one column"""
    d = math.log1p(math.exp(0.5))
    xbc = torch.tensor([[2.0, 3.0, 5.0], [0.0, 1.0, 5.0]])    # x, B, C
    state = torch.zeros(1, 1, 1, 1)
    y = ref.ssd_scan(xbc, torch.zeros(2, 1), torch.tensor([0.5]),
                     torch.tensor([0.7]), torch.tensor([10.0]), 1, state,
                     i32([0]), i32([0, 2]), i32([0, 1]))
    s = d * 3 * 2
    assert torch.allclose(y.view(-1), torch.tensor(
        [5 * s + 20.0, 5 * s * math.exp(-0.7 * d)]), rtol=1e-5)


@pytest.mark.parametrize("taps", [1, 2, 4])
@pytest.mark.parametrize("sched", [[13], [2] * 6 + [1], [1] * 13, [5, 1, 7]])
def test_short_conv_with_bias(taps, sched):
    torch.manual_seed(5)
    C, T = 6, 13
    u, w, b = torch.randn(T, C), torch.randn(C, taps), torch.randn(C)
    want = O.silu(O.causal_conv(u.double(), w.double(), b.double()))
    state = torch.full((2, taps - 1, C), NAN)
    got, at = [], 0
    for n in sched:
        pos = i32(list(range(at, at + n)))
        got.append(ref.short_conv(u[at:at + n], w.t().contiguous(), state,
                                  i32([1]), i32([0, n]), i32([0] * n), pos,
                                  True, bias=b))
        at += n
    assert torch.allclose(torch.cat(got).double(), want, atol=1e-5)


@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 6, 5), (3, 3, 4, 4), (6, 1, 3, 7),
                                      (1, 1, 1, 1)])
@pytest.mark.parametrize("window,keep", [(1, 1), (7, 3), (2, 9), (100, 4),
                                         (5, 0)])
@pytest.mark.parametrize("sched", [[23], [2] * 11 + [1], [1] * 23,
                                   [7, 1, 11, 4]])
def test_attention_with_kept_first_tokens(H, G, D, Dv, window, keep, sched):
    """per-head norms, the page store of separate values, the mask"""
    torch.manual_seed(6)
    T, eps, scale = 23, 1e-5, 0.7
    q, k, v = (torch.randn(T, n, d) for n, d in ((H, D), (G, D), (G, Dv)))
    wq, wk = torch.randn(D), torch.randn(D)
    ok = O.visible(T, {"size": window, "keep_first": keep})
    qn = O.unit(q.double(), eps) * wq
    kn = O.unit(k.double(), eps) * wk
    want = torch.stack([O.softmax_rows(
        qn[:, n] @ kn[:, n // (H // G)].t() * scale, ok) @
        v[:, n // (H // G)].double() for n in range(H)], 1)
    bs, m = 4, pages([T], [0], 4)
    kc = torch.full((m["nb"], G, bs, D), NAN)
    vc = torch.full((m["nb"], G, bs, Dv), NAN)
    got, at = [], 0
    for n in sched:
        qq = q[at:at + n].clone()
        pos = i32(list(range(at, at + n)))
        ref.qk_norm_rope_store(qq, k[at:at + n], wq, wk, eps, 0, pos, None,
                               None, torch.full((H,), scale), kc, vc,
                               m["slot"][at:at + n], v=v[at:at + n])
        out = torch.empty(n, H * Dv)
        ref.gqa_attn(qq, kc, vc, m["bt"], pos, i32([0] * n), i32([0, n]), 0.0,
                     None, None, None, window, out, out_scale=0.5,
                     keep_first=keep)
        got.append(out.view(n, H, Dv))
        at += n
    assert torch.allclose(torch.cat(got).double(), want * 0.5, atol=2e-5)


@pytest.mark.parametrize("E,top,shared", [(5, 2, 6), (4, 4, 0), (1, 1, 3),
                                          (9, 3, 7)])
def test_weight_on_the_experts_input(E, top, shared):
    """scores are not renormalized; relu(w z)^2, so the weight enters
    squared; both execution forms against the oracle's per-token loop"""
    torch.manual_seed(7)
    ff, Wd, T = 7, 6, 17
    h = torch.randn(T, Wd)
    W = {"router": torch.randn(E, Wd)}
    for n, f in [(f"e{e}.", ff) for e in range(E)] + [("shared.", shared)]:
        W.update({n + "up": torch.randn(f, Wd), n + "down": torch.randn(Wd, f)})
    f = {"router": {"top": top}, "shared": {"ff": shared} if shared else None}
    want = O.moe(W, "", f, h.double())
    wts, idx = ref.group_topk_gate(h @ W["router"].t(), top, 1, 1, "sigmoid")
    names = [f"e{e}." for e in range(E)] + (["shared."] if shared else [])
    up = torch.cat([W[n + "up"] for n in names])
    down = torch.cat([W[n + "down"] for n in names], 1)
    z = h @ up.t()
    got = ref.routed_relu2(z, wts, idx, E, ff) @ down.t()
    assert torch.allclose(got.double(), want, atol=2e-4)
    # an expert that was not chosen adds nothing even where it overflows
    off = ~(idx == 0).any(1)
    z[:, :ff] = float("inf")
    assert float(ref.routed_relu2(z, wts, idx, E, ff)[off, :ff].abs().sum()) \
        == 0.0
    pos, tok, offs = ref.moe_sort(idx, E)
    xs, y = h[tok.long()], torch.empty(T * top, Wd)
    for e in range(E):
        a, b = int(offs[e]), int(offs[e + 1])
        y[a:b] = torch.relu(xs[a:b] @ W[f"e{e}.up"].t()) ** 2 @ \
            W[f"e{e}.down"].t()
    got = ref.moe_combine(y, pos, wts * wts)
    if shared:
        got = got + torch.relu(h @ W["shared.up"].t()) ** 2 @ \
            W["shared.down"].t()
    assert torch.allclose(got.double(), want, atol=2e-4)


def test_dense_unit_clamps_and_gates():
    torch.manual_seed(8)
    h = torch.randn(5, 4, dtype=F64) * 3
    W = {k: torch.randn(s) for k, s in (
        ("gate", (6, 4)), ("up", (6, 4)), ("down", (4, 6)), ("gate.b", (6,)),
        ("up.b", (6,)), ("down.b", (4,)))}
    want = O.dense(W, "", {"limit": 0.9}, h)
    gu = torch.cat([h.float() @ W[n].t() + W[n + ".b"] for n in ("gate", "up")],
                   1)
    got = ref.clamped_glu(gu, 0.9, 1.702) @ W["down"].t() + W["down.b"]
    assert torch.allclose(got.double(), want, atol=1e-4)


def test_config_parsing():
    cfg = O.make_config()
    spec = losivik_spec("t", cfg)
    p, la = spec.layer_specs[0].mixer, spec.layer_specs[1].mixer
    a, r = p.left, p.right
    assert (a.kind, a.head_norm, a.rope_dims, a.window, a.keep_first) == \
        ("gqa_attention", True, 0, 9, 3)
    assert (r.kind, r.heads, r.vdim, r.state, r.groups, r.taps,
            r.norm_groups) == ("ssd", 4, 6, 7, 2, 4, 3)
    assert (p.left_scale, p.right_scale, p.combine) == (0.8, 1.3, "scaled_sum")
    assert (la.rot_dim, la.rope_dims, la.window, la.head_gate, la.sink,
            la.q_rank, la.cache_dim) == (0, 0, 6, True, False, 0, 11)
    f = spec.layer_specs[0].ffn
    assert (f.n_experts, f.top_k, f.act, f.score, f.renorm, f.weight_input,
            f.shared_ff, f.up_rows) == (5, 2, "relu2", "sigmoid_all", False,
                                        True, 8, 10)
    d = spec.layer_specs[1].ffn
    assert (d.act, d.limit, d.alpha, d.bias) == ("clamped_glu", 1.5, 1.702,
                                                 True)
    assert spec.layer_specs[2].ffn is None
    assert (spec.embed_scale, spec.side_dim, spec.pos_type,
            spec.tie_embeddings) == (3.0, 7, "sinusoid", True)
    for bad in (dict(heads=4, kv_heads=3), dict(top=6),
                dict(ssd_heads=4, groups=3), dict(norm_groups=5)):
        with pytest.raises(ValueError):
            losivik_spec("t", O.make_config(**bad))
    for key, val in (("type", "retention"), ("mlp", {"kind": "other"})):
        bad = O.make_config()
        bad["layers"][1][key] = val
        with pytest.raises(ValueError):
            losivik_spec("t", bad)


# ------------------------------------------------------------ the model

VARIANTS = {
    "base": dict(),
    # values that other models make equal or 1
    "ones": dict(heads=1, kv_heads=1, dim=1, vdim=1, window=1, keep=1,
                 lat_heads=1, lat_dim=1, lat_vdim=1, kv_rank=1, lat_window=1,
                 ssd_heads=1, ssd_vdim=1, state=1, groups=1, norm_groups=1,
                 conv=1, experts=1, top=1, expert_ff=1, shared_ff=1, ff=1,
                 side=1),
    "equal": dict(width=16, heads=4, kv_heads=4, dim=8, vdim=8, window=8,
                  keep=8, lat_heads=4, lat_dim=8, lat_vdim=8, kv_rank=8,
                  lat_window=8, ssd_heads=4, ssd_vdim=8, state=8, groups=4,
                  norm_groups=4, experts=4, top=4, expert_ff=16, shared_ff=16,
                  ff=16, side=8, conv=4, left_scale=1.0, right_scale=1.0,
                  embed_scale=1.0),
    "other-order": dict(kinds=("latent_attention", "parallel", "parallel",
                               "latent_attention", "latent_attention"),
                        mlps=("moe", "dense", "moe", None, "dense"),
                        width=21, heads=6, kv_heads=1, dim=4, vdim=12,
                        window=33, keep=1, lat_window=40, ssd_heads=6,
                        groups=3, ssd_vdim=5, state=12, norm_groups=1, conv=5,
                        experts=9, top=3, shared_ff=0, side=5),
    "wide-heads": dict(kinds=("parallel", "latent_attention"),
                       mlps=(None, None), lat_heads=5, lat_dim=3, lat_vdim=7,
                       kv_rank=24, lat_window=3, window=4, keep=12, dim=10,
                       vdim=3, ssd_heads=2, groups=1, ssd_vdim=9, state=20,
                       norm_groups=9, conv=2, embed_scale=0.5),
}


def _cfg(name):
    return O.make_config(**VARIANTS[name])


@pytest.mark.parametrize("name", list(VARIANTS))
def test_served_model_matches_oracle(tmp_path, name):
    cfg = _cfg(name)
    W = O.random_weights(cfg, seed=11)
    eng = make_engine(tmp_path, cfg, W)
    toks = random_tokens(45, cfg["vocab"], 1)
    want = oracle_logits(cfg, W, toks)
    schedules = {
        "whole": [[("a", 45)]],
        "decode": [[("a", 9)]] + [[("a", 1)]] * 36,
        "portions": chunk_schedule("a", 45, [2, 5, 1, 16, 3]),
        "twos": chunk_schedule("a", 45, [2]),
        "token-by-token": [[("a", 1)]] * 45,
    }
    for what, sched in schedules.items():
        got = replay(eng, {"a": toks}, sched)["a"]
        assert_logits(got, want, F32, what)
    assert eng.kv.free_blocks == eng.kv.n_blocks - 1     # scratch page only


def test_layer_residuals_match_oracle(tmp_path):
    cfg = _cfg("base")
    W = O.random_weights(cfg, seed=12)
    eng = make_engine(tmp_path, cfg, W)
    toks = random_tokens(19, cfg["vocab"], 2)
    layers, seen = [], []
    O.forward(cfg, W, toks, layers)
    eng.runner.layer_tap = lambda i, x: seen.append(x.clone())
    eng.feed([("a", toks, [18])], ["a"])
    assert len(seen) == len(layers) == 4
    for i, x in enumerate(seen):
        assert torch.allclose(x.double(), layers[i], atol=2e-4), i


def _edge_steps(sched, T, edge):
    return {"whole": [[("a", T)]],
            "decode": [[("a", 2)]] + [[("a", 1)]] * (T - 2),
            "portions": chunk_schedule("a", T, [edge, 2, 3])}[sched]


@pytest.mark.parametrize("window,keep,far", [
    (8, 3, 3), (8, 3, 2), (8, 1, 0), (8, 0, 0), (16, 4, 3), (16, 4, 4),
    (5, 17, 16), (5, 17, 17), (200, 4, 1), (200, 4, 5), (300, 2, 130)])
@pytest.mark.parametrize("sched", ["whole", "decode", "portions"])
def test_window_and_kept_edges_show(tmp_path, window, keep, far, sched):
    """A planted key takes nearly all weight while it is visible: the row
    window - 1 after it still sees it, the next one only if the key is one
    of the kept first tokens. Cut as one prompt, as decoding, as portions
    whose borders fall around the edge."""
    T = far + window + 6
    cfg, W, toks = planted_attention(window, keep, far, T)
    eng = make_engine(tmp_path, cfg, W, block_size=4, kv_blocks=120)
    edge = far + window - 1
    got = replay(eng, {"a": toks}, _edge_steps(sched, T, edge))["a"]
    assert_logits(got, oracle_logits(cfg, W, toks), F32)
    seen = float(got[far, 3])
    assert float(got[edge, 3]) > 0.8 * seen > 0.0
    for t in (edge + 1, T - 1):
        if far < keep:
            assert float(got[t, 3]) > 0.8 * seen
        else:
            assert abs(float(got[t, 3])) < 0.05 * seen


@pytest.mark.parametrize("window,far", [(1, 3), (8, 3), (8, 4), (16, 0),
                                        (17, 15), (5, 16), (300, 130)])
@pytest.mark.parametrize("sched", ["whole", "decode", "portions"])
def test_latent_window_edge_shows(tmp_path, window, far, sched):
    T = far + window + 6
    cfg, W, toks = planted_latent(window, far, T)
    eng = make_engine(tmp_path, cfg, W, block_size=4, kv_blocks=120)
    edge = far + window - 1
    got = replay(eng, {"a": toks}, _edge_steps(sched, T, max(edge, 2)))["a"]
    assert_logits(got, oracle_logits(cfg, W, toks), F32)
    assert float(got[edge, 3]) > 0.8 * float(got[far, 3]) > 0.0
    assert abs(float(got[edge + 1, 3])) < 0.05 * float(got[far, 3])


@pytest.mark.parametrize("far", [0, 5, 63, 64, 100])
@pytest.mark.parametrize("sched", [[400], [2] * 200, [105] + [1] * 295,
                                   [64, 1, 63, 128, 144]])
def test_memory_lasts(tmp_path, far, sched):
    """one write into a state that forgets nothing is read by every later
    row and by none before it"""
    cfg, W, toks = planted_memory(far, 400)
    eng = make_engine(tmp_path, cfg, W, kv_blocks=40)
    eng.kv.rec_state[0].fill_(NAN)
    got = replay(eng, {"a": toks}, [[("a", n)] for n in sched])["a"]
    assert_logits(got, oracle_logits(cfg, W, toks), F32)
    ref_ = float(got[far, 3])
    assert ref_ > 0.5
    for t in (far + 1, far + 65, 399):
        assert float(got[t, 3]) > 0.8 * ref_
    if far:
        assert abs(float(got[far - 1, 3])) < 0.3 * ref_


def test_mixed_batches_and_reuse(tmp_path):
    """Unequal requests side by side (portions next to single tokens, a
    request sitting out a step) equal each request alone; the pool is far
    smaller than the sum of the requests, so pages and slots come back."""
    cfg = _cfg("base")
    W = slow_decay(O.random_weights(cfg, seed=13))
    eng = make_engine(tmp_path, cfg, W, kv_blocks=7, block_size=8,
                      max_batch=3)
    # reused pages and slots hold garbage, never zeros
    for t in eng.kv.k_cache + eng.kv.v_cache + eng.kv.rec_state + \
            eng.kv.conv_state:
        if t is not None:
            t.fill_(NAN)
    lens = [21, 6, 30, 11, 17, 2, 26]
    reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 20 + i)
            for i, n in enumerate(lens)}
    sched = [
        [("r0", 9), ("r1", 2)],
        [("r0", 1), ("r1", 3), ("r2", 5)],
        [("r0", 11), ("r2", 1)],                    # r1 sits out; r0 ends
        [("r1", 1), ("r2", 2), ("r3", 11)],         # r1, r3 end
        [("r2", 22), ("r4", 2)],                    # r2 ends
        [("r4", 15), ("r5", 2), ("r6", 3)],         # r4, r5 end
        [("r6", 1)], [("r6", 22)],
    ]
    got = replay(eng, reqs, sched)
    for rid, toks in reqs.items():
        assert_logits(got[rid], oracle_logits(cfg, W, toks), F32, rid)
    assert eng.kv.free_blocks == eng.kv.n_blocks - 1
    assert eng.kv.free_state_slots == eng.kv.n_state_slots - 1


def test_long_decode_crosses_pages_and_windows(tmp_path):
    cfg = _cfg("base")                    # windows 9 and 6, pages of 4
    W = slow_decay(O.random_weights(cfg, seed=14))
    eng = make_engine(tmp_path, cfg, W, block_size=4, kv_blocks=50)
    toks = random_tokens(140, cfg["vocab"], 3)
    got = replay(eng, {"a": toks}, [[("a", 3)]] + [[("a", 1)]] * 137)["a"]
    assert_logits(got, oracle_logits(cfg, W, toks), F32)


def test_first_tokens_after_page_and_slot_reuse(tmp_path):
    """A request that takes over the pages and the slot another one just
    left must not see anything of it in its first tokens (conv rows,
    recurrent state, kept keys)."""
    cfg = _cfg("other-order")
    W = slow_decay(O.random_weights(cfg, seed=15))
    eng = make_engine(tmp_path, cfg, W, max_batch=1, kv_blocks=3, block_size=16)
    a, b = random_tokens(40, cfg["vocab"], 4), random_tokens(6, cfg["vocab"], 5)
    replay(eng, {"a": a}, [[("a", 40)]])
    for sched in ([[("b", 6)]], [[("b", 1)]] * 6, [[("b", 2)], [("b", 4)]]):
        got = replay(eng, {"b": b}, sched)["b"]
        assert_logits(got, oracle_logits(cfg, W, b), F32)


def test_large_steps_run_experts_apart(tmp_path):
    """a step of more tokens than the all-experts form takes"""
    cfg = O.make_config(kinds=("latent_attention",), mlps=("moe",), width=8)
    W = O.random_weights(cfg, seed=19)
    eng = make_engine(tmp_path, cfg, W, kv_blocks=40)
    toks = random_tokens(300, cfg["vocab"], 8)
    got = replay(eng, {"a": toks}, [[("a", 290)], [("a", 10)]])["a"]
    assert_logits(got, oracle_logits(cfg, W, toks), F32)


def test_greedy_generation_through_scheduler(tmp_path):
    """submit()/generate(): admission, chunked prompt prefill (budget of 7
    tokens a step), batched decode of concurrent requests, retirement."""
    cfg = _cfg("base")
    W = O.random_weights(cfg, seed=16)
    eng = make_engine(tmp_path, cfg, W, max_prefill_tokens=7)
    try:
        from bee2bee_amd.engine.engine import GenerationRequest
        from bee2bee_amd.engine.sampler import SamplingParams

        prompts = [random_tokens(n, cfg["vocab"], 30 + n) for n in (17, 3, 9)]
        reqs = [eng.submit(GenerationRequest(
            prompt_ids=list(p), max_new_tokens=10,
            sampling=SamplingParams(greedy=True))) for p in prompts]
        for r in reqs:
            while r.done_ts is None:
                r.out_queue.get(timeout=60)
        for p, r in zip(prompts, reqs):
            assert len(r.output_ids) == 10 and r.error is None
            seq = list(p)
            for tok in r.output_ids:
                logits = oracle_logits(cfg, W, seq)[-1]
                top2 = torch.topk(logits, 2).values
                if float(top2[0] - top2[1]) > 1e-3:
                    assert int(logits.argmax()) == tok
                seq.append(tok)
    finally:
        eng.shutdown()


def test_trace_replay_writes_wanted_logits(tmp_path, monkeypatch, capsys):
    from bee2bee_amd.engine import trace

    cfg = _cfg("other-order")
    W = O.random_weights(cfg, seed=17)
    O.save_checkpoint(str(tmp_path / "m"), cfg, W)
    toks = random_tokens(12, cfg["vocab"], 6)
    steps = [
        {"step": 0, "entries": [{"id": "q", "tokens": toks[:7], "want": [0, 6]}],
         "end": []},
        {"step": 1, "entries": [{"id": "q", "tokens": toks[7:8], "want": []}],
         "end": []},
        {"step": 2, "entries": [{"id": "q", "tokens": toks[8:], "want": [3]}],
         "end": ["q"]},
    ]
    monkeypatch.setattr(sys, "stdin", io.StringIO(
        "\n".join(json.dumps(s) for s in steps) + "\n"))
    out = tmp_path / "out"
    assert trace.main(["--model", str(tmp_path / "m"), "--dtype", "float32",
                       "--out", str(out), "--max-tokens", "64"]) == 0
    assert capsys.readouterr().out.split() == ["done", "0", "done", "1",
                                               "done", "2"]
    import numpy as np

    want = oracle_logits(cfg, W, toks)
    a = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(2, -1))
    c = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(1, -1))
    assert not (out / "1.f32").exists()
    assert rel_err(a, want[[0, 6]]) < 2e-4 and rel_err(c, want[[11]]) < 2e-4


def test_checkpoint_roundtrip(tmp_path):
    """load -> save_hf -> load: the same tensors under the same names, the
    same config, the same layers."""
    from safetensors.torch import load_file

    from bee2bee_amd.models.weights import safetensors_shapes, save_hf

    for name in ("base", "other-order"):
        cfg = _cfg(name)
        W = O.random_weights(cfg, seed=18)
        eng = make_engine(tmp_path / name, cfg, W)
        out = tmp_path / name / "resaved"
        save_hf(eng.weights, str(out))
        W2 = load_file(str(out / "model.safetensors"))
        assert set(W2) == set(W)
        for k in W2:
            assert W2[k].shape == W[k].shape, k
            # norm weights are held as 1 + w in fp32
            assert torch.allclose(W2[k].float(), W[k].float(), rtol=0,
                                  atol=1e-6 if "norm" in k else 0), k
        cfg2 = json.load(open(out / "config.json"))
        a, b = losivik_spec("a", cfg), losivik_spec("b", cfg2)
        assert a.layer_specs == b.layer_specs == eng.spec.layer_specs
        assert (a.side_dim, a.embed_scale) == (b.side_dim, b.embed_scale)
        # every tensor counts once in the parameter count
        n = sum(math.prod(s) for s in
                safetensors_shapes(str(out)).values())
        assert eng.spec.n_params() == n


def test_random_init_runs_and_is_consistent():
    """Synthetic serving (no checkpoint): random weights of a synthetic
    stack; decoding token by token equals the whole prompt."""
    from bee2bee_amd.engine.engine import InferenceEngine
    from bee2bee_amd.models.hybrid import losivik_layer_cfgs

    layers = losivik_layer_cfgs(6, 32, heads=4, kv_heads=2, dim=8, window=12,
                                keep_first=2, kv_rank=12, ssd_heads=4,
                                ssd_vdim=6, state=10, groups=2, taps=3,
                                experts=4, top_k=2, expert_ff=16, ff=24)
    assert {(l["type"], l["mlp"]["kind"]) for l in layers} == {
        (a, b) for a in ("parallel", "latent_attention")
        for b in ("dense", "moe")}
    spec = losivik_spec("lo-synth", {
        "vocab": 64, "width": 32, "norm": {"eps": 1e-6}, "layers": layers,
        "embedding": {"scale": 4.0}, "token_side": {"dim": 5},
        "max_seq_len": 256})
    eng = InferenceEngine(spec, device="cpu", dtype=F32, max_batch=2,
                          max_seq_len=256, use_graphs=False, kv_block_size=8,
                          kv_blocks=16, kv_margin_blocks=1)
    toks = random_tokens(20, 64, 9)
    whole = replay(eng, {"a": toks}, [[("a", 20)]])["a"]
    steps = replay(eng, {"a": toks}, [[("a", 1)]] * 20)["a"]
    assert float(row_errs(steps, whole).max()) < 1e-4
    assert spec.n_params() > spec.active_params_per_token() > 0


def test_bench_compare_option_runs_on_cpu():
    """bench.py --compare-losivik: one JSON line per model with prefill and
    decode throughput (CPU run: small stand-in sizes)."""
    import os
    import subprocess

    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run(
        [sys.executable, os.path.join(repo, "bench.py"), "--compare-losivik",
         "s", "--steps", "1", "--warmup", "0"],
        capture_output=True, text=True, timeout=300,
        env=dict(os.environ, HIP_VISIBLE_DEVICES="", CUDA_VISIBLE_DEVICES=""))
    assert r.returncode == 0, r.stderr[-2000:]
    lines = [json.loads(x) for x in r.stdout.splitlines() if x.startswith("{")]
    assert [x["model"] for x in lines] == ["losivik-s", "tudatar-s",
                                           "gqa-moe-s"]
    for x in lines:
        assert x["compare"] == "losivik-vs-others"
        assert x["prefill_tokens_per_s"] > 0 and x["decode_tokens_per_s"] > 0
