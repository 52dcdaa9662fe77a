"""Tudatar on the CPU reference path against the plain oracle
(tests/tudatar_oracle.py): each mechanism alone, then the served model —
whole prompts, decoding, portions, mixed batches with page and slot reuse,
far keys, window and page edges, the scheduler's own greedy generation."""
import io
import json
import math
import sys

import pytest
import torch

from bee2bee_amd.models.spec import tudatar_spec
from bee2bee_amd.ops import reference as ref
from tests import tudatar_oracle as O
from tests.tudatar_util import (assert_logits, chunk_schedule, make_engine,
                                oracle_logits, planted_attention,
                                random_tokens, rel_err, replay, row_errs)

F32, F64 = torch.float32, torch.float64


def i32(x):
    return torch.tensor(x, dtype=torch.int32)


def pages(lens, starts, bs, seed=0):
    """Packed-chunk metadata with scattered pages."""
    g = torch.Generator().manual_seed(seed)
    need = [-(-(s + L) // bs) for L, s in zip(lens, starts)]
    nb = sum(need) + 2
    perm = torch.randperm(nb, generator=g).tolist()
    bt = torch.zeros(len(lens), max(need), dtype=torch.int32)
    k = 0
    for b in range(len(lens)):
        for j in range(need[b]):
            bt[b, j] = perm[k]
            k += 1
    cu, pos, seq = [0], [], []
    for b, (L, s) in enumerate(zip(lens, starts)):
        cu.append(cu[-1] + L)
        pos += list(range(s, s + L))
        seq += [b] * L
    slot = [int(bt[b, p // bs]) * bs + p % bs for b, p in zip(seq, pos)]
    return dict(cu=i32(cu), pos=i32(pos), seq=i32(seq), bt=bt, slot=i32(slot),
                nb=nb, T=cu[-1])


# ----------------------------------------------------------- mechanisms

@pytest.mark.parametrize("W", [1, 5, 24])
def test_tanh_norm_pair(W):
    torch.manual_seed(0)
    x, y = torch.randn(4, W) * 3, torch.randn(4, W) * 2
    ws = {}
    for n, a in (("post", 0.8), ("pre", 0.3)):
        ws[n], ws[n + ".b"] = torch.randn(W), torch.randn(W)
        ws[n + ".alpha"] = torch.tensor(a)

    def n3(n):
        return float(ws[n + ".alpha"]), ws[n], ws[n + ".b"]

    want_x = x.double() + O.tanh_norm(ws, "post", y.double())
    r = x.clone()
    got = ref.add_tanh_norm(r, y, n3("post"), n3("pre"), F32)
    assert torch.allclose(r.double(), want_x, atol=1e-5)
    assert torch.allclose(got.double(), O.tanh_norm(ws, "pre", want_x),
                          atol=1e-5)
    # only the pre-norm; only the update
    r = x.clone()
    got = ref.add_tanh_norm(r, None, None, n3("pre"), F32)
    assert torch.equal(r, x)
    assert torch.allclose(got.double(), O.tanh_norm(ws, "pre", x.double()),
                          atol=1e-5)
    assert ref.add_tanh_norm(r, y, n3("post"), None, F32) is None
    # large inputs saturate at +-w + b, whatever their size
    big = ref.tanh_norm(torch.full((1, W), 1e6), n3("pre"), F32)
    assert torch.allclose(big, (ws["pre"] + ws["pre.b"])[None])


@pytest.mark.parametrize("scaling", [
    None, {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0},
    {"factor": 1.0, "original": 64, "fast": 8.0, "slow": 1.0},
    # lo clamps at 0, hi clamps at dims - 1
    {"factor": 8.0, "original": 7, "fast": 32.0, "slow": 1.0},
    {"factor": 2.0, "original": 10 ** 9, "fast": 2.0, "slow": 1.0}])
@pytest.mark.parametrize("dims,base", [(2, 50.0), (6, 300.0), (64, 1e6)])
def test_rotation_in_the_latent_store(scaling, dims, base):
    """interleaved pairs, scaled frequencies, the factor on cos and sin;
    coordinates past the rotated ones pass; latent normed; scattered pages
    keep what other rows hold"""
    torch.manual_seed(1)
    H, C, R, bs = 3, 5, dims + 2, 4
    m = pages([5, 2], [3, 0], bs)
    T = m["T"]
    q, kv = torch.randn(T, H, R), torch.randn(T, C + R)
    w = torch.randn(C)
    rot = {"dims": dims, "base": base, "scaling": scaling}
    f, mag = O.rotation(rot)
    cos, sin = ref.rope_tables_scaled(20, dims, base, scaling, "cpu")
    cache = torch.full((m["nb"], bs, C + R), float("nan"))
    q1 = q.clone()
    ref.latent_rope_store(q1, kv, w, 1e-5, C, dims, m["pos"], cos, sin, cache,
                          m["slot"], True)
    for lo, hi, start in ((0, 5, 3), (5, 7, 0)):
        def turn(x):
            pad = torch.zeros(start, x.shape[1], R, dtype=F64)
            return O.rotate_pairs(torch.cat([pad, x.double()]), f, mag)[start:]
        assert torch.allclose(q1[lo:hi].double(), turn(q[lo:hi]), atol=1e-5)
        kr = turn(kv[lo:hi, None, C:])[:, 0]
        lat = O.unit(kv[lo:hi, :C].double(), 1e-5) * w.double()
        for t in range(lo, hi):
            s = int(m["slot"][t])
            row = cache[s // bs, s % bs].double()
            assert torch.allclose(row[:C], lat[t - lo], atol=1e-5)
            assert torch.allclose(row[C:], kr[t - lo], atol=1e-5)
    assert int(torch.isnan(cache[..., 0]).sum()) == m["nb"] * bs - T


@pytest.mark.parametrize("v_unit", [True, False])
def test_projection_norm_and_store(v_unit):
    """one root mean square for all heads of a projection; heads of unequal
    size show that it is not taken per head"""
    torch.manual_seed(2)
    H, G, D, Dv, bs = 3, 2, 5, 4, 4
    m = pages([5, 2], [3, 0], bs)
    T = m["T"]
    q, k, v = (torch.randn(T, n, d) for n, d in ((H, D), (G, D), (G, Dv)))
    q[:, 0] *= 20.0
    k[:, 1] *= 20.0
    wq, wk = torch.randn(H * D), torch.randn(G * D)
    kc = torch.full((m["nb"], G, bs, D), float("nan"))
    vc = torch.full((m["nb"], G, bs, Dv), float("nan"))
    q1 = q.clone()
    ref.proj_norm_store(q1, k, v, wq, wk, v_unit, 1e-5, 0.7, kc, vc, m["slot"])
    un = lambda x: O.unit(x.double(), 1e-5)
    want_q = un(q.reshape(T, -1)) * wq.double() * 0.7
    assert torch.allclose(q1.double().view(T, -1), want_q, atol=1e-5)
    want_k = (un(k.reshape(T, -1)) * wk.double()).view(T, G, D)
    want_v = un(v) if v_unit else v.double()
    for t in range(T):
        s = int(m["slot"][t])
        assert torch.allclose(kc[s // bs, :, s % bs].double(), want_k[t],
                              atol=1e-5)
        assert torch.allclose(vc[s // bs, :, s % bs].double(), want_v[t],
                              atol=1e-5)
    per_head = un(q) * wq.double().view(H, D) * 0.7
    assert float((per_head - q1.double()).abs().max()) > 0.1


@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 6, 5), (3, 3, 4, 4), (6, 1, 3, 7),
                                      (1, 1, 2, 1)])
@pytest.mark.parametrize("window", [0, 1, 2, 7, 100])
@pytest.mark.parametrize("sched", [[23], [2] * 11 + [1], [1] * 23,
                                   [10, 1, 7, 2, 3]])
def test_distance_biased_attention(H, G, D, Dv, window, sched):
    torch.manual_seed(3)
    T, bs = 23, 4
    q, k, v = torch.randn(T, H, D), torch.randn(T, G, D), torch.randn(T, G, Dv)
    dist = torch.stack([torch.randn(H), torch.rand(H) * 3])
    m = pages([T], [0], bs, seed=window)
    kc = torch.full((m["nb"], G, bs, D), float("nan"))
    vc = torch.full((m["nb"], G, bs, Dv), float("nan"))
    out = torch.zeros(T, H * Dv)
    at = 0
    for n in sched:
        pos = i32(list(range(at, at + n)))
        s = m["slot"][at:at + n].long()
        kc[s // bs, :, s % bs] = k[at:at + n]
        vc[s // bs, :, s % bs] = v[at:at + n]
        ref.gqa_attn(q[at:at + n], kc, vc, m["bt"], pos, i32([0] * n),
                     i32([0, n]), 0.0, None, None, None, window,
                     out[at:at + n], dist)
        at += n
    ok = O.visible(T, window)
    for h in range(H):
        g = h // (H // G)
        s = q[:, h].double() @ k[:, g].double().t() - O.distance_bias(
            float(dist[0, h]), float(dist[1, h]), T)
        want = O.softmax_rows(s, ok) @ v[:, g].double()
        got = out[:, h * Dv : (h + 1) * Dv].double()
        assert torch.allclose(got, want, atol=1e-5)


def test_distance_bias_values():
    """equal scores: two keys d and e back share as (1 + r2 d)^-r1 to
    (1 + r2 e)^-r1"""
    H, D, bs, T = 2, 2, 4, 10
    m = pages([T], [0], bs)
    kc = torch.zeros(m["nb"], 1, bs, D)
    vc = torch.zeros(m["nb"], 1, bs, T)
    s = m["slot"].long()
    vc[s // bs, 0, s % bs] = torch.eye(T)
    dist = torch.tensor([[0.5, 2.0], [3.0, 0.25]])
    out = torch.zeros(1, H * T)
    ref.gqa_attn(torch.zeros(1, H, D), kc, vc, m["bt"], i32([T - 1]), i32([0]),
                 i32([0, 1]), 0.0, None, None, None, 0, out, dist)
    for h in range(H):
        a, b = float(dist[0, h]), float(dist[1, h])
        w = [(1 + b * (T - 1 - j)) ** -a for j in range(T)]
        for j in range(T):
            assert abs(float(out[0, h * T + j]) - w[j] / sum(w)) < 1e-6


@pytest.mark.parametrize("sched", [[19], [2] * 9 + [1], [1] * 19, [7, 1, 11]])
@pytest.mark.parametrize("taps", [1, 2, 4])
def test_channel_delta_portions(sched, taps):
    """conv + silu + unit vectors + per-channel decay + delta rule + gated
    head norm through the ops, from a NaN-filled slot, in portions"""
    torch.manual_seed(4)
    H, G, D, Dv, T = 4, 2, 5, 3, 19
    n_q, n = G * D, 2 * G * D + H * Dv
    x, b = torch.randn(T, n), torch.randn(T, H)
    a, gate = torch.randn(T, H * D), torch.randn(T, H * Dv)
    w, dtb = torch.randn(n, taps), torch.randn(H * D)
    A_log, nw = torch.randn(H), torch.randn(Dv)
    y = O.silu(O.short_conv(x.double(), w.double()))
    own = [h // (H // G) for h in range(H)]
    q = (O.unit_length(y[:, :n_q].view(T, G, D)) * D ** -0.5)[:, own]
    k = O.unit_length(y[:, n_q : 2 * n_q].view(T, G, D))[:, own]
    sp = torch.log1p(torch.exp(a.double() + dtb.double())).view(T, H, D)
    g = torch.exp(-torch.exp(A_log.double())[None, :, None] * sp)
    o = O.delta_scan(q, k, y[:, 2 * n_q :].view(T, H, Dv),
                     O.sigmoid(b.double()), g)
    want = (O.unit(o, 1e-5) * nw.double()).reshape(T, -1) * \
        O.sigmoid(gate.double())
    conv_state = torch.full((3, taps - 1, n), float("nan"))
    state = torch.full((3, H, D, Dv), float("nan"))
    got, at, slot = torch.zeros(T, H * Dv), 0, i32([1])
    for c in sched:
        sl = slice(at, at + c)
        pos, cu = i32(list(range(at, at + c))), i32([0, c])
        qkv = ref.short_conv(x[sl], w.t().contiguous(), conv_state, slot, cu,
                             i32([0] * c), pos, True)
        beta, gg = ref.delta_gates(qkv, G, D, b[sl], a[sl], dtb,
                                   torch.exp(A_log), True)
        oo = ref.delta_rule(qkv[:, :n_q].view(c, G, D),
                            qkv[:, n_q : 2 * n_q].view(c, G, D),
                            qkv[:, 2 * n_q :].view(c, H, Dv), beta, gg, state,
                            slot, cu, pos)
        ref.head_gated_norm(oo, nw, gate[sl], "sigmoid", 1e-5, got[sl], 1.0)
        at += c
    assert torch.allclose(got.double(), want, atol=2e-5)


def test_delta_reads_its_own_write_and_decays_rows():
    """one channel kept (decay 1), one dropped (decay 0): the first token's
    write is recalled through the kept channel only; a token's read-out sees
    the token's own write"""
    D, Dv = 2, 1
    q = torch.tensor([[[1.0, 0.0]], [[1.0, 0.0]], [[0.0, 1.0]]])
    k = torch.tensor([[[0.6, 0.8]], [[0.0, 0.0]], [[0.0, 0.0]]])
    v = torch.tensor([[[5.0]], [[0.0]], [[0.0]]])
    g = torch.tensor([1.0, 0.0]).expand(3, D).contiguous()
    o = ref.delta_rule(q, k, v, torch.ones(3, 1), g, torch.zeros(1, 1, D, Dv),
                       i32([0]), i32([0, 3]), i32([0, 1, 2]))
    assert torch.allclose(o.view(-1), torch.tensor([3.0, 3.0, 0.0]))


@pytest.mark.parametrize("E,top", [(5, 2), (4, 4), (1, 1), (9, 3)])
def test_router_choice_bias(E, top):
    torch.manual_seed(5)
    h, r = torch.randn(13, 6), torch.randn(E, 6)
    cor = torch.randn(E)
    W = {"router": r, "correction": cor}
    idx, w = O.route(W, "", {"top": top, "scale": 1.3}, h.double())
    w1, i1 = ref.group_topk_gate(h @ r.t(), top, 1, 1, "sigmoid", 1, cor, True,
                                 1.3)
    a, b = idx.sort(1), i1.long().sort(1)
    assert torch.equal(a.values, b.values)
    assert torch.allclose(w.gather(1, a.indices).float(),
                          w1.gather(1, b.indices), atol=1e-6)
    assert torch.allclose(w1.sum(1), torch.full((13,), 1.3), atol=1e-5)


def test_router_bias_moves_the_choice_not_the_weight():
    logits = torch.tensor([[2.0, 0.0, -1.0, 1.0]])
    cor = torch.tensor([-5.0, 0.0, 3.0, 0.0])       # choice scores < 0 too
    w, i = ref.group_topk_gate(logits, 2, 1, 1, "sigmoid", 1, cor, True, 1.0)
    s = torch.sigmoid(logits[0])
    assert i.tolist() == [[2, 3]]
    assert torch.allclose(w[0], s[[2, 3]] / (s[2] + s[3]))
    # a very negative correction everywhere still chooses `top` experts
    w, i = ref.group_topk_gate(logits, 3, 1, 1, "sigmoid", 1,
                               torch.full((4,), -9.0), False, 2.0)
    assert sorted(i[0].tolist()) == [0, 1, 3]
    assert torch.allclose(w[0], 2.0 * s[i[0].long()])


def test_expert_execution_forms_agree():
    """all experts as two plain products, and the sorted form, against the
    oracle's per-token loop"""
    torch.manual_seed(6)
    E, top, ff, Wd, T = 5, 2, 7, 6, 17
    h = torch.randn(T, Wd)
    W = {"router": torch.randn(E, Wd), "correction": torch.randn(E) * 0.2}
    for e in range(E):
        W.update({f"e{e}.gate": torch.randn(ff, Wd),
                  f"e{e}.up": torch.randn(ff, Wd),
                  f"e{e}.down": torch.randn(Wd, ff)})
    f = {"router": {"top": top, "scale": 0.8}}
    want = O.moe(W, "", f, h.double())
    wts, idx = ref.group_topk_gate(h @ W["router"].t(), top, 1, 1, "sigmoid",
                                   1, W["correction"], True, 0.8)
    gu_w = torch.stack([torch.cat([W[f"e{e}.gate"], W[f"e{e}.up"]])
                        for e in range(E)])
    down = torch.cat([W[f"e{e}.down"] for e in range(E)], 1)
    gu = (h @ gu_w.view(E * 2 * ff, Wd).t()).view(T, E, 2 * ff)
    got = ref.routed_silu_glu(gu, wts, idx) @ down.t()
    assert torch.allclose(got.double(), want, atol=1e-4)
    # an expert that was not chosen adds nothing even where it overflows
    gu[:, 0] = float("inf")
    y = ref.routed_silu_glu(gu, wts, idx).view(T, E, ff)
    assert torch.equal(y[:, 0][~(idx == 0).any(1)],
                       torch.zeros(int((~(idx == 0).any(1)).sum()), ff))
    pos, tok, offs = ref.moe_sort(idx, E)
    xs, y = h[tok.long()], torch.empty(T * top, Wd)
    for e in range(E):
        a, b = int(offs[e]), int(offs[e + 1])
        assert bool((idx.reshape(-1)[torch.argsort(pos.reshape(-1))][a:b]
                     == e).all())
        y[a:b] = ref.silu_glu(xs[a:b] @ gu_w[e].t()) @ W[f"e{e}.down"].t()
    assert torch.allclose(ref.moe_combine(y, pos, wts).double(), want,
                          atol=1e-4)


def test_config_parsing():
    cfg = O.make_config(no_mlp=(2,))
    spec = tudatar_spec("t", cfg)
    d, a, la, _ = [l.mixer for l in spec.layer_specs]
    assert (d.kind, d.channel_decay, d.gate, d.taps) == ("delta", True,
                                                         "sigmoid", 3)
    assert (a.kind, a.proj_norm, a.v_norm, a.distance_bias, a.bias,
            a.out_bias, a.rope_dims, a.window) == \
        ("gqa_attention", True, True, True, True, False, 0, 9)
    assert (la.window, la.head_gate, la.sink, la.rope_layout) == \
        (0, False, False, "interleaved")
    assert la.rope_scaling == {"factor": 3.0, "original": 40.0, "fast": 4.0,
                               "slow": 1.0}
    f = spec.layer_specs[0].ffn
    assert (f.n_experts, f.top_k, f.renorm, f.choice_bias, f.route_scale,
            f.act, f.score) == (5, 2, True, True, 1.7, "silu_glu",
                                "sigmoid_all")
    assert spec.layer_specs[2].ffn is None
    assert spec.logit_scale == 0.6 and spec.is_hybrid
    with pytest.raises(ValueError):
        tudatar_spec("t", O.make_config(heads=4, kv_heads=3))
    with pytest.raises(ValueError):
        tudatar_spec("t", O.make_config(top=6))
    bad = O.make_config()
    bad["layers"][1]["type"] = "retention"
    with pytest.raises(ValueError):
        tudatar_spec("t", bad)


# ------------------------------------------------------------ the model

VARIANTS = {
    "base": dict(),
    # values that other models make equal or 1
    "ones": dict(heads=1, kv_heads=1, dim=1, vdim=1, window=1, lat_heads=1,
                 lat_dim=1, rot_dim=2, lat_vdim=1, kv_rank=1, q_rank=1,
                 delta_heads=1, delta_kv=1, delta_dim=1, delta_vdim=1, conv=1,
                 experts=1, top=1, ff=1),
    "equal": dict(width=16, heads=4, kv_heads=4, dim=8, vdim=8, window=16,
                  lat_heads=4, lat_dim=8, rot_dim=8, lat_vdim=8, kv_rank=8,
                  q_rank=8, delta_heads=4, delta_kv=4, delta_dim=8,
                  delta_vdim=8, experts=4, top=4, ff=16, conv=4),
    "other-order": dict(kinds=("latent_attention", "channel_delta",
                               "channel_delta", "attention",
                               "latent_attention"), heads=6, kv_heads=1,
                        dim=4, vdim=12, window=33, conv=5, scaling=False,
                        no_mlp=(1, 4), experts=9, top=3, delta_heads=6,
                        delta_kv=3, logit_scale=2.5),
    "latent-wide": dict(kinds=("latent_attention", "attention"), lat_heads=5,
                        lat_dim=3, rot_dim=10, lat_vdim=7, kv_rank=24,
                        q_rank=30, window=5, no_mlp=(0, 1), base=20.0,
                        scaling={"factor": 16.0, "original": 12, "fast": 1.5,
                                 "slow": 0.5}),
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


@pytest.mark.parametrize("window,far", [(8, 3), (8, 4), (16, 0), (17, 15),
                                        (5, 16), (200, 1), (300, 130)])
@pytest.mark.parametrize("sched", ["whole", "decode", "portions"])
def test_window_edge_shows(tmp_path, window, far, sched):
    """A planted key takes nearly all weight while it is visible: the row
    window - 1 after it still sees it, the next one does not. Cut as one
    prompt, as decoding, as portions whose borders fall around the edge."""
    T = far + window + 6
    cfg, W, toks = planted_attention(window, far, T)
    eng = make_engine(tmp_path, cfg, W, block_size=4, kv_blocks=120)
    steps = {"whole": [[("a", T)]],
             "decode": [[("a", 2)]] + [[("a", 1)]] * (T - 2),
             "portions": chunk_schedule("a", T, [far + window - 1, 2, 3])
             }[sched]
    got = replay(eng, {"a": toks}, steps)["a"]
    want = oracle_logits(cfg, W, toks)
    assert_logits(got, want, F32)
    inside, outside = got[far + window - 1], got[far + window]
    assert float(inside[0]) > 0.8 * float(got[far][0])
    assert abs(float(outside[0])) < 0.05 * float(inside[0])


@pytest.mark.parametrize("j", [0, 15, 16, 131])
@pytest.mark.parametrize("sched", [[300], [280] + [1] * 20])
def test_latent_far_key_among_hundreds(j, sched):
    """one key far back — the first token, both sides of a page border —
    dominates among 300; every later row returns its latent row, without a
    gate or a sink"""
    torch.manual_seed(9)
    H, C, R, T, bs = 2, 6, 2, 300, 16
    lat = torch.randn(T, C) * 0.05
    lat[j] = torch.tensor([4.0, -3.0, 2.0, 1.0, -2.0, 3.0])
    m = pages([T], [0], bs)
    cache = torch.full((m["nb"], bs, C + R), float("nan"))
    cache.view(-1, C + R)[m["slot"].long()] = torch.cat(
        [lat, torch.zeros(T, R)], -1)
    q_abs = (lat[j] * 3.0).expand(H, T, C).contiguous()
    got, at = [], 0
    for n in sched:
        got.append(ref.latent_attn(
            q_abs[:, at:at + n].contiguous(), torch.zeros(n, H, R), None,
            cache, m["bt"], i32(list(range(at, at + n))), i32([0] * n),
            i32([0, n]), 0, 1.0))
        at += n
    got = torch.cat(got, 1)
    for t in (j, j + 1, 299):
        assert torch.allclose(got[:, t], lat[j].expand(H, C), atol=1e-3), t
    if j > 0:       # rows before it do not see it
        assert float(got[:, j - 1].abs().max()) < 1.0


def test_mixed_batches_and_reuse(tmp_path):
    """Unequal requests side by side (portions next to single tokens, a
    request sitting out a step) equal each request alone; the pool is far
    smaller than the sum of the requests, so pages and slots come back."""
    cfg = _cfg("base")
    W = O.random_weights(cfg, seed=13)
    eng = make_engine(tmp_path, cfg, W, kv_blocks=7, block_size=8,
                      max_batch=3)
    # reused pages and slots hold garbage, never zeros
    for t in eng.kv.k_cache + eng.kv.v_cache + eng.kv.rec_state + \
            eng.kv.conv_state:
        if t is not None:
            t.fill_(float("nan"))
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
    cfg = _cfg("base")                    # window 9, pages of 4
    W = O.random_weights(cfg, seed=14)
    eng = make_engine(tmp_path, cfg, W, block_size=4, kv_blocks=50)
    toks = random_tokens(140, cfg["vocab"], 3)
    got = replay(eng, {"a": toks}, [[("a", 3)]] + [[("a", 1)]] * 137)["a"]
    assert_logits(got, oracle_logits(cfg, W, toks), F32)


def test_first_tokens_after_page_and_slot_reuse(tmp_path):
    """A request that takes over the pages and the slot another one just
    left must not see anything of it in its first tokens (conv rows,
    recurrent state, keys)."""
    cfg = _cfg("other-order")
    W = O.random_weights(cfg, seed=15)
    eng = make_engine(tmp_path, cfg, W, max_batch=1, kv_blocks=3, block_size=16)
    a, b = random_tokens(40, cfg["vocab"], 4), random_tokens(6, cfg["vocab"], 5)
    replay(eng, {"a": a}, [[("a", 40)]])
    for sched in ([[("b", 6)]], [[("b", 1)]] * 6, [[("b", 2)], [("b", 4)]]):
        got = replay(eng, {"b": b}, sched)["b"]
        assert_logits(got, oracle_logits(cfg, W, b), F32)


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
            assert torch.equal(W2[k].float(), W[k].float()), k
        cfg2 = json.load(open(out / "config.json"))
        shapes = safetensors_shapes(str(out))
        a, b = tudatar_spec("a", cfg, shapes), tudatar_spec("b", cfg2, shapes)
        assert a.layer_specs == b.layer_specs == eng.spec.layer_specs
        assert a.logit_scale == b.logit_scale
        # every tensor counts once in the parameter count
        n = sum(math.prod(s) for s in shapes.values())
        assert abs(eng.spec.n_params() - n) <= 2 * cfg["width"] + 1


def test_random_init_runs_and_is_consistent():
    """Synthetic serving (no checkpoint): random weights of a synthetic
    stack; decoding token by token equals the whole prompt."""
    from bee2bee_amd.engine.engine import InferenceEngine
    from bee2bee_amd.models.hybrid import tudatar_layer_cfgs

    layers = tudatar_layer_cfgs(3, 32, heads=4, kv_heads=2, dim=8, window=12,
                                kv_rank=12, rot_dim=4, q_rank=10,
                                delta_heads=4, delta_kv_heads=2, delta_dim=6,
                                rank=5, taps=3, experts=4, top_k=2,
                                expert_ff=16)
    spec = tudatar_spec("td-synth", {
        "vocab": 64, "width": 32, "norm": {"eps": 1e-6}, "layers": layers,
        "logit_scale": 0.5, "max_seq_len": 256})
    eng = InferenceEngine(spec, device="cpu", dtype=F32, max_batch=2,
                          max_seq_len=256, use_graphs=False, kv_block_size=8,
                          kv_blocks=16, kv_margin_blocks=1)
    toks = random_tokens(20, 64, 9)
    whole = replay(eng, {"a": toks}, [[("a", 20)]])["a"]
    steps = replay(eng, {"a": toks}, [[("a", 1)]] * 20)["a"]
    assert float(row_errs(steps, whole).max()) < 1e-4
    assert spec.n_params() > spec.active_params_per_token() > 0


def test_bench_compare_option_runs_on_cpu():
    """bench.py --compare-tudatar: one JSON line per model with prefill and
    decode throughput (CPU run: small stand-in sizes)."""
    import os
    import subprocess

    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run(
        [sys.executable, os.path.join(repo, "bench.py"), "--compare-tudatar",
         "s", "--steps", "1", "--warmup", "0"],
        capture_output=True, text=True, timeout=300,
        env=dict(os.environ, HIP_VISIBLE_DEVICES="", CUDA_VISIBLE_DEVICES=""))
    assert r.returncode == 0, r.stderr[-2000:]
    lines = [json.loads(x) for x in r.stdout.splitlines() if x.startswith("{")]
    assert [x["model"] for x in lines] == ["tudatar-s", "zevilorn-s",
                                           "gqa-moe-s"]
    for x in lines:
        assert x["compare"] == "tudatar-vs-others"
        assert x["prefill_tokens_per_s"] > 0 and x["decode_tokens_per_s"] > 0
