"""HIP kernels of the dynamic-tanh stacks (the norm pair around the residual
update, query/key norms over the whole projection with the page store, the
distance bias in the grouped-query attention kernels incl. the matrix-core
path, the latent attention without a gate and its interleaved rotation, the
router with a choice bias, the sort and weighted sum of routed experts)
against the fp32 torch reference of the same op (ops/reference.py), in bf16
and fp32, at sizes that are neither powers of two nor multiples of the wave
size, on column slices of wider buffers as the runner passes them."""
import pytest
import torch

from bee2bee_amd import ops
from bee2bee_amd.ops import reference as ref

pytestmark = pytest.mark.gpu

if not torch.cuda.is_available():
    pytest.skip("needs a GPU", allow_module_level=True)

from tests.test_hybrid_ops_gpu import DEV, DTYPES, batch_meta, tol  # noqa: E402


def _norm(W):
    return 0.7, torch.randn(W, device=DEV), torch.randn(W, device=DEV)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [1, 37, 48, 200, 1028, 4096])
def test_add_tanh_norm(dtype, W):
    torch.manual_seed(0)
    T = 6
    x = torch.randn(T, W, device=DEV) * 3
    y = (torch.randn(T, W, device=DEV) * 2).to(dtype)
    for yy, post, pre in ((y, _norm(W), _norm(W)), (None, None, _norm(W)),
                          (y, _norm(W), None)):
        r1, r2 = x.clone(), x.clone()
        o1 = ops.add_tanh_norm(r1, yy, post, pre, dtype)
        o2 = ref.add_tanh_norm(r2, yy, post, pre, dtype)
        torch.testing.assert_close(r1, r2, rtol=2e-6, atol=4e-6)
        if pre is None:
            assert o1 is None and o2 is None
        else:
            torch.testing.assert_close(o1.float(), o2.float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 96, 96), (3, 1, 7, 5),
                                      (16, 4, 128, 128), (6, 6, 20, 36),
                                      (1, 1, 1, 1)])
@pytest.mark.parametrize("v_unit", [True, False])
def test_proj_norm_store(dtype, H, G, D, Dv, v_unit):
    torch.manual_seed(1)
    bs = 16
    m = batch_meta([9, 1, 4], [5, 30, 0], bs, 8, 1)
    T = m["T"]
    n = H * D + G * D + G * Dv
    wide = (torch.randn(T, (n + 23) // 8 * 8, device=DEV) * 2).to(dtype)
    wq, wk = (torch.randn(k * D, device=DEV) for k in (H, G))
    res = []
    for mod in (ops, ref):
        w = wide.clone()
        q = w[:, : H * D].view(T, H, D)
        k = w[:, H * D : (H + G) * D].view(T, G, D)
        v = w[:, (H + G) * D : n].view(T, G, Dv)
        kc = torch.full((8, G, bs, D), 7.0, device=DEV, dtype=dtype)
        vc = torch.full((8, G, bs, Dv), 7.0, device=DEV, dtype=dtype)
        mod.proj_norm_store(q, k, v, wq, wk, v_unit, 1e-5, 0.37, kc, vc,
                            m["slot_map"])
        res.append((w, kc, vc))
    for a, b in zip(*res):
        torch.testing.assert_close(a.float(), b.float(), **tol(dtype))


def _dist_case(dtype, lens, starts, H, G, D, Dv, window, bs=16, seed=3):
    torch.manual_seed(seed)
    need = sum(-(-(s + L) // bs) for L, s in zip(lens, starts))
    m = batch_meta(lens, starts, bs, need + 2, seed)
    T = m["T"]
    kc = torch.randn(need + 2, G, bs, D, device=DEV).to(dtype)
    vc = torch.randn(need + 2, G, bs, Dv, device=DEV).to(dtype)
    q = (torch.randn(T, H, D, device=DEV) * D ** -0.5).to(dtype)
    dist = torch.stack([torch.randn(H, device=DEV) + 0.5,
                        torch.rand(H, device=DEV) * 3])
    outs = []
    for mod, kw in ((ops, {"max_qlen": max(lens)}), (ref, {})):
        out = torch.zeros(T, H * Dv, device=DEV, dtype=dtype)
        mod.gqa_attn(q, kc, vc, m["bt"], m["pos"], m["seq"], m["cu"], 0.0,
                     None, None, None, window, out, dist=dist, **kw)
        outs.append(out.float())
    return outs


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,Dv", [(8, 8, 96, 96), (3, 1, 7, 5),
                                      (8, 2, 64, 64), (6, 3, 20, 33)])
@pytest.mark.parametrize("window", [0, 1, 9, 72])
def test_distance_biased_attention(dtype, H, G, D, Dv, window):
    """mixed steps, prompt portions and decode steps with key splits"""
    for lens, starts in (([33, 1, 2, 1], [0, 47, 15, 0]),
                         ([40, 17], [0, 30]),
                         ([1, 1, 1, 1, 1], [0, 47, 15, 600, 95])):
        a, b = _dist_case(dtype, lens, starts, H, G, D, Dv, window)
        torch.testing.assert_close(a, b, **tol(dtype))


@pytest.mark.parametrize("D,G", [(64, 4), (128, 2)])
@pytest.mark.parametrize("window", [0, 1, 63, 64, 65, 100])
def test_distance_biased_attention_matrix_core(D, G, window):
    """bf16 prompt portions of head size 64/128: windows that end inside,
    at and before a key tile, chunks with history, a chunk shorter than a
    tile, single rows riding along"""
    a, b = _dist_case(torch.bfloat16, [70, 1, 130, 16, 1],
                      [0, 200, 57, 500, 0], 2 * G, G, D, D, window, 32)
    torch.testing.assert_close(a, b, rtol=2e-2, atol=4e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,C,R,dims", [(4, 96, 32, 32), (3, 7, 10, 6),
                                        (16, 128, 64, 64)])
@pytest.mark.parametrize("inter", [True, False])
def test_latent_store_layouts_and_attention_without_gate(dtype, H, C, R, dims,
                                                         inter):
    torch.manual_seed(4)
    bs = 16
    for lens, starts in (([33, 1, 2, 1], [0, 47, 15, 0]), ([40, 17], [0, 30]),
                         ([1, 1, 1, 1, 1], [0, 47, 15, 200, 95])):
        need = sum(-(-(s + L) // bs) for L, s in zip(lens, starts))
        m = batch_meta(lens, starts, bs, need + 2, 4)
        T = m["T"]
        cos, sin = ref.rope_tables_scaled(
            256, dims, 1e4, {"factor": 4.0, "original": 64, "fast": 8.0,
                             "slow": 1.0}, DEV)
        q = torch.randn(T, H, 5 + R, device=DEV).to(dtype)
        kv = torch.randn(T, C + R + 3, device=DEV).to(dtype)[:, : C + R]
        w = torch.rand(C, device=DEV) + 0.5
        base = torch.randn(need + 2, bs, C + R, device=DEV).to(dtype)
        q1, q2, c1, c2 = q.clone(), q.clone(), base.clone(), base.clone()
        ops.latent_rope_store(q1[..., 5:], kv, w, 1e-5, C, dims, m["pos"],
                              cos, sin, c1, m["slot_map"], inter)
        ref.latent_rope_store(q2[..., 5:], kv, w, 1e-5, C, dims, m["pos"],
                              cos, sin, c2, m["slot_map"], inter)
        torch.testing.assert_close(q1.float(), q2.float(), **tol(dtype))
        torch.testing.assert_close(c1.float(), c2.float(), **tol(dtype))
        qa = (torch.randn(H, T, C, device=DEV) * C ** -0.5).to(dtype)
        args = (qa, q2[..., 5:], None, c2, m["bt"], m["pos"], m["seq"],
                m["cu"], 0, 0.2)
        torch.testing.assert_close(
            ops.latent_attn(*args, max(lens)).float(),
            ref.latent_attn(*args).float(), **tol(dtype))


@pytest.mark.parametrize("E,top,groups,keep", [
    (8, 3, 1, 1), (1, 1, 1, 1), (9, 9, 1, 1), (64, 8, 8, 4), (128, 6, 1, 1),
    (300, 5, 1, 1)])
@pytest.mark.parametrize("score", ["sigmoid", "softmax"])
@pytest.mark.parametrize("shift", [0.0, -4.0])
def test_router_choice_bias(E, top, groups, keep, score, shift):
    torch.manual_seed(5)
    logits = torch.randn(333, E, device=DEV) * 2
    cb = torch.randn(E, device=DEV) + shift
    args = (logits, top, groups, keep, score, 2, cb, True, 1.6)
    w1, i1 = ops.group_topk_gate(*args)
    w2, i2 = ref.group_topk_gate(*args)
    o1, o2 = i1.long().sort(1), i2.long().sort(1)
    assert torch.equal(o1.values, o2.values)
    torch.testing.assert_close(w1.gather(1, o1.indices),
                               w2.gather(1, o2.indices), rtol=1e-4,
                               atol=1e-6)


@pytest.mark.parametrize("T,E,k", [(1, 1, 1), (3, 5, 2), (700, 8, 2),
                                   (5000, 13, 3), (9000, 64, 6)])
def test_moe_sort_and_combine(T, E, k):
    torch.manual_seed(6)
    idx = torch.rand(T, E, device=DEV).topk(k, dim=1).indices.to(torch.int32)
    got, want = ops.moe_sort(idx, E), ref.moe_sort(idx, E)
    for a, b in zip(got, want):
        assert a.dtype == torch.int32 and torch.equal(a, b.to(a.dtype))
    # one expert takes everything, the others nothing
    idx = torch.full((T, 1), E - 1, dtype=torch.int32, device=DEV)
    for a, b in zip(ops.moe_sort(idx, E), ref.moe_sort(idx, E)):
        assert torch.equal(a, b.to(a.dtype))
    for W in (5, 36):
        for dtype in DTYPES:
            y = torch.randn(T * k, W, device=DEV).to(dtype)
            wt = torch.rand(T, k, device=DEV)
            torch.testing.assert_close(
                ops.moe_combine(y, got[0], wt).float(),
                ref.moe_combine(y, got[0], wt).float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,I,k", [(8, 64, 3), (5, 7, 2), (1, 1, 1),
                                   (4, 516, 4)])
def test_routed_silu_glu(dtype, E, I, k):
    torch.manual_seed(7)
    T = 11
    gu = torch.randn(T, E, 2 * I, device=DEV).to(dtype)
    idx = torch.rand(T, E, device=DEV).topk(k, dim=1).indices.to(torch.int32)
    wt = torch.rand(T, k, device=DEV) + 0.1
    # what was not chosen must not enter, whatever it holds
    dead = torch.ones(T, E, dtype=torch.bool, device=DEV)
    dead.scatter_(1, idx.long(), False)
    gu[dead] = float("nan")
    a = ops.routed_silu_glu(gu, wt, idx)
    b = ref.routed_silu_glu(gu, wt, idx)
    torch.testing.assert_close(a.float(), b.float(), **tol(dtype))
    assert not bool(torch.isnan(a).any())


def test_grouped_gemm_on_a_strided_weight_view():
    torch.manual_seed(8)
    E, N, K, S = 3, 128, 256, 200
    cat = (torch.randn(N, E * K, device=DEV) * K ** -0.5).bfloat16()
    w = cat.view(N, E, K).permute(1, 0, 2)
    x = torch.randn(S, K, device=DEV).bfloat16()
    offs = torch.tensor([0, 50, 50, S], dtype=torch.int32, device=DEV)
    a = ops.grouped_gemm(x, w, offs)
    assert torch.equal(a, ops.grouped_gemm(x, w.contiguous(), offs))
    torch.testing.assert_close(a.float(),
                               ref.grouped_gemm(x, w, offs).float(),
                               rtol=2e-2, atol=2e-2)
