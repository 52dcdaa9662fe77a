"""HIP kernels of the scaled parallel-form stacks (embedding with sinusoidal
positions, scaled residual update, side norm + pair of norms, side gate,
state-space recurrence in its serial and chunk-parallel forms, gated grouped
norm, relu^2 experts with the weight on the input) and the options the
existing kernels gained (kept first tokens in the grouped-query attention,
values of their own beside per-head normed keys, a bias on the short conv, a
latent row without a rotated part) against the fp32 torch reference of the
same op (ops/reference.py), in bf16 and fp32, at sizes that are neither
powers of two nor multiples of the wave size, on column slices of wider
buffers as the runner passes them."""
import pytest
import torch

from bee2bee_amd import ops
from bee2bee_amd.ops import reference as ref

pytestmark = pytest.mark.gpu

if not torch.cuda.is_available():
    pytest.skip("needs a GPU", allow_module_level=True)

from tests.test_hybrid_ops_gpu import DEV, DTYPES, batch_meta, tol  # noqa: E402
from tests.test_pugozen_ops_gpu import sliced  # noqa: E402


def both(name, *args, **kw):
    """The op and its reference on equal copies of every tensor."""
    res = []
    for mod in (ops, ref):
        a = [x.clone() if torch.is_tensor(x) and x.is_contiguous() else x
             for x in args]
        res.append((getattr(mod, name)(*a, **kw), a))
    return res


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [1, 37, 48, 1030])
def test_embed_sinusoid(dtype, W):
    torch.manual_seed(0)
    table = torch.randn(50, W, device=DEV).to(dtype)
    ids = torch.randint(0, 50, (7,), device=DEV)
    pos = torch.tensor([0, 1, 2, 63, 1000, 31999, 100000], device=DEV,
                       dtype=torch.int32)
    a = ops.embed_sinusoid(ids, table, 3.5, pos)
    # against an evaluation on the host
    f = ref.sinusoid_freqs(W, "cpu")
    b = ref.embed_sinusoid(ids.cpu(), table.cpu(), 3.5, pos.cpu(), f)
    assert a.dtype == torch.float32
    torch.testing.assert_close(a.cpu(), b, rtol=1e-6, atol=2e-6)
    bad = ops.embed_sinusoid(torch.full_like(ids, 50), table, 3.5, pos)
    assert bool(bad.isnan().all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [1, 37, 48, 1028, 4096])
def test_residual_kernels(dtype, W):
    torch.manual_seed(1)
    T = 6
    x = torch.randn(T, W, device=DEV) * 3
    y1, y2, y3 = ((torch.randn(T, W, device=DEV) * 2).to(dtype)
                  for _ in range(3))
    s1, s2, wp, wa, wb = (torch.randn(W, device=DEV) for _ in range(5))
    for a2, b2, a3 in ((None, None, None), (y2, s2, None), (y2, s2, y3)):
        (o, ia), (p, ib) = both("scaled_add", x, y1, s1, a2, b2, a3, dtype)
        torch.testing.assert_close(ia[0], ib[0], rtol=2e-6, atol=4e-6)
        assert o.dtype == dtype
        torch.testing.assert_close(o.float(), p.float(), **tol(dtype))
    for y, w, a, b in ((None, None, wa, wb), (y1, wp, wa, wb),
                       (y1, wp, None, None), (y1, wp, wa, None),
                       (y1, wp, None, wb)):
        (o, ia), (p, ib) = both("add_norm_pair", x, y, w, a, b, 1e-5, dtype)
        torch.testing.assert_close(ia[0], ib[0], rtol=2e-6, atol=4e-6)
        for u, v, wt in zip(o, p, (a, b)):
            assert (u is None) == (wt is None)
            if u is not None:
                torch.testing.assert_close(u.float(), v.float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d,off", [(1, 0), (28, 56), (37, 11)])
def test_side_gate(dtype, d, off):
    torch.manual_seed(2)
    g = (torch.randn(9, d, device=DEV) * 2).to(dtype)
    table = torch.randn(33, off + d + 5, device=DEV).to(dtype)
    ids = torch.randint(0, 33, (9,), device=DEV)
    (a, _), (b, _) = both("side_gate", g, table, off, ids)
    torch.testing.assert_close(a.float(), b.float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,groups", [(12, 3), (37, 1), (128, 2), (2048, 1),
                                      (2048, 8), (30, 30)])
def test_gated_group_norm(dtype, N, groups):
    torch.manual_seed(3)
    T = 5
    y = torch.randn(T, N, device=DEV) * 3
    z = sliced(T, N, dtype, 8, scale=2.0)
    w = torch.randn(N, device=DEV)
    o1 = sliced(T, N, dtype, 8)
    o2 = o1.clone()
    ops.gated_group_norm(y, z, w, groups, 1e-5, o1, 0.7)
    ref.gated_group_norm(y, z, w, groups, 1e-5, o2, 0.7)
    torch.testing.assert_close(o1.float(), o2.float(), **tol(dtype))


SSD_SHAPES = [(4, 2, 7, 6), (4, 2, 32, 48), (3, 1, 24, 40), (2, 2, 1, 1),
              (4, 1, 128, 64), (2, 1, 200, 20), (2, 2, 16, 100), (6, 3, 9, 33),
              (1, 1, 300, 8), (2, 1, 130, 128)]


def _ssd_case(dtype, H, G, N, V, lens, starts, rate=1.0, seed=4):
    torch.manual_seed(seed)
    need = sum(-(-(s + L) // 16) for L, s in zip(lens, starts))
    m = batch_meta(lens, starts, 16, need + 1)
    T = m["T"]
    xbc = torch.randn(T, H * V + 2 * G * N, device=DEV).to(dtype)
    dt = sliced(T, H, dtype, 3)
    dt_bias = torch.randn(H, device=DEV) - 1.0
    rates = torch.exp(torch.randn(H, device=DEV)) * rate
    skip = torch.randn(H, device=DEV)
    st1 = torch.randn(m["state_slots"].max() + 2, H, N, V, device=DEV)
    for i, s in enumerate(starts):
        if s == 0:      # must not be read
            st1[m["state_slots"].long()[i]] = float("nan")
    st2 = st1.clone()
    y1 = ops.ssd_scan(xbc, dt, dt_bias, rates, skip, G, st1,
                      m["state_slots"], m["cu"], m["pos"], max(lens))
    y2 = ref.ssd_scan(xbc, dt, dt_bias, rates, skip, G, st2,
                      m["state_slots"], m["cu"], m["pos"])
    assert y1.dtype == torch.float32
    scale = float(y2.abs().max())
    torch.testing.assert_close(y1, y2, rtol=2e-4, atol=2e-6 * scale + 2e-5)
    live = m["state_slots"].long()
    scale = float(st2[live].abs().max())
    torch.testing.assert_close(st1[live], st2[live], rtol=2e-4,
                               atol=2e-6 * scale + 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,N,V", SSD_SHAPES)
def test_ssd_scan_serial(dtype, H, G, N, V):
    _ssd_case(dtype, H, G, N, V, [1, 1, 1, 1, 1], [0, 7, 1, 3, 900])
    _ssd_case(dtype, H, G, N, V, [2, 1, 16, 9], [0, 7, 1, 3])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,N,V", SSD_SHAPES)
def test_ssd_scan_chunk_parallel(dtype, H, G, N, V):
    """portions that end inside, at and just past a 64-token piece, single
    rows riding along, a portion of many pieces"""
    _ssd_case(dtype, H, G, N, V, [64, 1, 65, 17, 63], [0, 7, 5, 0, 130])
    _ssd_case(dtype, H, G, N, V, [330, 2, 128], [3, 0, 0])


@pytest.mark.parametrize("lens", [[1, 1], [16, 3], [200, 64]])
@pytest.mark.parametrize("rate", [30.0, 0.001])
def test_ssd_scan_decay_extremes(lens, rate):
    """a decay that forgets within a token (running log decays far below
    any difference that matters) and one that forgets nothing"""
    _ssd_case(torch.float32, 4, 2, 40, 24, lens, [5, 0], rate=rate)


def test_ssd_forms_agree():
    """one sequence through the serial form in portions and through the
    chunk-parallel form at once: same outputs, same final state"""
    torch.manual_seed(5)
    H, G, N, V, T = 4, 2, 48, 24, 150
    xbc = torch.randn(T, H * V + 2 * G * N, device=DEV)
    dt = torch.randn(T, H, device=DEV)
    par = (torch.randn(H, device=DEV), torch.rand(H, device=DEV),
           torch.randn(H, device=DEV))
    slots = torch.tensor([1], dtype=torch.int32, device=DEV)
    st = [torch.full((3, H, N, V), float("nan"), device=DEV)
          for _ in range(2)]
    outs = []
    for s, cuts in zip(st, ([150], [16] * 9 + [6])):
        at, ys = 0, []
        for n in cuts:
            cu = torch.tensor([0, n], dtype=torch.int32, device=DEV)
            pos = torch.arange(at, at + n, dtype=torch.int32, device=DEV)
            ys.append(ops.ssd_scan(xbc[at : at + n], dt[at : at + n], *par, G,
                                   s, slots, cu, pos, n))
            at += n
        outs.append(torch.cat(ys))
    torch.testing.assert_close(*outs, rtol=2e-4, atol=2e-5)
    torch.testing.assert_close(st[0][1], st[1][1], rtol=2e-4, atol=2e-5)
    assert bool(st[0][0].isnan().all()) and bool(st[0][2].isnan().all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps,pad", [(40, 4, 8), (37, 3, 3), (24, 1, 8)])
def test_short_conv_bias(dtype, C, taps, pad):
    torch.manual_seed(6)
    m = batch_meta([5, 1, 2, 9], [0, 7, 1, 3], 16, 8)
    x = sliced(m["T"], C, dtype, pad)
    w = torch.randn(taps, C, device=DEV) * 0.5
    b = torch.randn(C, device=DEV)
    st1 = torch.randn(6, max(taps - 1, 0), C, device=DEV).to(dtype)
    st1[m["state_slots"].long()[0]] = float("nan")   # starts at position 0
    st2 = st1.clone()
    for od in (torch.float32, dtype):
        args = (m["state_slots"], m["cu"], m["seq"], m["pos"], True)
        a = ops.short_conv(x, w, st1, *args, bias=b, out_dtype=od)
        c = ref.short_conv(x, w, st2, *args, bias=b, out_dtype=od)
        assert a.dtype == c.dtype == od
        torch.testing.assert_close(a.float(), c.float(), **tol(od))
        live = m["state_slots"].long()
        torch.testing.assert_close(st1[live].float(), st2[live].float(),
                                   rtol=0, atol=0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 96, 40), (3, 1, 7, 5),
                                      (16, 4, 128, 128), (1, 1, 1, 70)])
def test_head_norm_store_with_values(dtype, H, G, D, Dv):
    torch.manual_seed(7)
    bs = 16
    m = batch_meta([9, 1, 4], [5, 30, 0], bs, 8, 1)
    T = m["T"]
    n = H * D + G * D + G * Dv
    wide = (torch.randn(T, (n + 23) // 8 * 8, device=DEV) * 2).to(dtype)
    wq, wk = torch.randn(D, device=DEV), torch.randn(D, device=DEV)
    mult = torch.full((H,), 0.37, device=DEV)
    res = []
    for mod in (ops, ref):
        w = wide.clone()
        q = w[:, : H * D].view(T, H, D)
        k = w[:, H * D : (H + G) * D].view(T, G, D)
        v = w[:, (H + G) * D : n].view(T, G, Dv)
        kc = torch.full((8, G, bs, D), 7.0, device=DEV, dtype=dtype)
        vc = torch.full((8, G, bs, Dv), 7.0, device=DEV, dtype=dtype)
        mod.qk_norm_rope_store(q, k, wq, wk, 1e-5, 0, m["pos"], None, None,
                               mult, kc, vc, m["slot_map"], v=v)
        res.append((w, kc, vc))
    for a, b in zip(*res):
        torch.testing.assert_close(a.float(), b.float(), **tol(dtype))


def _keep_case(dtype, lens, starts, H, G, D, Dv, window, keep, bs=16, seed=3):
    torch.manual_seed(seed)
    need = sum(-(-(s + L) // bs) for L, s in zip(lens, starts))
    m = batch_meta(lens, starts, bs, need + 2, seed)
    T = m["T"]
    kc = torch.randn(need + 2, G, bs, D, device=DEV).to(dtype)
    vc = torch.randn(need + 2, G, bs, Dv, device=DEV).to(dtype)
    q = (torch.randn(T, H, D, device=DEV) * 2 * D ** -0.5).to(dtype)
    outs = []
    for mod, kw in ((ops, {"max_qlen": max(lens)}), (ref, {})):
        out = torch.zeros(T, H * Dv + 8, device=DEV, dtype=dtype)[:, : H * Dv]
        mod.gqa_attn(q, kc, vc, m["bt"], m["pos"], m["seq"], m["cu"], 0.0,
                     None, None, None, window, out, out_scale=0.8,
                     keep_first=keep, **kw)
        outs.append(out.float())
    return outs


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,Dv", [(8, 8, 96, 96), (3, 1, 7, 5),
                                      (8, 2, 64, 64), (6, 3, 20, 33)])
@pytest.mark.parametrize("window,keep", [(1, 1), (9, 3), (72, 20), (5, 100),
                                         (0, 4), (9, 0)])
def test_kept_first_tokens(dtype, H, G, D, Dv, window, keep):
    """mixed steps, prompt portions and decode steps with key splits"""
    for lens, starts in (([33, 1, 2, 1], [0, 47, 15, 0]),
                         ([40, 17], [0, 30]),
                         ([1, 1, 1, 1, 1], [0, 47, 15, 600, 95])):
        a, b = _keep_case(dtype, lens, starts, H, G, D, Dv, window, keep)
        torch.testing.assert_close(a, b, **tol(dtype))


@pytest.mark.parametrize("D,G", [(64, 4), (128, 2)])
@pytest.mark.parametrize("window,keep", [(1, 1), (63, 4), (64, 64), (65, 65),
                                         (100, 3), (40, 130), (300, 2)])
def test_kept_first_tokens_matrix_core(D, G, window, keep):
    """bf16 prompt portions of head size 64/128: kept keys inside, at and
    past a key tile, windows that begin before, in and after them, chunks
    with history, single rows riding along"""
    a, b = _keep_case(torch.bfloat16, [70, 1, 130, 16, 1],
                      [0, 200, 57, 500, 0], 2 * G, G, D, D, window, keep, 32)
    torch.testing.assert_close(a, b, rtol=2e-2, atol=4e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,C", [(4, 64), (3, 7), (16, 128), (5, 96)])
@pytest.mark.parametrize("window", [1, 9, 72])
def test_latent_attention_without_rotated_part(dtype, H, C, window):
    torch.manual_seed(8)
    bs, nb = 16, 64
    for lens, starts in (([33, 1, 2, 1], [0, 47, 15, 0]),
                         ([1, 1, 1], [0, 47, 600])):
        m = batch_meta(lens, starts, bs, nb, 2)
        T = m["T"]
        kv = sliced(T, C, dtype, 8)
        w = torch.randn(C, device=DEV)
        q = (torch.randn(T, H, C, device=DEV)).to(dtype)
        q_abs = (torch.randn(H, T, C, device=DEV) * C ** -0.5).to(dtype)
        gate = sliced(T, H, dtype, 8)
        none = torch.zeros(1, 0, device=DEV)
        cache0 = torch.randn(nb, bs, C, device=DEV).to(dtype)
        outs = []
        for mod, kw in ((ops, {"max_qlen": max(lens)}), (ref, {})):
            cache = cache0.clone()
            mod.latent_rope_store(q[..., C:], kv, w, 1e-5, C, 0, m["pos"],
                                  none, none, cache, m["slot_map"])
            o = mod.latent_attn(q_abs, q[..., C:], gate, cache, m["bt"],
                                m["pos"], m["seq"], m["cu"], window, 0.9, **kw)
            outs.append((cache.float(), o.float()))
        for a, b in zip(*outs):
            torch.testing.assert_close(a, b, **tol(dtype))


@pytest.mark.parametrize("H,G,D", [(4, 4, 64), (2, 1, 128), (6, 3, 64)])
@pytest.mark.parametrize("window", [0, 1, 63, 64, 65, 200])
def test_packed_attention(H, G, D, window):
    """whole prompts on packed keys: windows around a key tile, prompts
    shorter than, at and past a query tile"""
    torch.manual_seed(10)
    lens = [70, 1, 130, 16, 64]
    T = sum(lens)
    cu = torch.tensor([0] + lens, device=DEV).cumsum(0).to(torch.int32)
    wide = torch.randn(T, (H + 2 * G) * D + 16, device=DEV).bfloat16()
    q = wide[:, : H * D].view(T, H, D)
    k = wide[:, H * D : (H + G) * D].view(T, G, D)
    v = wide[:, (H + G) * D : (H + 2 * G) * D].view(T, G, D)
    for gate in (None, sliced(T, H, torch.bfloat16, 8)):
        a = ops.packed_attn(q, k, v, cu, 0.13, window, gate, max(lens))
        b = ref.packed_attn(q, k, v, cu, 0.13, window, gate)
        torch.testing.assert_close(a.float(), b.float(), rtol=2e-2, atol=3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,I,limit", [(7, 5, 1.0), (9, 64, 0.7),
                                          (3, 2052, 7.0)])
def test_clamped_glu_rows(dtype, rows, I, limit):
    torch.manual_seed(11)
    gu = (torch.randn(rows, 2 * I, device=DEV) * 3).to(dtype)
    torch.testing.assert_close(
        ops.clamped_glu(gu, limit, 1.702).float(),
        ref.clamped_glu(gu, limit, 1.702).float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
def test_short_conv_many_tokens(dtype):
    """enough tokens that a workgroup walks several of them, borders of
    sequences inside its share"""
    torch.manual_seed(12)
    lens = [4001, 3, 1, 200]
    m = batch_meta(lens, [0, 7, 1, 3], 16, 300)
    C, taps = 40, 4
    x = sliced(m["T"], C, dtype, 8)
    w, b = torch.randn(taps, C, device=DEV), torch.randn(C, device=DEV)
    st1 = torch.randn(6, taps - 1, C, device=DEV).to(dtype)
    st2 = st1.clone()
    args = (m["state_slots"], m["cu"], m["seq"], m["pos"], True)
    a = ops.short_conv(x, w, st1, *args, bias=b)
    c = ref.short_conv(x, w, st2, *args, bias=b)
    torch.testing.assert_close(a, c, **tol(torch.float32))
    assert torch.equal(st1, st2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,ff,n,k", [(5, 10, 7, 2), (8, 64, 32, 1),
                                      (1, 4, 0, 1), (12, 20, 12, 12)])
def test_routed_relu2(dtype, E, ff, n, k):
    torch.manual_seed(9)
    T = 6
    z = torch.randn(T, E * ff + n, device=DEV).to(dtype)
    idx = torch.stack([torch.randperm(E, device=DEV)[:k] for _ in range(T)])
    idx = idx.to(torch.int32)
    w = torch.rand(T, k, device=DEV)
    ref_out = ref.routed_relu2(z, w, idx, E, ff)
    # columns of experts nobody chose are never read
    for t in range(T):
        for e in range(E):
            if e not in idx[t].tolist():
                z[t, e * ff : (e + 1) * ff] = float("nan")
    out = ops.routed_relu2(z, w, idx, E, ff)
    torch.testing.assert_close(out.float(), ref_out.float(), **tol(dtype))
