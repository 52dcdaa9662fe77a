// Torch bindings for the scaled parallel-form stack kernels (scaled.hip,
// ssd.hip). Shapes, strides and dtypes are validated here so the kernels
// index without checks. Activations are bf16 or fp32; residual, norm weights,
// scales and recurrent state are fp32. All entry points are hipGraph-capture
// safe (no sync, no host reads).
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include <hip/hip_runtime.h>

#include <optional>
#include <vector>

using torch::Tensor;

extern "C" {
void launch_embed_sinusoid(const long*, const void*, float, const int*,
                           const double*, float*, long, int, long, int,
                           hipStream_t);
void launch_scaled_add(float*, const void*, const float*, const void*,
                       const float*, const void*, void*, long, int, int, int,
                       hipStream_t);
void launch_add_norm_pair(float*, const void*, const float*, const float*,
                          const float*, void*, void*, long, int, float, int,
                          int, hipStream_t);
void launch_side_gate(const void*, const void*, long, long, const long*,
                      void*, long, int, long, int, hipStream_t);
void launch_gated_group_norm(const float*, long, const void*, long,
                             const float*, void*, long, long, int, int, float,
                             float, int, int, hipStream_t);
int launch_attn_prefill_packed(const unsigned short*, long,
                               const unsigned short*, long,
                               const unsigned short*, long, const int*,
                               unsigned short*, long, int, int, int, int, int,
                               float, float, int, const unsigned short*, long,
                               hipStream_t);
int ssd_piece_tokens();
int launch_ssd_scan(const void*, long, const void*, long, const float*,
                    const float*, const float*, float*, const int*,
                    const int*, const int*, float*, float*, double*, float*,
                    float*, float*, int*, int, int, int, int, int, int, int,
                    int, hipStream_t);
}

namespace {

inline hipStream_t stream() {
    return at::hip::getCurrentHIPStreamMasqueradingAsCUDA().stream();
}

// 0 = bf16, 1 = fp32
int act_code(at::ScalarType t, const char* name) {
    TORCH_CHECK(t == torch::kBFloat16 || t == torch::kFloat32, name,
                " must be bf16 or fp32");
    return t == torch::kFloat32 ? 1 : 0;
}

int act_code(const Tensor& t, const char* name) {
    TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
    return act_code(t.scalar_type(), name);
}

void check_f32(const Tensor& t, const char* name) {
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kFloat32 &&
                    t.is_contiguous(),
                name, " must be a contiguous fp32 GPU tensor");
}

void check_i32(const Tensor& t, const char* name) {
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt32 &&
                    t.is_contiguous(),
                name, " must be a contiguous int32 GPU tensor");
}

// a [T, n] view with unit column stride (a column slice of a wider buffer)
void check_slice(const Tensor& t, long T, long n, at::ScalarType dt,
                 const char* name) {
    TORCH_CHECK(t.is_cuda() && t.scalar_type() == dt && t.dim() == 2 &&
                    t.size(0) == T && t.size(1) == n &&
                    (n == 1 || t.stride(1) == 1),
                name, ": expected a [", T, ", ", n, "] column slice");
}

// base address and row stride allow 4-element accesses
bool aligned4(const Tensor& t) {
    return (t.dim() < 2 || t.stride(0) % 4 == 0) &&
           reinterpret_cast<uintptr_t>(t.data_ptr()) %
                   (4 * t.element_size()) == 0;
}

// rows are held in LDS as fp32
constexpr long MAX_ROW = 16000;

const float* vec_ptr(const Tensor& t, long W, const char* name, bool& vec) {
    check_f32(t, name);
    TORCH_CHECK(t.numel() == W, name, " must have one number per column");
    vec = vec && aligned4(t.view({-1}));
    return t.data_ptr<float>();
}

const void* row_ptr(const Tensor& t, const Tensor& resid, const char* name,
                    bool& vec) {
    act_code(t, name);
    TORCH_CHECK(t.sizes() == resid.sizes() && t.is_contiguous(), name,
                " must be contiguous with the residual's shape");
    vec = vec && aligned4(t);
    return t.data_ptr();
}

Tensor embed_sinusoid(const Tensor& ids, const Tensor& table, double scale,
                      const Tensor& positions, const Tensor& freqs) {
    const int c = act_code(table, "table");
    check_i32(positions, "positions");
    TORCH_CHECK(ids.is_cuda() && ids.scalar_type() == torch::kInt64 &&
                ids.dim() == 1 && ids.is_contiguous());
    const long T = ids.numel();
    TORCH_CHECK(table.dim() == 2 && table.is_contiguous() &&
                positions.numel() == T);
    const int W = (int)table.size(1);
    TORCH_CHECK(freqs.is_cuda() && freqs.scalar_type() == torch::kFloat64 &&
                freqs.is_contiguous() && freqs.numel() == (W + 1) / 2);
    Tensor x = torch::empty({T, (long)W},
                            table.options().dtype(torch::kFloat32));
    launch_embed_sinusoid((const long*)ids.data_ptr<int64_t>(),
                          table.data_ptr(), (float)scale,
                          positions.data_ptr<int>(), freqs.data_ptr<double>(),
                          x.data_ptr<float>(), T, W, table.size(0), c,
                          stream());
    return x;
}

Tensor scaled_add(Tensor& resid, const Tensor& y1, const Tensor& s1,
                  const std::optional<Tensor>& y2,
                  const std::optional<Tensor>& s2,
                  const std::optional<Tensor>& y3,
                  at::ScalarType out_dtype) {
    check_f32(resid, "resid");
    TORCH_CHECK(resid.dim() == 2);
    const long T = resid.size(0), W = resid.size(1);
    const int c = act_code(out_dtype, "out_dtype");
    bool vec = W % 4 == 0 && aligned4(resid);
    const void* p1 = row_ptr(y1, resid, "y1", vec);
    const float* f1 = vec_ptr(s1, W, "s1", vec);
    const void *p2 = nullptr, *p3 = nullptr;
    const float* f2 = nullptr;
    TORCH_CHECK(y1.scalar_type() == out_dtype);
    if (y2.has_value()) {
        TORCH_CHECK(y2->scalar_type() == out_dtype && s2.has_value());
        p2 = row_ptr(*y2, resid, "y2", vec);
        f2 = vec_ptr(*s2, W, "s2", vec);
        if (y3.has_value()) {
            TORCH_CHECK(y3->scalar_type() == out_dtype);
            p3 = row_ptr(*y3, resid, "y3", vec);
        }
    }
    Tensor out = resid;
    void* op = nullptr;
    if (out_dtype != torch::kFloat32) {
        out = torch::empty(resid.sizes(), resid.options().dtype(out_dtype));
        op = out.data_ptr();
    }
    launch_scaled_add(resid.data_ptr<float>(), p1, f1, p2, f2, p3, op, T,
                      (int)W, c, vec ? 1 : 0, stream());
    return out;
}

std::vector<std::optional<Tensor>> add_norm_pair(
    Tensor& resid, const std::optional<Tensor>& y,
    const std::optional<Tensor>& w_post, const std::optional<Tensor>& wa,
    const std::optional<Tensor>& wb, double eps, at::ScalarType out_dtype) {
    check_f32(resid, "resid");
    TORCH_CHECK(resid.dim() == 2 && resid.size(1) <= MAX_ROW);
    const long T = resid.size(0), W = resid.size(1);
    const int c = act_code(out_dtype, "out_dtype");
    bool vec = W % 4 == 0 && aligned4(resid);
    const void* yp = nullptr;
    const float *pp = nullptr, *ap = nullptr, *bp = nullptr;
    if (y.has_value()) {
        TORCH_CHECK(y->scalar_type() == out_dtype && w_post.has_value());
        yp = row_ptr(*y, resid, "y", vec);
        pp = vec_ptr(*w_post, W, "w_post", vec);
    }
    std::optional<Tensor> oa, ob;
    void *pa = nullptr, *pb = nullptr;
    auto opt = resid.options().dtype(out_dtype);
    if (wa.has_value()) {
        ap = vec_ptr(*wa, W, "wa", vec);
        oa = torch::empty(resid.sizes(), opt);
        pa = oa->data_ptr();
    }
    if (wb.has_value()) {
        bp = vec_ptr(*wb, W, "wb", vec);
        ob = torch::empty(resid.sizes(), opt);
        pb = ob->data_ptr();
    }
    launch_add_norm_pair(resid.data_ptr<float>(), yp, pp, ap, bp, pa, pb, T,
                         (int)W, (float)eps, c, vec ? 1 : 0, stream());
    return {oa, ob};
}

Tensor side_gate(const Tensor& g, const Tensor& table, int64_t offset,
                 const Tensor& ids) {
    const int c = act_code(g, "g");
    TORCH_CHECK(g.dim() == 2 && g.is_contiguous());
    const long T = g.size(0);
    const int d = (int)g.size(1);
    TORCH_CHECK(table.is_cuda() && table.scalar_type() == g.scalar_type() &&
                table.dim() == 2 && table.is_contiguous() && offset >= 0 &&
                offset + d <= table.size(1));
    TORCH_CHECK(ids.is_cuda() && ids.scalar_type() == torch::kInt64 &&
                ids.numel() == T && ids.is_contiguous());
    Tensor out = torch::empty_like(g);
    launch_side_gate(g.data_ptr(), table.data_ptr(), table.size(1), offset,
                     (const long*)ids.data_ptr<int64_t>(), out.data_ptr(), T,
                     d, table.size(0), c, stream());
    return out;
}

void gated_group_norm(const Tensor& y, const Tensor& z, const Tensor& w,
                      int64_t groups, double eps, Tensor& out,
                      double out_scale) {
    check_f32(y, "y");
    TORCH_CHECK(y.dim() == 2);
    const long T = y.size(0), N = y.size(1);
    const int c = act_code(z, "z");
    check_slice(z, T, N, z.scalar_type(), "z");
    check_slice(out, T, N, z.scalar_type(), "out");
    TORCH_CHECK(groups >= 1 && N % groups == 0 && N / groups <= MAX_ROW);
    const long n = N / groups;
    bool vec = n % 4 == 0 && aligned4(y) && aligned4(z) && aligned4(out);
    const float* wp = vec_ptr(w, N, "w", vec);
    launch_gated_group_norm(y.data_ptr<float>(), N, z.data_ptr(), z.stride(0),
                            wp, out.data_ptr(), out.stride(0), T, (int)groups,
                            (int)n, (float)eps, (float)out_scale, c,
                            vec ? 1 : 0, stream());
}

Tensor ssd_scan(const Tensor& xbc, const Tensor& dt, const Tensor& dt_bias,
                const Tensor& rate, const Tensor& skip, int64_t groups,
                Tensor& state, const Tensor& state_slots, const Tensor& cu,
                const Tensor& positions, int64_t max_qlen) {
    const int c = act_code(xbc, "xbc");
    check_f32(dt_bias, "dt_bias");
    check_f32(rate, "rate");
    check_f32(skip, "skip");
    check_f32(state, "state");
    check_i32(state_slots, "state_slots");
    check_i32(cu, "cu_seqlens");
    check_i32(positions, "positions");
    TORCH_CHECK(state.dim() == 4 && xbc.dim() == 2);
    const long T = xbc.size(0);
    const int H = (int)state.size(1), N = (int)state.size(2),
              V = (int)state.size(3), G = (int)groups;
    TORCH_CHECK(G >= 1 && H % G == 0);
    const long cols = (long)H * V + 2L * G * N;
    check_slice(xbc, T, cols, xbc.scalar_type(), "xbc");
    check_slice(dt, T, H, xbc.scalar_type(), "dt");
    TORCH_CHECK(dt_bias.numel() == H && rate.numel() == H &&
                skip.numel() == H);
    const int B = (int)cu.numel() - 1;
    TORCH_CHECK(state_slots.numel() == B && positions.numel() == T);
    auto f32opt = state.options();
    Tensor y = torch::empty({T, (long)H * V}, f32opt);
    // portions past this length: 64-token pieces in parallel. `pieces`
    // bounds the batch's piece count without reading the lengths.
    long pieces = 0;
    Tensor ws, logs, per_tok, fade, table;
    float *wp = nullptr, *steps = nullptr, *tails = nullptr, *fp = nullptr;
    double* lp = nullptr;
    int* tp = nullptr;
    if (max_qlen > 16) {
        const long L = ssd_piece_tokens();
        pieces = T / L + B;
        ws = torch::empty({pieces, (long)H, (long)N, (long)V}, f32opt);
        logs = torch::empty({pieces, (long)H, L},
                            f32opt.dtype(torch::kFloat64));
        per_tok = torch::empty({2, pieces, (long)H, L}, f32opt);
        fade = torch::empty({pieces, (long)H}, f32opt);
        table = torch::empty({pieces, 2}, f32opt.dtype(torch::kInt32));
        wp = ws.data_ptr<float>();
        lp = logs.data_ptr<double>();
        steps = per_tok.data_ptr<float>();
        tails = steps + pieces * H * L;
        fp = fade.data_ptr<float>();
        tp = table.data_ptr<int>();
    }
    const bool vec = N % 4 == 0 && V % 4 == 0 && xbc.stride(0) % 4 == 0 &&
                     reinterpret_cast<uintptr_t>(xbc.data_ptr()) % 16 == 0 &&
                     reinterpret_cast<uintptr_t>(state.data_ptr()) % 16 == 0;
    const int rc = launch_ssd_scan(
        xbc.data_ptr(), xbc.stride(0), dt.data_ptr(), dt.stride(0),
        dt_bias.data_ptr<float>(), rate.data_ptr<float>(),
        skip.data_ptr<float>(), state.data_ptr<float>(),
        state_slots.data_ptr<int>(), cu.data_ptr<int>(),
        positions.data_ptr<int>(), y.data_ptr<float>(), wp, lp, steps, tails,
        fp, tp, (int)pieces, B, H, G, N, V, c, vec ? 1 : 0, stream());
    TORCH_CHECK(rc == 0, "ssd_scan: state size must be <= 512");
    return y;
}

// q [T, H, D], k, v [T, G, D]: rows whose heads lie side by side (bf16, D 64
// or 128); gate [T, H] raw or none -> [T, H * D]
Tensor packed_attn(const Tensor& q, const Tensor& k, const Tensor& v,
                   const Tensor& cu, double scale, int64_t window,
                   const std::optional<Tensor>& gate, int64_t max_qlen) {
    check_i32(cu, "cu_seqlens");
    TORCH_CHECK(q.dim() == 3 && k.dim() == 3 && v.sizes() == k.sizes() &&
                window >= 0 && max_qlen >= 1);
    const long T = q.size(0);
    const int H = (int)q.size(1), D = (int)q.size(2), G = (int)k.size(1);
    TORCH_CHECK(k.size(0) == T && k.size(2) == D && G >= 1 && H % G == 0);
    for (const Tensor* t : {&q, &k, &v})
        TORCH_CHECK(t->is_cuda() && t->scalar_type() == torch::kBFloat16 &&
                        t->stride(2) == 1 && t->stride(1) == D &&
                        t->stride(0) % 8 == 0 &&
                        reinterpret_cast<uintptr_t>(t->data_ptr()) % 16 == 0,
                    "packed_attn: bf16 rows on 16-byte boundaries");
    const unsigned short* gp = nullptr;
    long gs = 0;
    if (gate.has_value()) {
        check_slice(*gate, T, H, torch::kBFloat16, "gate");
        gp = (const unsigned short*)gate->data_ptr();
        gs = gate->stride(0);
    }
    Tensor out = torch::empty({T, (long)H * D}, q.options());
    const int rc = launch_attn_prefill_packed(
        (const unsigned short*)q.data_ptr(), q.stride(0),
        (const unsigned short*)k.data_ptr(), k.stride(0),
        (const unsigned short*)v.data_ptr(), v.stride(0), cu.data_ptr<int>(),
        (unsigned short*)out.data_ptr(), out.stride(0), (int)cu.numel() - 1,
        H, G, D, (int)max_qlen, (float)scale, 1.f, (int)window, gp, gs,
        stream());
    TORCH_CHECK(rc == 0, "packed_attn: head size must be 64 or 128");
    return out;
}

}  // namespace

void register_scaled_ops(pybind11::module_& m) {
    m.def("embed_sinusoid", &embed_sinusoid,
          "scaled embedding + sinusoidal position vector -> fp32");
    m.def("scaled_add", &scaled_add,
          "resid(fp32) += s1*y1 + s2*(y2 + y3); -> resid, activation type");
    m.def("add_norm_pair", &add_norm_pair,
          "resid(fp32) += unit(y)*w; -> two weighted norms of resid");
    m.def("side_gate", &side_gate, "gelu_tanh(g) * token side row");
    m.def("gated_group_norm", &gated_group_norm,
          "group_norm(y * silu(z)) * w into a column slice");
    m.def("packed_attn", &packed_attn,
          "windowed causal attention of whole prompts on packed keys");
    m.def("ssd_scan", &ssd_scan,
          "state-space recurrence with carried fp32 state");
}
