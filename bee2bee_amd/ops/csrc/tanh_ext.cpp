// Torch bindings for the dynamic-tanh stack kernels (tanh_stack.hip).
// Shapes, strides and dtypes are validated here so the kernels index without
// checks. Activations are bf16 or fp32; residual and norm weights are fp32.
// All entry points are hipGraph-capture safe (no sync, no host reads).
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include <hip/hip_runtime.h>

#include <optional>

using torch::Tensor;

extern "C" {
void launch_add_tanh_norm(float*, const void*, float, const float*,
                          const float*, float, const float*, const float*,
                          void*, long, int, int, int, int, hipStream_t);
void launch_proj_norm_store(void*, long, int, const void*, long, const void*,
                            long, int, int, int, const float*, const float*,
                            int, float, float, void*, void*, int, const int*,
                            long, int, int, hipStream_t);
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

// base address and row stride allow 4-element accesses
bool aligned4(const Tensor& t) {
    return t.stride(0) % 4 == 0 &&
           reinterpret_cast<uintptr_t>(t.data_ptr()) %
                   (4 * t.element_size()) == 0;
}

const float* norm_vec(const std::optional<Tensor>& t, int W, const char* name,
                      bool& vec) {
    TORCH_CHECK(t.has_value(), name, " is missing");
    check_f32(*t, name);
    TORCH_CHECK(t->numel() == W, name, " must have one number per column");
    vec = vec && reinterpret_cast<uintptr_t>(t->data_ptr()) % 16 == 0;
    return t->data_ptr<float>();
}

std::optional<Tensor> add_tanh_norm(Tensor& resid,
                                    const std::optional<Tensor>& y, double pa,
                                    const std::optional<Tensor>& pw,
                                    const std::optional<Tensor>& pb, double na,
                                    const std::optional<Tensor>& nw,
                                    const std::optional<Tensor>& nb,
                                    at::ScalarType out_dtype) {
    check_f32(resid, "resid");
    TORCH_CHECK(resid.dim() == 2);
    const long T = resid.size(0);
    const int W = (int)resid.size(1);
    const int oc = act_code(out_dtype, "out_dtype");
    int yc = oc;
    bool vec = W % 4 == 0 && aligned4(resid);
    const void* yp = nullptr;
    const float *pwp = nullptr, *pbp = nullptr, *nwp = nullptr,
                *nbp = nullptr;
    if (y.has_value()) {
        yc = act_code(*y, "y");
        TORCH_CHECK(y->is_contiguous() && y->sizes() == resid.sizes());
        yp = y->data_ptr();
        vec = vec && aligned4(*y);
        pwp = norm_vec(pw, W, "post-norm weight", vec);
        pbp = norm_vec(pb, W, "post-norm bias", vec);
    }
    std::optional<Tensor> out;
    void* op = nullptr;
    if (nw.has_value()) {
        nwp = norm_vec(nw, W, "pre-norm weight", vec);
        nbp = norm_vec(nb, W, "pre-norm bias", vec);
        out = torch::empty(resid.sizes(), resid.options().dtype(out_dtype));
        op = out->data_ptr();
    }
    launch_add_tanh_norm(resid.data_ptr<float>(), yp, (float)pa, pwp, pbp,
                         (float)na, nwp, nbp, op, T, W, yc, oc, vec ? 1 : 0,
                         stream());
    return out;
}

void proj_norm_store(Tensor& q, const Tensor& k, const Tensor& v,
                     const Tensor& q_norm, const Tensor& k_norm, bool v_unit,
                     double eps, double q_mult, Tensor& k_cache,
                     Tensor& v_cache, const Tensor& slot_mapping) {
    const int c = act_code(q, "q");
    check_f32(q_norm, "q_norm");
    check_f32(k_norm, "k_norm");
    check_i32(slot_mapping, "slot_mapping");
    TORCH_CHECK(q.dim() == 3 && k.dim() == 3 && v.dim() == 3);
    const long T = q.size(0);
    const int H = (int)q.size(1), D = (int)q.size(2);
    const int G = (int)k.size(1), Dv = (int)v.size(2);
    TORCH_CHECK(k.size(0) == T && v.size(0) == T && k.size(2) == D &&
                v.size(1) == G);
    bool vec = D % 4 == 0 && Dv % 4 == 0;
    for (const Tensor* t : {(const Tensor*)&q, &k, &v}) {
        TORCH_CHECK(t->is_cuda() && t->scalar_type() == q.scalar_type() &&
                        t->stride(2) == 1 &&
                        (t->size(1) == 1 || t->stride(1) == t->size(2)),
                    "q, k, v must be slices with contiguous head rows");
        vec = vec && aligned4(*t);
    }
    TORCH_CHECK(q_norm.numel() == (long)H * D && k_norm.numel() == (long)G * D);
    for (const Tensor* t : {(const Tensor*)&k_cache, (const Tensor*)&v_cache})
        TORCH_CHECK(t->is_cuda() && t->is_contiguous() && t->dim() == 4 &&
                    t->scalar_type() == q.scalar_type() && t->size(1) == G);
    TORCH_CHECK(k_cache.size(3) == D && v_cache.size(3) == Dv &&
                v_cache.size(0) == k_cache.size(0) &&
                v_cache.size(2) == k_cache.size(2));
    TORCH_CHECK(slot_mapping.numel() == T);
    for (const Tensor* t : {&q_norm, &k_norm})
        vec = vec && reinterpret_cast<uintptr_t>(t->data_ptr()) % 16 == 0;
    launch_proj_norm_store(
        q.data_ptr(), q.stride(0), H, k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), G, D, Dv, q_norm.data_ptr<float>(),
        k_norm.data_ptr<float>(), v_unit ? 1 : 0, (float)eps, (float)q_mult,
        k_cache.data_ptr(), v_cache.data_ptr(), (int)k_cache.size(2),
        slot_mapping.data_ptr<int>(), T, c, vec ? 1 : 0, stream());
}

}  // namespace

void register_tanh_ops(pybind11::module_& m) {
    m.def("add_tanh_norm", &add_tanh_norm,
          "resid += tanh(a y) w + b; out = tanh(a' resid) w' + b'");
    m.def("proj_norm_store", &proj_norm_store,
          "q/k norm over the whole projection, value norm; keys and values "
          "to the pages");
}
