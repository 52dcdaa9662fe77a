// Torch bindings for the routed-expert plumbing (moe.hip). Shapes, strides
// and dtypes are validated here so the kernels index without checks.
// Activations are bf16 or fp32; routing weights are fp32. All entry points
// are hipGraph-capture safe (no sync, no host reads).
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include <hip/hip_runtime.h>

#include <vector>

using torch::Tensor;

extern "C" {
void launch_moe_sort(const int*, long, int, int, int*, int*, int*,
                     hipStream_t);
void launch_moe_combine(const void*, const int*, const float*, void*, long,
                        int, int, int, int, hipStream_t);
void launch_routed_silu_glu(const void*, const float*, const int*, void*, long,
                            int, int, int, int, int, hipStream_t);
void launch_routed_relu2(const void*, const float*, const int*, void*, long,
                         int, int, int, int, int, int, hipStream_t);
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

// idx [T, k] int32, every entry in [0, n_experts) -> [pos, tok, offs]
std::vector<Tensor> moe_sort(const Tensor& idx, int64_t n_experts) {
    check_i32(idx, "idx");
    TORCH_CHECK(idx.dim() == 2 && n_experts >= 1);
    Tensor pos = torch::empty_like(idx);
    Tensor tok = torch::empty({idx.numel()}, idx.options());
    Tensor offs = torch::empty({n_experts + 1}, idx.options());
    launch_moe_sort(idx.data_ptr<int>(), idx.numel(), (int)idx.size(1),
                    (int)n_experts, pos.data_ptr<int>(), tok.data_ptr<int>(),
                    offs.data_ptr<int>(), stream());
    return {pos, tok, offs};
}

Tensor moe_combine(const Tensor& y, const Tensor& pos,
                   const Tensor& weights) {
    const int c = act_code(y, "y");
    check_i32(pos, "pos");
    check_f32(weights, "weights");
    TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && pos.dim() == 2 &&
                weights.sizes() == pos.sizes() && y.size(0) == pos.numel());
    const long T = pos.size(0);
    const int W = (int)y.size(1);
    Tensor out = torch::empty({T, (long)W}, y.options());
    const bool vec = W % 4 == 0 && aligned4(y) && aligned4(out);
    launch_moe_combine(y.data_ptr(), pos.data_ptr<int>(),
                       weights.data_ptr<float>(), out.data_ptr(), T, W,
                       (int)pos.size(1), c, vec ? 1 : 0, stream());
    return out;
}

Tensor routed_silu_glu(const Tensor& gu, const Tensor& weights,
                       const Tensor& idx) {
    const int c = act_code(gu, "gate_up");
    check_f32(weights, "weights");
    check_i32(idx, "idx");
    TORCH_CHECK(gu.dim() == 3 && gu.is_contiguous() && gu.size(2) % 2 == 0);
    const long T = gu.size(0);
    const int E = (int)gu.size(1), I = (int)gu.size(2) / 2;
    TORCH_CHECK(weights.dim() == 2 && weights.size(0) == T &&
                idx.sizes() == weights.sizes());
    Tensor out = torch::empty({T, (long)E * I}, gu.options());
    const bool vec = I % 4 == 0 && aligned4(gu) && aligned4(out);
    launch_routed_silu_glu(gu.data_ptr(), weights.data_ptr<float>(),
                           idx.data_ptr<int>(), out.data_ptr(), T, E, I,
                           (int)weights.size(1), c, vec ? 1 : 0, stream());
    return out;
}

// z [T, E * ff + n]: the experts' input products, then n always-on columns
Tensor routed_relu2(const Tensor& z, const Tensor& weights, const Tensor& idx,
                    int64_t n_experts, int64_t ff) {
    const int c = act_code(z, "z");
    check_f32(weights, "weights");
    check_i32(idx, "idx");
    TORCH_CHECK(z.dim() == 2 && z.is_contiguous() && n_experts >= 1 &&
                ff >= 1 && z.size(1) >= n_experts * ff);
    const long T = z.size(0);
    const int N = (int)z.size(1);
    TORCH_CHECK(weights.dim() == 2 && weights.size(0) == T &&
                idx.sizes() == weights.sizes());
    Tensor out = torch::empty_like(z);
    const bool vec = ff % 4 == 0 && N % 4 == 0 && aligned4(z) && aligned4(out);
    launch_routed_relu2(z.data_ptr(), weights.data_ptr<float>(),
                        idx.data_ptr<int>(), out.data_ptr(), T,
                        (int)n_experts, (int)ff, N, (int)weights.size(1), c,
                        vec ? 1 : 0, stream());
    return out;
}

}  // namespace

void register_moe_ops(pybind11::module_& m) {
    m.def("moe_sort", &moe_sort, "(token, choice) pairs in expert order");
    m.def("moe_combine", &moe_combine,
          "weighted sum of each token's expert outputs");
    m.def("routed_silu_glu", &routed_silu_glu,
          "silu GLU of every expert times the routing weight");
    m.def("routed_relu2", &routed_relu2,
          "relu(w z)^2 of every expert, relu(z)^2 of the always-on columns");
}
