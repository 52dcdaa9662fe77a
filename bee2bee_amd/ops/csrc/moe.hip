// Routed-expert plumbing around the expert products: the sort of a step's
// (token, choice) pairs by expert, the weighted sum of a token's expert
// outputs, and the expert activation of steps whose tokens run through every
// expert's columns of one product.
//
// Activations are bf16 (ushort bits) or fp32, routing weights fp32, sums
// fp32. Everything is deterministic: no atomics, fixed orders.
#include "common.h"

namespace {

template <typename T, int VEC> DEV_INLINE void ldn(const T* p, float* o);
template <> DEV_INLINE void ldn<float, 1>(const float* p, float* o) { o[0] = *p; }
template <> DEV_INLINE void ldn<unsigned short, 1>(const unsigned short* p,
                                                   float* o) {
    o[0] = bf2f(*p);
}
template <> DEV_INLINE void ldn<float, 4>(const float* p, float* o) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(p);
    o[0] = v[0]; o[1] = v[1]; o[2] = v[2]; o[3] = v[3];
}
template <> DEV_INLINE void ldn<unsigned short, 4>(const unsigned short* p,
                                                   float* o) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    o[0] = bf2f((unsigned short)(w.x & 0xffffu));
    o[1] = bf2f((unsigned short)(w.x >> 16));
    o[2] = bf2f((unsigned short)(w.y & 0xffffu));
    o[3] = bf2f((unsigned short)(w.y >> 16));
}
template <typename T, int VEC> DEV_INLINE void stn(T* p, const float* o);
template <> DEV_INLINE void stn<float, 1>(float* p, const float* o) { *p = o[0]; }
template <> DEV_INLINE void stn<unsigned short, 1>(unsigned short* p,
                                                   const float* o) {
    *p = f2bf(o[0]);
}
template <> DEV_INLINE void stn<float, 4>(float* p, const float* o) {
    *reinterpret_cast<f32x4*>(p) = f32x4{o[0], o[1], o[2], o[3]};
}
template <> DEV_INLINE void stn<unsigned short, 4>(unsigned short* p,
                                                   const float* o) {
    uint2 w;
    w.x = (unsigned int)f2bf(o[0]) | ((unsigned int)f2bf(o[1]) << 16);
    w.y = (unsigned int)f2bf(o[2]) | ((unsigned int)f2bf(o[3]) << 16);
    *reinterpret_cast<uint2*>(p) = w;
}

constexpr int MO_THREADS = 256;

// ------------------------------------------------------- sort by expert
// idx [S] (S = tokens * top_k, expert of each pair) -> pos [S], the pair's
// row in expert order (pairs of one expert keep their order), tok [S], the
// token of each row, offs [E + 1]. Workgroup per expert: one pass counts the
// pairs of lower experts (its first row), a second one ranks its own pairs
// with wave scans, SORT_PER consecutive pairs a thread.
constexpr int SORT_THREADS = 1024;
constexpr int SORT_PER = 4;
__global__ void __launch_bounds__(SORT_THREADS)
moe_sort_kernel(const int* __restrict__ idx, long S, int top_k, int E,
                int* __restrict__ pos, int* __restrict__ tok,
                int* __restrict__ offs) {
    __shared__ int part[SORT_THREADS / WAVE];
    const int e = blockIdx.x, tid = threadIdx.x;
    const int wid = tid / WAVE, lane = tid % WAVE;
    constexpr int NW = SORT_THREADS / WAVE;
    int below = 0;
    for (long i = tid; i < S; i += SORT_THREADS) below += idx[i] < e;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) below += __shfl_xor(below, off);
    if (lane == 0) part[wid] = below;
    __syncthreads();
    int base = 0;
#pragma unroll
    for (int w = 0; w < NW; ++w) base += part[w];
    if (tid == 0) {
        offs[e] = base;
        if (e == E - 1) offs[E] = (int)S;
    }
    for (long c0 = 0; c0 < S; c0 += SORT_THREADS * SORT_PER) {
        const long i0 = c0 + (long)tid * SORT_PER;
        bool mine[SORT_PER];
        int n = 0;
#pragma unroll
        for (int j = 0; j < SORT_PER; ++j) {
            mine[j] = i0 + j < S && idx[i0 + j] == e;
            n += mine[j];
        }
        int scan = n;               // inclusive over the wave
#pragma unroll
        for (int off = 1; off < WAVE; off <<= 1) {
            const int y = __shfl_up(scan, off);
            if (lane >= off) scan += y;
        }
        __syncthreads();            // part may still be read
        if (lane == WAVE - 1) part[wid] = scan;
        __syncthreads();
        int row = base + scan - n, total = 0;
#pragma unroll
        for (int w = 0; w < NW; ++w) {
            if (w < wid) row += part[w];
            total += part[w];
        }
#pragma unroll
        for (int j = 0; j < SORT_PER; ++j)
            if (mine[j]) {
                pos[i0 + j] = row;
                tok[row] = (int)((i0 + j) / top_k);
                ++row;
            }
        base += total;
    }
}

// -------------------------------------------------- weighted expert sum
// out[t] = sum_j wt[t, j] * y[pos[t, j]], fp32 sums in j order.
template <typename T, int VEC>
__global__ void __launch_bounds__(MO_THREADS)
moe_combine_kernel(const T* __restrict__ y, const int* __restrict__ pos,
                   const float* __restrict__ wt, T* __restrict__ out, int W,
                   int top_k) {
    const int c = (blockIdx.y * MO_THREADS + threadIdx.x) * VEC;
    if (c >= W) return;             // VEC = 4 only when 4 divides W
    const long t = blockIdx.x;
    float a[VEC];
#pragma unroll
    for (int v = 0; v < VEC; ++v) a[v] = 0.f;
    for (int j = 0; j < top_k; ++j) {
        const float w = wt[t * top_k + j];
        float x[VEC];
        ldn<T, VEC>(y + (long)pos[t * top_k + j] * W + c, x);
#pragma unroll
        for (int v = 0; v < VEC; ++v) a[v] += w * x[v];
    }
    stn<T, VEC>(out + t * (long)W + c, a);
}

// --------------------------------------------------- routed gated unit
// gu [T, E, 2I] (gate | up of every expert) -> out [T, E * I]:
// silu(gate) * up * weight, the token's routing weight for that expert;
// zeros, without reading gu, for experts the token did not choose.
template <typename T, int VEC>
__global__ void __launch_bounds__(MO_THREADS)
routed_silu_glu_kernel(const T* __restrict__ gu, const float* __restrict__ wt,
                       const int* __restrict__ idx, T* __restrict__ out,
                       int E, int I, int top_k) {
    const int c = (blockIdx.y * MO_THREADS + threadIdx.x) * VEC;
    if (c >= E * I) return;         // VEC = 4 only when 4 divides I
    const long t = blockIdx.x;
    const int e = c / I, i = c - e * I;
    float w = 0.f;
    bool chosen = false;
    for (int j = 0; j < top_k; ++j)
        if (idx[t * top_k + j] == e) {
            w = wt[t * top_k + j];
            chosen = true;
        }
    float y[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) y[j] = 0.f;
    if (chosen) {
        const T* row = gu + (t * E + e) * 2L * I + i;
        float g[VEC], u[VEC];
        ldn<T, VEC>(row, g);
        ldn<T, VEC>(row + I, u);
#pragma unroll
        for (int j = 0; j < VEC; ++j)
            y[j] = g[j] / (1.f + expf(-g[j])) * u[j] * w;
    }
    stn<T, VEC>(out + t * E * (long)I + c, y);
}

// --------------------------------------------- routed square of relu
// z, out [T, E*I + n]: relu(w z)^2 in the columns of an expert the token
// chose (w its routing weight, applied to what the expert reads), zeros,
// without reading z, for the others; relu(z)^2 in the last n columns.
template <typename T, int VEC>
__global__ void __launch_bounds__(MO_THREADS)
routed_relu2_kernel(const T* __restrict__ z, const float* __restrict__ wt,
                    const int* __restrict__ idx, T* __restrict__ out, int E,
                    int I, int N, int top_k) {
    const int c = (blockIdx.y * MO_THREADS + threadIdx.x) * VEC;
    if (c >= N) return;             // VEC = 4 only when 4 divides I and N
    const long t = blockIdx.x;
    const int e = c / I;
    float w = e >= E ? 1.f : 0.f;
    bool used = e >= E;
    if (!used)
        for (int j = 0; j < top_k; ++j)
            if (idx[t * top_k + j] == e) {
                w = wt[t * top_k + j];
                used = true;
            }
    float y[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) y[j] = 0.f;
    if (used) {
        ldn<T, VEC>(z + t * (long)N + c, y);
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            const float r = fmaxf(w * y[j], 0.f);
            y[j] = r * r;
        }
    }
    stn<T, VEC>(out + t * (long)N + c, y);
}

}  // namespace

// ---------------------------------------------------------------- launchers
// c: 0 = bf16, 1 = fp32. vec: row lengths and base addresses allow
// 4-element accesses.

extern "C" void launch_moe_sort(const int* idx, long S, int top_k, int E,
                                int* pos, int* tok, int* offs,
                                hipStream_t s) {
    if (E == 0) return;
    moe_sort_kernel<<<E, SORT_THREADS, 0, s>>>(idx, S, top_k, E, pos, tok,
                                               offs);
}

extern "C" void launch_moe_combine(const void* y, const int* pos,
                                   const float* wt, void* out, long T, int W,
                                   int top_k, int c, int vec, hipStream_t s) {
    if (T == 0) return;
    const int per = MO_THREADS * (vec ? 4 : 1);
    const dim3 grid((unsigned)T, (W + per - 1) / per);
#define MC_LAUNCH(TT, V)                                                      \
    moe_combine_kernel<TT, V><<<grid, MO_THREADS, 0, s>>>(                    \
        (const TT*)y, pos, wt, (TT*)out, W, top_k)
    if (c && vec) MC_LAUNCH(float, 4);
    else if (c) MC_LAUNCH(float, 1);
    else if (vec) MC_LAUNCH(unsigned short, 4);
    else MC_LAUNCH(unsigned short, 1);
#undef MC_LAUNCH
}

extern "C" void launch_routed_silu_glu(const void* gu, const float* wt,
                                       const int* idx, void* out, long T,
                                       int E, int I, int top_k, int c,
                                       int vec, hipStream_t s) {
    if (T == 0) return;
    const int per = MO_THREADS * (vec ? 4 : 1);
    const dim3 grid((unsigned)T, (E * I + per - 1) / per);
#define RG_LAUNCH(TT, V)                                                      \
    routed_silu_glu_kernel<TT, V><<<grid, MO_THREADS, 0, s>>>(                \
        (const TT*)gu, wt, idx, (TT*)out, E, I, top_k)
    if (c && vec) RG_LAUNCH(float, 4);
    else if (c) RG_LAUNCH(float, 1);
    else if (vec) RG_LAUNCH(unsigned short, 4);
    else RG_LAUNCH(unsigned short, 1);
#undef RG_LAUNCH
}

extern "C" void launch_routed_relu2(const void* z, const float* wt,
                                    const int* idx, void* out, long T, int E,
                                    int I, int N, int top_k, int c, int vec,
                                    hipStream_t s) {
    if (T == 0) return;
    const int per = MO_THREADS * (vec ? 4 : 1);
    const dim3 grid((unsigned)T, (N + per - 1) / per);
#define RR_LAUNCH(TT, V)                                                      \
    routed_relu2_kernel<TT, V><<<grid, MO_THREADS, 0, s>>>(                   \
        (const TT*)z, wt, idx, (TT*)out, E, I, N, top_k)
    if (c && vec) RR_LAUNCH(float, 4);
    else if (c) RR_LAUNCH(float, 1);
    else if (vec) RR_LAUNCH(unsigned short, 4);
    else RR_LAUNCH(unsigned short, 1);
#undef RR_LAUNCH
}
