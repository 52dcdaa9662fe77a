// Memory-bound kernels of the scaled parallel-form layer stacks
//   x += s1 * mixer(n1(x)) + s2 * ffn(n2(x));  x += unit(P (gelu(G x) * e)) * w
// with vectors s1, s2 and two weighted norms n1, n2 of the same x: the token
// embedding with its sinusoidal position vector, the scaled residual update,
// the side norm with its add fused with both norms of the next layer, the
// side gate, and the gated grouped norm of the state-space mixer.
//
// Activations are bf16 (ushort bits) or fp32; the residual stream, norm
// statistics and angles are fp32 (angles reduced in fp64) in both.
#include "common.h"

namespace {

template <typename T, int VEC> DEV_INLINE void ldv(const T* p, float* o);
template <> DEV_INLINE void ldv<float, 1>(const float* p, float* o) { o[0] = *p; }
template <> DEV_INLINE void ldv<unsigned short, 1>(const unsigned short* p, float* o) {
    o[0] = bf2f(*p);
}
template <> DEV_INLINE void ldv<float, 4>(const float* p, float* o) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(p);
    o[0] = v[0]; o[1] = v[1]; o[2] = v[2]; o[3] = v[3];
}
template <> DEV_INLINE void ldv<unsigned short, 4>(const unsigned short* p, float* o) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    o[0] = bf2f((unsigned short)(w.x & 0xffffu));
    o[1] = bf2f((unsigned short)(w.x >> 16));
    o[2] = bf2f((unsigned short)(w.y & 0xffffu));
    o[3] = bf2f((unsigned short)(w.y >> 16));
}
template <typename T, int VEC> DEV_INLINE void stv(T* p, const float* o);
template <> DEV_INLINE void stv<float, 1>(float* p, const float* o) { *p = o[0]; }
template <> DEV_INLINE void stv<unsigned short, 1>(unsigned short* p, const float* o) {
    *p = f2bf(o[0]);
}
template <> DEV_INLINE void stv<float, 4>(float* p, const float* o) {
    *reinterpret_cast<f32x4*>(p) = f32x4{o[0], o[1], o[2], o[3]};
}
template <> DEV_INLINE void stv<unsigned short, 4>(unsigned short* p, const float* o) {
    uint2 w;
    w.x = (unsigned int)f2bf(o[0]) | ((unsigned int)f2bf(o[1]) << 16);
    w.y = (unsigned int)f2bf(o[2]) | ((unsigned int)f2bf(o[3]) << 16);
    *reinterpret_cast<uint2*>(p) = w;
}

constexpr int SC_THREADS = 256;

// sum over the workgroup; red: LDS [SC_THREADS / WAVE]; every thread gets it
DEV_INLINE float block_sum(float v, float* red) {
    const int wid = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
    v = wave_sum(v);
    __syncthreads();            // earlier readers of red are done
    if (lane == 0) red[wid] = v;
    __syncthreads();
    float t = 0.f;
    for (int w = 0; w < (int)(blockDim.x / WAVE); ++w) t += red[w];
    return t;
}

// ------------------------------------------------- embedding + positions
// x[t] = table[id] * scale + (sin, cos) pairs: columns 2i and 2i+1 take sin
// and cos of p * freq[i]. The angle is formed and reduced to turns in fp64,
// then evaluated once in fp32. A thread owns column pairs. An id outside the
// table gives NaN instead of an access.
template <typename T>
__global__ void __launch_bounds__(SC_THREADS)
embed_sinusoid_kernel(const long* __restrict__ ids,
                      const T* __restrict__ table, float scale,
                      const int* __restrict__ positions,
                      const double* __restrict__ freq, float* __restrict__ x,
                      int W, long V) {
    const long t = blockIdx.x;
    const bool known = ids[t] >= 0 && ids[t] < V;
    const T* row = table + (known ? ids[t] : 0) * (long)W;
    if (!known) scale = NAN;
    const double p = (double)positions[t] * 0.15915494309189533577;  // 1/2pi
    float* xr = x + t * (long)W;
    for (int i = threadIdx.x; 2 * i < W; i += blockDim.x) {
        double turns = p * freq[i];
        turns -= rint(turns);
        float s, c;
        sincospif(2.f * (float)turns, &s, &c);
        float e[1];
        ldv<T, 1>(row + 2 * i, e);
        xr[2 * i] = e[0] * scale + s;
        if (2 * i + 1 < W) {
            ldv<T, 1>(row + 2 * i + 1, e);
            xr[2 * i + 1] = e[0] * scale + c;
        }
    }
}

// ------------------------------------------------ scaled residual update
// resid += s1 * y1 [+ s2 * (y2 [+ y3])]; cast (optional) <- resid in the
// activation type. (row, column part) grid, one element group a thread.
template <typename T, int VEC>
__global__ void __launch_bounds__(SC_THREADS)
scaled_add_kernel(float* __restrict__ resid, const T* __restrict__ y1,
                  const float* __restrict__ s1, const T* __restrict__ y2,
                  const float* __restrict__ s2, const T* __restrict__ y3,
                  T* __restrict__ cast, int W) {
    const int c = (blockIdx.y * SC_THREADS + threadIdx.x) * VEC;
    if (c >= W) return;             // VEC = 4 only when 4 divides W
    const long at = blockIdx.x * (long)W + c;
    float v[VEC], a[VEC], s[VEC];
    ldv<float, VEC>(resid + at, v);
    ldv<T, VEC>(y1 + at, a);
    ldv<float, VEC>(s1 + c, s);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] += a[j] * s[j];
    if (y2) {
        ldv<T, VEC>(y2 + at, a);
        ldv<float, VEC>(s2 + c, s);
        if (y3) {
            float b[VEC];
            ldv<T, VEC>(y3 + at, b);
#pragma unroll
            for (int j = 0; j < VEC; ++j) a[j] += b[j];
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += a[j] * s[j];
    }
    stv<float, VEC>(resid + at, v);
    if (cast) stv<T, VEC>(cast + at, v);
}

// ------------------------------------- post-normed add + two weighted norms
// resid += unit(y) * wp (y given); oa = unit(resid) * wa, ob = unit(resid) *
// wb (each when given). Workgroup per row; the rows are held in LDS between
// the passes, so every operand crosses HBM once.
template <typename T, int VEC>
__global__ void __launch_bounds__(SC_THREADS)
add_norm_pair_kernel(float* __restrict__ resid, const T* __restrict__ y,
                     const float* __restrict__ wp,
                     const float* __restrict__ wa,
                     const float* __restrict__ wb, T* __restrict__ oa,
                     T* __restrict__ ob, int W, float eps) {
    extern __shared__ __attribute__((aligned(16))) float np_row[];
    __shared__ float red[SC_THREADS / WAVE];
    const long t = blockIdx.x;
    float* rr = resid + t * (long)W;
    float r = 0.f;
    if (y) {
        const T* yr = y + t * (long)W;
        float ss = 0.f;
        // each thread reads back only what it wrote itself
        for (int i = threadIdx.x * VEC; i < W; i += blockDim.x * VEC) {
            float a[VEC];
            ldv<T, VEC>(yr + i, a);
#pragma unroll
            for (int j = 0; j < VEC; ++j) {
                np_row[i + j] = a[j];
                ss += a[j] * a[j];
            }
        }
        r = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
    }
    float ss = 0.f;
    for (int i = threadIdx.x * VEC; i < W; i += blockDim.x * VEC) {
        float v[VEC];
        ldv<float, VEC>(rr + i, v);
        if (y) {
            float w[VEC];
            ldv<float, VEC>(wp + i, w);
#pragma unroll
            for (int j = 0; j < VEC; ++j) v[j] += np_row[i + j] * r * w[j];
            stv<float, VEC>(rr + i, v);
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            np_row[i + j] = v[j];
            ss += v[j] * v[j];
        }
    }
    if (!oa && !ob) return;
    r = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
    for (int i = threadIdx.x * VEC; i < W; i += blockDim.x * VEC) {
        float v[VEC], w[VEC];
        if (oa) {
            ldv<float, VEC>(wa + i, w);
#pragma unroll
            for (int j = 0; j < VEC; ++j) v[j] = np_row[i + j] * r * w[j];
            stv<T, VEC>(oa + t * (long)W + i, v);
        }
        if (ob) {
            ldv<float, VEC>(wb + i, w);
#pragma unroll
            for (int j = 0; j < VEC; ++j) v[j] = np_row[i + j] * r * w[j];
            stv<T, VEC>(ob + t * (long)W + i, v);
        }
    }
}

// ------------------------------------------------------------- side gate
// out[t, c] = gelu_tanh(g[t, c]) * table[ids[t], offset + c]
template <typename T>
__global__ void __launch_bounds__(SC_THREADS)
side_gate_kernel(const T* __restrict__ g, const T* __restrict__ table,
                 long row, long offset, const long* __restrict__ ids,
                 T* __restrict__ out, long n, int d, long V) {
    const long i = (long)blockIdx.x * SC_THREADS + threadIdx.x;
    if (i >= n) return;
    const long t = i / d;
    const int c = (int)(i - t * d);
    float z[1], e[1];
    ldv<T, 1>(g + i, z);
    const bool known = ids[t] >= 0 && ids[t] < V;
    ldv<T, 1>(table + (known ? ids[t] : 0) * row + offset + c, e);
    const float u = known ? z[0] : NAN;
    const float k = 0.79788456080286536f * (u + 0.044715f * u * u * u);
    float o[1] = {0.5f * u * (1.f + tanhf(k)) * e[0]};
    stv<T, 1>(out + i, o);
}

// ---------------------------------------------------- gated grouped norm
// v = y * silu(z); out = v / sqrt(mean over the group(v^2) + eps) * w *
// out_scale. Workgroup per (token, group of n columns), the group's v in LDS.
template <typename T, int VEC>
__global__ void __launch_bounds__(SC_THREADS)
gated_group_norm_kernel(const float* __restrict__ y, long ys,
                        const T* __restrict__ z, long zs,
                        const float* __restrict__ w, T* __restrict__ out,
                        long os, int n, float eps, float out_scale) {
    extern __shared__ __attribute__((aligned(16))) float gg_row[];
    __shared__ float red[SC_THREADS / WAVE];
    const long t = blockIdx.x;
    const int c0 = blockIdx.y * n;
    float ss = 0.f;
    for (int i = threadIdx.x * VEC; i < n; i += blockDim.x * VEC) {
        float a[VEC], g[VEC];
        ldv<float, VEC>(y + t * ys + c0 + i, a);
        ldv<T, VEC>(z + t * zs + c0 + i, g);
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            const float v = a[j] * g[j] / (1.f + expf(-g[j]));
            gg_row[i + j] = v;
            ss += v * v;
        }
    }
    const float r = out_scale / sqrtf(block_sum(ss, red) / (float)n + eps);
    for (int i = threadIdx.x * VEC; i < n; i += blockDim.x * VEC) {
        float v[VEC], wv[VEC];
        ldv<float, VEC>(w + c0 + i, wv);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = gg_row[i + j] * r * wv[j];
        stv<T, VEC>(out + t * os + c0 + i, v);
    }
}

inline int row_threads(int n) {
    int th = WAVE;
    while (th < n && th < SC_THREADS) th <<= 1;
    return th;
}

}  // namespace

// ---------------------------------------------------------------- launchers
// c: 0 = bf16, 1 = fp32. vec: row lengths, strides and base addresses allow
// 4-element accesses.

extern "C" void launch_embed_sinusoid(const long* ids, const void* table,
                                      float scale, const int* positions,
                                      const double* freq, float* x, long T,
                                      int W, long V, int c, hipStream_t s) {
    if (T == 0) return;
    const int th = row_threads((W + 1) / 2);
    if (c)
        embed_sinusoid_kernel<float><<<T, th, 0, s>>>(
            ids, (const float*)table, scale, positions, freq, x, W, V);
    else
        embed_sinusoid_kernel<unsigned short><<<T, th, 0, s>>>(
            ids, (const unsigned short*)table, scale, positions, freq, x, W,
            V);
}

extern "C" void launch_scaled_add(float* resid, const void* y1,
                                  const float* s1, const void* y2,
                                  const float* s2, const void* y3, void* cast,
                                  long T, int W, int c, int vec,
                                  hipStream_t s) {
    if (T == 0) return;
    const int per = SC_THREADS * (vec ? 4 : 1);
    const dim3 grid((unsigned)T, (W + per - 1) / per);
#define SA_LAUNCH(TT, V)                                                      \
    scaled_add_kernel<TT, V><<<grid, SC_THREADS, 0, s>>>(                     \
        resid, (const TT*)y1, s1, (const TT*)y2, s2, (const TT*)y3,           \
        (TT*)cast, W)
    if (c && vec) SA_LAUNCH(float, 4);
    else if (c) SA_LAUNCH(float, 1);
    else if (vec) SA_LAUNCH(unsigned short, 4);
    else SA_LAUNCH(unsigned short, 1);
#undef SA_LAUNCH
}

extern "C" void launch_add_norm_pair(float* resid, const void* y,
                                     const float* wp, const float* wa,
                                     const float* wb, void* oa, void* ob,
                                     long T, int W, float eps, int c, int vec,
                                     hipStream_t s) {
    if (T == 0) return;
    const size_t sh = (size_t)W * sizeof(float);
    const int th = row_threads(vec ? W / 4 : W);
#define NP_LAUNCH(TT, V)                                                      \
    add_norm_pair_kernel<TT, V><<<T, th, sh, s>>>(                            \
        resid, (const TT*)y, wp, wa, wb, (TT*)oa, (TT*)ob, W, eps)
    if (c && vec) NP_LAUNCH(float, 4);
    else if (c) NP_LAUNCH(float, 1);
    else if (vec) NP_LAUNCH(unsigned short, 4);
    else NP_LAUNCH(unsigned short, 1);
#undef NP_LAUNCH
}

extern "C" void launch_side_gate(const void* g, const void* table, long row,
                                 long offset, const long* ids, void* out,
                                 long T, int d, long V, int c,
                                 hipStream_t s) {
    const long n = T * d;
    if (n == 0) return;
    const unsigned blocks = (unsigned)((n + SC_THREADS - 1) / SC_THREADS);
    if (c)
        side_gate_kernel<float><<<blocks, SC_THREADS, 0, s>>>(
            (const float*)g, (const float*)table, row, offset, ids,
            (float*)out, n, d, V);
    else
        side_gate_kernel<unsigned short><<<blocks, SC_THREADS, 0, s>>>(
            (const unsigned short*)g, (const unsigned short*)table, row,
            offset, ids, (unsigned short*)out, n, d, V);
}

extern "C" void launch_gated_group_norm(const float* y, long ys,
                                        const void* z, long zs,
                                        const float* w, void* out, long os,
                                        long T, int groups, int n, float eps,
                                        float out_scale, int c, int vec,
                                        hipStream_t s) {
    if (T == 0) return;
    const dim3 grid((unsigned)T, groups);
    const size_t sh = (size_t)n * sizeof(float);
    const int th = row_threads(vec ? n / 4 : n);
#define GG_LAUNCH(TT, V)                                                      \
    gated_group_norm_kernel<TT, V><<<grid, th, sh, s>>>(                      \
        y, ys, (const TT*)z, zs, w, (TT*)out, os, n, eps, out_scale)
    if (c && vec) GG_LAUNCH(float, 4);
    else if (c) GG_LAUNCH(float, 1);
    else if (vec) GG_LAUNCH(unsigned short, 4);
    else GG_LAUNCH(unsigned short, 1);
#undef GG_LAUNCH
}
