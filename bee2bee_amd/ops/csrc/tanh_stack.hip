// Memory-bound kernels of the dynamic-tanh layer stacks
// (x += n_b(f(n_a(x))), n(x) = tanh(alpha x) * w + b): the norm pair around
// the fp32 residual update, and query/key norms over the whole projection
// with the key/value page store.
//
// Every kernel is instantiated for bf16 (ushort bits) and fp32 activations;
// residual, norm weights and statistics are fp32 in both.
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

constexpr int TS_THREADS = 256;

// ---------------------------------------------------- dynamic-tanh norms
// resid += tanh(pa * y) * pw + pb   (y given)
// out    = tanh(na * resid) * nw + nb   (out given)
// Element-wise: workgroup = TS_THREADS * VEC columns of one row, every
// operand crosses HBM once.
template <typename YT, typename OT, int VEC>
__global__ void __launch_bounds__(TS_THREADS)
add_tanh_norm_kernel(float* __restrict__ resid, const YT* __restrict__ y,
                     float pa, const float* __restrict__ pw,
                     const float* __restrict__ pb, float na,
                     const float* __restrict__ nw,
                     const float* __restrict__ nb, OT* __restrict__ out,
                     int W) {
    const int c = (blockIdx.y * TS_THREADS + threadIdx.x) * VEC;
    if (c >= W) return;             // VEC = 4 only when 4 divides W
    const long at = (long)blockIdx.x * W + c;
    float x[VEC];
    ldn<float, VEC>(resid + at, x);
    if (y) {
        float v[VEC], w[VEC], b[VEC];
        ldn<YT, VEC>(y + at, v);
        ldn<float, VEC>(pw + c, w);
        ldn<float, VEC>(pb + c, b);
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[j] += tanhf(pa * v[j]) * w[j] + b[j];
        stn<float, VEC>(resid + at, x);
    }
    if (!out) return;
    float w[VEC], b[VEC];
    ldn<float, VEC>(nw + c, w);
    ldn<float, VEC>(nb + c, b);
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[j] = tanhf(na * x[j]) * w[j] + b[j];
    stn<OT, VEC>(out + at, x);
}

// ----------------------- query/key norm over the projection, page store
// Workgroup per token. Query: all H * D numbers divided by their common root
// mean square, times wq and q_mult, in place. Key: the same over G * D with
// wk, to k_cache [n_blocks, G, bs, D]. Value: to v_cache
// [n_blocks, G, bs, Dv], each head divided by its own root mean square
// first when v_unit. VEC = 4 needs D, Dv and all rows 4-aligned.
DEV_INLINE float ts_block_sum(float v, float* red) {
    v = wave_sum(v);
    const int wid = threadIdx.x / WAVE;
    __syncthreads();                // red may still be read
    if (threadIdx.x % WAVE == 0) red[wid] = v;
    __syncthreads();
    float total = 0.f;
#pragma unroll
    for (int i = 0; i < TS_THREADS / WAVE; ++i) total += red[i];
    return total;
}

template <typename T, int VEC>
__global__ void __launch_bounds__(TS_THREADS)
proj_norm_store_kernel(T* __restrict__ q, long q_tok, int H,
                       const T* __restrict__ k, long k_tok,
                       const T* __restrict__ v, long v_tok, int G, int D,
                       int Dv, const float* __restrict__ wq,
                       const float* __restrict__ wk, int v_unit, float eps,
                       float q_mult, T* __restrict__ k_cache,
                       T* __restrict__ v_cache, int bs,
                       const int* __restrict__ slot_mapping) {
    __shared__ float red[TS_THREADS / WAVE];
    const long t = blockIdx.x;
    const int slot = slot_mapping[t];
    const long blk = slot / bs, off = slot % bs;
    const int nq = H * D, nk = G * D;
    T* qr = q + t * q_tok;
    const T* kr = k + t * k_tok;
    float sq = 0.f, sk = 0.f;
    for (int i = threadIdx.x * VEC; i < nq; i += TS_THREADS * VEC) {
        float x[VEC];
        ldn<T, VEC>(qr + i, x);
#pragma unroll
        for (int j = 0; j < VEC; ++j) sq += x[j] * x[j];
    }
    for (int i = threadIdx.x * VEC; i < nk; i += TS_THREADS * VEC) {
        float x[VEC];
        ldn<T, VEC>(kr + i, x);
#pragma unroll
        for (int j = 0; j < VEC; ++j) sk += x[j] * x[j];
    }
    const float rq =
        q_mult / sqrtf(ts_block_sum(sq, red) / (float)nq + eps);
    const float rk = 1.f / sqrtf(ts_block_sum(sk, red) / (float)nk + eps);
    // every thread rewrites exactly the query numbers it has read
    for (int i = threadIdx.x * VEC; i < nq; i += TS_THREADS * VEC) {
        float x[VEC], w[VEC];
        ldn<T, VEC>(qr + i, x);
        ldn<float, VEC>(wq + i, w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[j] *= rq * w[j];
        stn<T, VEC>(qr + i, x);
    }
    for (int i = threadIdx.x * VEC; i < nk; i += TS_THREADS * VEC) {
        float x[VEC], w[VEC];
        ldn<T, VEC>(kr + i, x);
        ldn<float, VEC>(wk + i, w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[j] *= rk * w[j];
        const int g = i / D, d = i - g * D;
        stn<T, VEC>(k_cache + ((blk * G + g) * bs + off) * D + d, x);
    }
    const int wid = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
    for (int g = wid; g < G; g += TS_THREADS / WAVE) {
        const T* vr = v + t * v_tok + (long)g * Dv;
        T* dst = v_cache + ((blk * G + g) * bs + off) * Dv;
        float ss = 0.f;
        if (v_unit)
            for (int i = lane * VEC; i < Dv; i += WAVE * VEC) {
                float x[VEC];
                ldn<T, VEC>(vr + i, x);
#pragma unroll
                for (int j = 0; j < VEC; ++j) ss += x[j] * x[j];
            }
        const float r =
            v_unit ? 1.f / sqrtf(wave_sum(ss) / (float)Dv + eps) : 1.f;
        for (int i = lane * VEC; i < Dv; i += WAVE * VEC) {
            float x[VEC];
            ldn<T, VEC>(vr + i, x);
#pragma unroll
            for (int j = 0; j < VEC; ++j) x[j] *= r;
            stn<T, VEC>(dst + i, x);
        }
    }
}

}  // namespace

// ---------------------------------------------------------------- launchers
// yc / oc / c: 0 = bf16, 1 = fp32. vec: row lengths, strides and base
// addresses allow 4-element accesses.

extern "C" void launch_add_tanh_norm(float* resid, const void* y, float pa,
                                     const float* pw, const float* pb,
                                     float na, const float* nw,
                                     const float* nb, void* out, long T,
                                     int W, int yc, int oc, int vec,
                                     hipStream_t s) {
    if (T == 0 || W == 0) return;
    const int per = TS_THREADS * (vec ? 4 : 1);
    const dim3 grid((unsigned)T, (W + per - 1) / per);
#define TN_LAUNCH(YT, OT, V)                                                  \
    add_tanh_norm_kernel<YT, OT, V><<<grid, TS_THREADS, 0, s>>>(              \
        resid, (const YT*)y, pa, pw, pb, na, nw, nb, (OT*)out, W)
#define TN_PICK(YT, OT)                                                       \
    do {                                                                      \
        if (vec) TN_LAUNCH(YT, OT, 4);                                        \
        else TN_LAUNCH(YT, OT, 1);                                            \
    } while (0)
    if (yc && oc) TN_PICK(float, float);
    else if (yc) TN_PICK(float, unsigned short);
    else if (oc) TN_PICK(unsigned short, float);
    else TN_PICK(unsigned short, unsigned short);
#undef TN_PICK
#undef TN_LAUNCH
}

extern "C" void launch_proj_norm_store(
    void* q, long q_tok, int H, const void* k, long k_tok, const void* v,
    long v_tok, int G, int D, int Dv, const float* wq, const float* wk,
    int v_unit, float eps, float q_mult, void* k_cache, void* v_cache, int bs,
    const int* slot_mapping, long T, int c, int vec, hipStream_t s) {
    if (T == 0) return;
#define PN_LAUNCH(TT, V)                                                      \
    proj_norm_store_kernel<TT, V><<<(unsigned)T, TS_THREADS, 0, s>>>(         \
        (TT*)q, q_tok, H, (const TT*)k, k_tok, (const TT*)v, v_tok, G, D, Dv, \
        wq, wk, v_unit, eps, q_mult, (TT*)k_cache, (TT*)v_cache, bs,          \
        slot_mapping)
    if (c && vec) PN_LAUNCH(float, 4);
    else if (c) PN_LAUNCH(float, 1);
    else if (vec) PN_LAUNCH(unsigned short, 4);
    else PN_LAUNCH(unsigned short, 1);
#undef PN_LAUNCH
}
