// State-space recurrence with one decay per head and token:
//   S_t = exp(-rate_h d_t) S_(t-1) + d_t B_t x_t^T      (S is N x V, fp32)
//   y_t = S_t^T C_t + skip_h x_t,   d_t = softplus(dt_t + dt_bias_h)
// B and C are shared by the H/G heads of a group. x | B | C are columns of
// one row per token (bf16 or fp32, after their convolution), dt is a column
// slice, y is fp32 [Tn, H * V]. A chunk that starts at position 0 starts from
// S = 0 without reading its slot.
//
// Two forms:
//  * ssd_serial: decode rows and short portions. A workgroup keeps a 64-column
//    slice of one (sequence, head) state in registers and walks the tokens.
//  * chunk-parallel, for long portions, in pieces of 64 tokens:
//    ssd_states   what a piece adds to the state, sum_t exp(A_L - A_t) d_t
//                 B_t x_t^T, A the running log decay inside the piece;
//    ssd_carry    walks the pieces of each (sequence, head) in order, turning
//                 those into the state at every piece's start;
//    ssd_outputs  y = (C B^T . exp(A_t - A_s) d_s, s <= t) X + exp(A_t) C S.
//    All products run on v_mfma_f32_16x16x4_f32: fp32 operands and sums, for
//    bf16 and fp32 activations alike. Running log decays are kept in fp64, so
//    that their differences hold fp32 precision however far they run.
//
// Fragment maps of v_mfma_f32_16x16x4_f32: A: lane -> row l & 15, k = l >> 4;
// B: lane -> column l & 15, k = l >> 4; C: column l & 15, rows (l >> 4) * 4 +
// r. Which four k values a step takes is free as long as A and B agree: where
// a lane reads four neighbours at once, step e of four takes k = 4 (l >> 4) + e.
#include "common.h"

namespace {

template <typename T> DEV_INLINE float ldf(const T* p);
template <> DEV_INLINE float ldf<float>(const float* p) { return *p; }
template <> DEV_INLINE float ldf<unsigned short>(const unsigned short* p) {
    return bf2f(*p);
}
template <typename T> DEV_INLINE void ld4(const T* p, float* o);
template <> DEV_INLINE void ld4<float>(const float* p, float* o) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(p);
    o[0] = v[0]; o[1] = v[1]; o[2] = v[2]; o[3] = v[3];
}
template <> DEV_INLINE void ld4<unsigned short>(const unsigned short* p,
                                                float* o) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    o[0] = bf2f((unsigned short)(w.x & 0xffffu));
    o[1] = bf2f((unsigned short)(w.x >> 16));
    o[2] = bf2f((unsigned short)(w.y & 0xffffu));
    o[3] = bf2f((unsigned short)(w.y >> 16));
}
// four neighbours at column c of a row of n; zeros past its end
template <typename T, bool VEC>
DEV_INLINE void ld4_row(const T* row, int c, int n, float* o) {
    if (VEC) {                      // n is a multiple of 4: all or none
        if (c < n) {
            ld4<T>(row + c, o);
        } else {
            o[0] = o[1] = o[2] = o[3] = 0.f;
        }
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = c + e < n ? ldf(row + c + e) : 0.f;
    }
}

DEV_INLINE float softplus_f(float z) {
    return z > 20.f ? z : log1pf(expf(z));
}

struct SsdArgs {
    const void* xbc;        // [Tn, xs]: x (H*V) | B (G*N) | C (G*N)
    long xs;
    const void* dt;         // [Tn, H], row stride dts
    long dts;
    const float* dt_bias;   // [H]
    const float* rate;      // [H]
    const float* skip;      // [H]
    float* state;           // [slots, H, N, V]
    const int* state_slots;
    const int* cu;
    const int* positions;
    float* y;               // [Tn, H * V]
    float* ws;              // chunk form: [pieces, H, N, V]
    float* fade;            // chunk form: [pieces, H]
    int B, H, G, N, V;
};

// ---------------------------------------------------------------- serial
constexpr int SS_THREADS = 256;
constexpr int SS_COLS = 64;      // state columns per workgroup
constexpr int SS_MAXN = 512;

// Thread (row group rg, column unit cl): columns cl*VW.. of the slice and
// rows rg, rg + RG, ...; RG = 256 / lpr row groups, lpr (a power of two)
// lanes span the slice's columns.
template <typename T, int VW, int RPT>
__global__ void __launch_bounds__(SS_THREADS)
ssd_serial_kernel(SsdArgs a, int lpr) {
    __shared__ float bs[SS_MAXN], cs[SS_MAXN];
    __shared__ float part[SS_THREADS / WAVE][SS_COLS];
    const int b = blockIdx.x, h = blockIdx.y;
    const int lo = a.cu[b], hi = a.cu[b + 1];
    if (hi <= lo) return;
    const int tid = threadIdx.x, lane = tid % WAVE, wid = tid / WAVE;
    const int RG = SS_THREADS / lpr;
    const int rg = tid / lpr, cl = tid % lpr;
    const int c0 = blockIdx.z * SS_COLS + cl * VW;
    const bool live = c0 < a.V;         // VW = 4 only when 4 divides V
    const int N = a.N, V = a.V, g = h / (a.H / a.G);
    const T* X = (const T*)a.xbc + (long)h * V;
    const T* Bp = (const T*)a.xbc + (long)a.H * V + (long)g * N;
    const T* Cp = Bp + (long)a.G * N;
    float* st = a.state + ((long)a.state_slots[b] * a.H + h) * N * V + c0;
    const bool fresh = a.positions[lo] == 0;
    const float rate = a.rate[h], bias = a.dt_bias[h], skip = a.skip[h];
    float s[RPT][VW];
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
        const int n = rg + j * RG;
#pragma unroll
        for (int v = 0; v < VW; ++v) s[j][v] = 0.f;
        if (!fresh && live && n < N) {
            if (VW == 4) {
                ld4<float>(st + (long)n * V, s[j]);
            } else {
                s[j][0] = st[(long)n * V];
            }
        }
    }
    for (int t = lo; t < hi; ++t) {
        const long at = (long)t * a.xs;
        for (int n = tid; n < N; n += SS_THREADS) {
            bs[n] = ldf(Bp + at + n);
            cs[n] = ldf(Cp + at + n);
        }
        const float d =
            softplus_f(ldf((const T*)a.dt + (long)t * a.dts + h) + bias);
        const float fade = expf(-rate * d);
        float x[VW], acc[VW];
#pragma unroll
        for (int v = 0; v < VW; ++v) x[v] = acc[v] = 0.f;
        if (live) {
            if (VW == 4) ld4<T>(X + at + c0, x);
            else x[0] = ldf(X + at + c0);
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < RPT; ++j) {
            const int n = rg + j * RG;
            if (n < N) {
                const float w = d * bs[n], c = cs[n];
#pragma unroll
                for (int v = 0; v < VW; ++v) {
                    s[j][v] = fade * s[j][v] + w * x[v];
                    acc[v] += s[j][v] * c;
                }
            }
        }
        // row groups of a wave, then the waves
        for (int off = lpr; off < WAVE; off <<= 1)
#pragma unroll
            for (int v = 0; v < VW; ++v) acc[v] += __shfl_xor(acc[v], off);
        if (lane < lpr)
#pragma unroll
            for (int v = 0; v < VW; ++v) part[wid][cl * VW + v] = acc[v];
        __syncthreads();
        if (rg == 0 && live) {
            float* yr = a.y + (long)t * a.H * V + (long)h * V + c0;
#pragma unroll
            for (int v = 0; v < VW; ++v) {
                float o = skip * x[v];
#pragma unroll
                for (int w = 0; w < SS_THREADS / WAVE; ++w)
                    o += part[w][cl * VW + v];
                yr[v] = o;
            }
        }
        // the next token's staging writes bs/cs, which every thread has
        // read by the barrier above; part is rewritten after the next one
    }
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
        const int n = rg + j * RG;
        if (live && n < N) {
            if (VW == 4)
                *reinterpret_cast<f32x4*>(st + (long)n * V) =
                    f32x4{s[j][0], s[j][1], s[j][2], s[j][3]};
            else
                st[(long)n * V] = s[j][0];
        }
    }
}

// ----------------------------------------------------------- chunk form
constexpr int SD_L = 64;         // tokens per piece = lanes of a wave
constexpr int SD_THREADS = 256;

// piece index -> (sequence, first row, rows); false when out of range
DEV_INLINE bool sd_piece(const int* __restrict__ cu, int B, int piece,
                         int* lo, int* n) {
    int first = 0;
    for (int b = 0; b < B; ++b) {
        const int len = cu[b + 1] - cu[b];
        const int k = (len + SD_L - 1) / SD_L;
        if (piece < first + k) {
            const int off = (piece - first) * SD_L;
            *lo = cu[b] + off;
            *n = min(SD_L, len - off);
            return true;
        }
        first += k;
    }
    return false;
}

// lane t of a wave: step size d and running log decay A of token lo + t
// (d = 0 and A unchanged past the piece's end)
template <typename T>
DEV_INLINE void sd_decay(const SsdArgs& a, int h, int lo, int n, int lane,
                         float* d, double* A) {
    *d = 0.f;
    if (lane < n)
        *d = softplus_f(ldf((const T*)a.dt + (long)(lo + lane) * a.dts + h) +
                        a.dt_bias[h]);
    double s = -(double)a.rate[h] * (double)*d;
#pragma unroll
    for (int off = 1; off < WAVE; off <<= 1) {
        const double u = __shfl_up(s, off);
        if (lane >= off) s += u;
    }
    *A = s;
}

constexpr int SD_NS = 128;       // state rows per workgroup of ssd_states
constexpr int SD_BS = SD_NS + 16;    // LDS row strides: the four k rows a
constexpr int SD_XS = SD_L + 16;     // fragment read touches sit 16 banks apart

// (piece, head, 128-row x 64-column block of the state); a wave owns every
// fourth 16-row tile against all the block's columns.
template <typename T, int VT, bool VEC>
__global__ void __launch_bounds__(SD_THREADS)
ssd_states_kernel(SsdArgs a) {
    __shared__ float bs[SD_L * SD_BS];
    __shared__ float xs[SD_L * SD_XS];
    __shared__ float wt[SD_L];
    int lo, n;
    if (!sd_piece(a.cu, a.B, blockIdx.x, &lo, &n)) return;
    const int h = blockIdx.y, g = h / (a.H / a.G);
    const int vblk = (a.V + SD_L - 1) / SD_L;
    const int n0 = blockIdx.z / vblk * SD_NS, v0 = blockIdx.z % vblk * SD_L;
    const int tid = threadIdx.x, lane = tid % WAVE;
    const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
    const int N = a.N, V = a.V;
    if (wid == 0) {
        float d;
        double A;
        sd_decay<T>(a, h, lo, n, lane, &d, &A);
        const double last = __shfl(A, WAVE - 1);
        wt[lane] = d * expf((float)(last - A));
        if (lane == 0 && blockIdx.z == 0)
            a.fade[(long)blockIdx.x * a.H + h] = expf((float)last);
    }
    __syncthreads();
    const T* X = (const T*)a.xbc + (long)h * V;
    const T* Bp = (const T*)a.xbc + (long)a.H * V + (long)g * N;
    // rows past the end repeat the last one; their weight is zero
    constexpr int BU = SD_NS / 4, XU = SD_L / 4;
    const int nlive = min(SD_NS, (N - n0 + 15) / 16 * 16);
    for (int i = tid; i < SD_L * BU; i += SD_THREADS) {
        const int t = i / BU, c = (i - t * BU) * 4;
        if (c >= nlive) continue;
        float v[4];
        ld4_row<T, VEC>(Bp + (long)(lo + min(t, n - 1)) * a.xs, n0 + c, N, v);
        const float w = wt[t];
#pragma unroll
        for (int e = 0; e < 4; ++e) bs[t * SD_BS + c + e] = w * v[e];
    }
    for (int i = tid; i < SD_L * XU; i += SD_THREADS) {
        const int t = i / XU, c = (i - t * XU) * 4;
        if (c >= VT * 16) continue;
        float v[4];
        ld4_row<T, VEC>(X + (long)(lo + min(t, n - 1)) * a.xs, v0 + c, V, v);
#pragma unroll
        for (int e = 0; e < 4; ++e) xs[t * SD_XS + c + e] = v[e];
    }
    __syncthreads();
    const int lg = lane >> 4, li = lane & 15;
    constexpr int NT = SD_NS / 16 / (SD_THREADS / WAVE);    // row tiles a wave
    f32x4 acc[NT][VT];
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int v = 0; v < VT; ++v) acc[i][v] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < SD_L; k += 4) {
        float xb[VT];
#pragma unroll
        for (int v = 0; v < VT; ++v)
            xb[v] = xs[(k + lg) * SD_XS + v * 16 + li];
#pragma unroll
        for (int i = 0; i < NT; ++i) {
            const int nt = i * (SD_THREADS / WAVE) + wid;
            if (nt * 16 >= nlive) continue;
            const float ba = bs[(k + lg) * SD_BS + nt * 16 + li];
#pragma unroll
            for (int v = 0; v < VT; ++v)
                acc[i][v] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    ba, xb[v], acc[i][v], 0, 0, 0);
        }
    }
    float* out = a.ws + ((long)blockIdx.x * a.H + h) * N * V;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
        const int nt = i * (SD_THREADS / WAVE) + wid;
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int c = v0 + v * 16 + li;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int row = n0 + nt * 16 + lg * 4 + r;
                if (row < N && c < V) out[(long)row * V + c] = acc[i][v][r];
            }
        }
    }
}

// per (sequence, head), VW state elements a thread: replace each piece's own
// contribution in ws by the state at the piece's start, leave the final
// state in the sequence's slot. Loads of SD_AHEAD pieces are in flight.
constexpr int SD_AHEAD = 4;
template <int VW>
__global__ void __launch_bounds__(SD_THREADS)
ssd_carry_kernel(SsdArgs a) {
    const int b = blockIdx.x, h = blockIdx.y;
    const long NV = (long)a.N * a.V;
    const long e = ((long)blockIdx.z * SD_THREADS + threadIdx.x) * VW;
    if (e >= NV) return;            // VW = 4 only when 4 divides N * V
    const int lo = a.cu[b], len = a.cu[b + 1] - lo;
    if (len <= 0) return;
    int first = 0;
    for (int i = 0; i < b; ++i)
        first += (a.cu[i + 1] - a.cu[i] + SD_L - 1) / SD_L;
    float* slot = a.state + ((long)a.state_slots[b] * a.H + h) * NV + e;
    float S[VW];
#pragma unroll
    for (int v = 0; v < VW; ++v) S[v] = 0.f;
    if (a.positions[lo] != 0) {
        if (VW == 4) ld4<float>(slot, S);
        else S[0] = *slot;
    }
    const int np = (len + SD_L - 1) / SD_L;
    const long step = (long)a.H * NV;
    float* w = a.ws + ((long)first * a.H + h) * NV + e;
    const float* fade = a.fade + (long)first * a.H + h;
    for (int p = 0; p < np; p += SD_AHEAD) {
        float add[SD_AHEAD][VW], f[SD_AHEAD];
#pragma unroll
        for (int u = 0; u < SD_AHEAD; ++u) {
            const int pc = min(p + u, np - 1);
            f[u] = fade[(long)pc * a.H];
            if (VW == 4) ld4<float>(w + pc * step, add[u]);
            else add[u][0] = w[pc * step];
        }
#pragma unroll
        for (int u = 0; u < SD_AHEAD; ++u) {
            if (p + u >= np) break;
            if (VW == 4)
                *reinterpret_cast<f32x4*>(w + (p + u) * step) =
                    f32x4{S[0], S[1], S[2], S[3]};
            else
                w[(p + u) * step] = S[0];
#pragma unroll
            for (int v = 0; v < VW; ++v) S[v] = f[u] * S[v] + add[u][v];
        }
    }
    if (VW == 4) *reinterpret_cast<f32x4*>(slot) = f32x4{S[0], S[1], S[2], S[3]};
    else *slot = S[0];
}

// (piece, head, 64-column block); wave w owns token rows 16w .. 16w+15 of the
// piece and needs no other wave's results. MS: LDS row stride of its masked
// C B^T tile, in the C layout's rows and read back as the A operand.
constexpr int SD_MS = SD_L + 4;

template <typename T, int VT, bool VEC>
__global__ void __launch_bounds__(SD_THREADS)
ssd_outputs_kernel(SsdArgs a) {
    __shared__ __attribute__((aligned(16))) float ms[SD_THREADS / WAVE]
                                                    [16 * SD_MS];
    __shared__ double As[SD_L];
    __shared__ float ds[SD_L];
    int lo, n;
    if (!sd_piece(a.cu, a.B, blockIdx.x, &lo, &n)) return;
    const int h = blockIdx.y, g = h / (a.H / a.G);
    const int v0 = blockIdx.z * SD_L;
    const int tid = threadIdx.x, lane = tid % WAVE;
    const int wid = __builtin_amdgcn_readfirstlane(tid / WAVE);
    const int lg = lane >> 4, li = lane & 15;
    const int N = a.N, V = a.V;
    if (wid == 0) {
        float d;
        double A;
        sd_decay<T>(a, h, lo, n, lane, &d, &A);
        As[lane] = A;
        ds[lane] = d;
    }
    __syncthreads();
    const int t0 = wid * 16;
    if (t0 >= n) return;                // no workgroup barrier below
    const T* X = (const T*)a.xbc + (long)h * V;
    const T* Bp = (const T*)a.xbc + (long)a.H * V + (long)g * N;
    const T* Cp = Bp + (long)a.G * N;
    const T* crow = Cp + (long)(lo + min(t0 + li, n - 1)) * a.xs;
    const float* S = a.ws + ((long)blockIdx.x * a.H + h) * N * V;

    f32x4 acc[VT], cb[4];
#pragma unroll
    for (int v = 0; v < VT; ++v) acc[v] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; ++j) cb[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    // C S and C B^T share the C fragments
    for (int k = 0; k < N; k += 16) {
        const int kc = k + lg * 4;
        float c[4];
        ld4_row<T, VEC>(crow, kc, N, c);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (j > wid) continue;      // keys after every row of the wave
            float bb[4];
            ld4_row<T, VEC>(Bp + (long)(lo + min(j * 16 + li, n - 1)) * a.xs,
                            kc, N, bb);
#pragma unroll
            for (int e = 0; e < 4; ++e)
                cb[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(c[e], bb[e],
                                                             cb[j], 0, 0, 0);
        }
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int col = v0 + v * 16 + li;
            float s[4];
#pragma unroll
            for (int e = 0; e < 4; ++e)
                s[e] = kc + e < N && col < V ? S[(long)(kc + e) * V + col]
                                             : 0.f;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                acc[v] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    c[e], s[e], acc[v], 0, 0, 0);
        }
    }
    float* m = ms[wid];
    double At[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        At[r] = As[t0 + lg * 4 + r];
        const float f = expf((float)At[r]);
#pragma unroll
        for (int v = 0; v < VT; ++v) acc[v][r] *= f;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        if (j > wid) continue;
        const int s = j * 16 + li;
        const double Asv = As[s];
        const float d = ds[s];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = t0 + lg * 4 + r;
            m[(lg * 4 + r) * SD_MS + s] =
                s <= t ? cb[j][r] * expf((float)(At[r] - Asv)) * d : 0.f;
        }
    }
    WAVE_LDS_SYNC();
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        if (j > wid) continue;
        const f32x4 mv = *reinterpret_cast<const f32x4*>(
            m + li * SD_MS + j * 16 + lg * 4);
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int col = v0 + v * 16 + li;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int s = min(j * 16 + lg * 4 + e, n - 1);
                const float x =
                    col < V ? ldf(X + (long)(lo + s) * a.xs + col) : 0.f;
                acc[v] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    mv[e], x, acc[v], 0, 0, 0);
            }
        }
    }
    const float skip = a.skip[h];
#pragma unroll
    for (int v = 0; v < VT; ++v) {
        const int col = v0 + v * 16 + li;
        if (col >= V) continue;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = t0 + lg * 4 + r;
            if (t >= n) continue;
            const float x = ldf(X + (long)(lo + t) * a.xs + col);
            a.y[(long)(lo + t) * a.H * V + (long)h * V + col] =
                acc[v][r] + skip * x;
        }
    }
}

template <typename T>
int ssd_dispatch(const SsdArgs& a, int pieces, bool vec, hipStream_t s) {
    const int vblk = (a.V + SD_L - 1) / SD_L;
    if (pieces == 0) {
        const bool v4 = vec && a.V % 4 == 0;
        int lpr = 1;
        const int units = v4 ? (a.V + 3) / 4 : a.V;
        while (lpr < units && lpr < SS_COLS / (v4 ? 4 : 1)) lpr <<= 1;
        const int need = (a.N * lpr + SS_THREADS - 1) / SS_THREADS;
        const dim3 grid(a.B, a.H, vblk);
#define SS_CASE(VW, R)                                                        \
    if (need <= R) {                                                          \
        hipLaunchKernelGGL((ssd_serial_kernel<T, VW, R>), grid,               \
                           dim3(SS_THREADS), 0, s, a, lpr);                   \
        return 0;                                                             \
    }
        if (a.N > SS_MAXN) return 1;
        if (v4) {
            SS_CASE(4, 1) SS_CASE(4, 2) SS_CASE(4, 4) SS_CASE(4, 8)
            SS_CASE(4, 16) SS_CASE(4, 32)
        } else {
            SS_CASE(1, 2) SS_CASE(1, 8) SS_CASE(1, 32) SS_CASE(1, 128)
        }
#undef SS_CASE
        return 1;
    }
    const int nblk = (a.N + SD_NS - 1) / SD_NS;
    const dim3 gs(pieces, a.H, nblk * vblk), go(pieces, a.H, vblk);
    const long NV = (long)a.N * a.V;
    const bool cv = NV % 4 == 0;
    const long per = SD_THREADS * (cv ? 4 : 1);
    const dim3 gc(a.B, a.H, (unsigned)((NV + per - 1) / per));
    const int vt = a.V <= 16 ? 1 : a.V <= 32 ? 2 : 4;
#define SD_RUN(K, VT, GRID)                                                   \
    do {                                                                      \
        if (vec)                                                              \
            hipLaunchKernelGGL((K<T, VT, true>), GRID, dim3(SD_THREADS), 0,   \
                               s, a);                                         \
        else                                                                  \
            hipLaunchKernelGGL((K<T, VT, false>), GRID, dim3(SD_THREADS), 0,  \
                               s, a);                                         \
    } while (0)
#define SD_VT(K, GRID)                                                        \
    do {                                                                      \
        if (vt == 1) SD_RUN(K, 1, GRID);                                      \
        else if (vt == 2) SD_RUN(K, 2, GRID);                                 \
        else SD_RUN(K, 4, GRID);                                              \
    } while (0)
    SD_VT(ssd_states_kernel, gs);
    if (cv)
        hipLaunchKernelGGL((ssd_carry_kernel<4>), gc, dim3(SD_THREADS), 0, s,
                           a);
    else
        hipLaunchKernelGGL((ssd_carry_kernel<1>), gc, dim3(SD_THREADS), 0, s,
                           a);
    SD_VT(ssd_outputs_kernel, go);
#undef SD_VT
#undef SD_RUN
    return 0;
}

}  // namespace

extern "C" int ssd_piece_tokens() { return SD_L; }

// pieces 0: token-serial form; else an upper bound of the number of 64-token
// pieces in the batch, ws [pieces, H, N, V] and fade [pieces, H] sized for
// it. c: 0 = bf16, 1 = fp32 activations. vec: N, V, xs and the addresses
// allow 4-element accesses. Returns nonzero when the state size is above 512.
extern "C" int launch_ssd_scan(const void* xbc, long xs, const void* dt,
                               long dts, const float* dt_bias,
                               const float* rate, const float* skip,
                               float* state, const int* state_slots,
                               const int* cu, const int* positions, float* y,
                               float* ws, float* fade, int pieces, int B,
                               int H, int G, int N, int V, int c, int vec,
                               hipStream_t s) {
    if (B == 0) return 0;
    SsdArgs a{xbc, xs, dt, dts, dt_bias, rate, skip, state, state_slots, cu,
              positions, y, ws, fade, B, H, G, N, V};
    if (c) return ssd_dispatch<float>(a, pieces, vec != 0, s);
    return ssd_dispatch<unsigned short>(a, pieces, vec != 0, s);
}
