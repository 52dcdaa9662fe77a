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
//    ssd_prep     piece table, step sizes d and running log decays A;
//    ssd_states   what a piece adds to the state, sum_t exp(A_L - A_t) d_t
//                 B_t x_t^T;
//    ssd_carry    walks the pieces of each (sequence, head) in order, turning
//                 those into the state at every piece's start;
//    ssd_outputs  y = (C B^T . exp(A_t - A_s) d_s, s <= t) X + exp(A_t) C S.
//    Products with an fp32 operand run on v_mfma_f32_16x16x4_f32, fp32 sums,
//    for bf16 and fp32 activations alike; C B^T of bf16 activations runs on
//    v_mfma_f32_16x16x32_bf16 (its products are exact). Running log decays
//    are kept in fp64, so that their differences hold fp32 precision however
//    far they run.
//
// Fragment maps of v_mfma_f32_16x16x4_f32: A: lane -> row l & 15, k = l >> 4;
// B: lane -> column l & 15, k = l >> 4; C: column l & 15, rows (l >> 4) * 4 +
// r. Which four k values a step takes is free as long as A and B agree: where
// a lane reads E neighbours at once, step e of E takes k = E (l >> 4) + e. With
// E = 8 the same registers are an A or B fragment of the bf16 instruction.
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
// eight neighbours at column c of a row of n; zeros past its end. VEC: n is a
// multiple of 8 and the addresses are aligned.
template <typename T> struct Row8;
template <> struct Row8<unsigned short> {
    short8 v;
    template <bool VEC>
    DEV_INLINE void load(const unsigned short* row, int c, int n) {
        v = short8{0, 0, 0, 0, 0, 0, 0, 0};
        if (VEC) {
            if (c < n) v = *reinterpret_cast<const short8*>(row + c);
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (c + e < n) v[e] = (short)row[c + e];
        }
    }
    DEV_INLINE float get(int e) const { return bf2f((unsigned short)v[e]); }
};
template <> struct Row8<float> {
    float v[8];
    template <bool VEC>
    DEV_INLINE void load(const float* row, int c, int n) {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = 0.f;
        if (VEC) {
            if (c < n) {
                ld4<float>(row + c, v);
                ld4<float>(row + c + 4, v + 4);
            }
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (c + e < n) v[e] = row[c + e];
        }
    }
    DEV_INLINE float get(int e) const { return v[e]; }
};
// acc += A B^T over the 32 columns that the lanes' pieces of both cover
DEV_INLINE f32x4 mma32(const Row8<unsigned short>& a,
                       const Row8<unsigned short>& b, f32x4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(
        __builtin_bit_cast(bf16x8, a.v), __builtin_bit_cast(bf16x8, b.v), acc,
        0, 0, 0);
}
DEV_INLINE f32x4 mma32(const Row8<float>& a, const Row8<float>& b, f32x4 acc) {
#pragma unroll
    for (int e = 0; e < 8; ++e)
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[e], b.v[e], acc, 0, 0,
                                                   0);
    return acc;
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
    // chunk form
    float* ws;              // [pieces, H, N, V]
    double* logs;           // [pieces, H, 64] running log decay A
    float* steps;           // [pieces, H, 64] d
    float* tails;           // [pieces, H, 64] d exp(A_L - A), 0 past the end
    float* fade;            // [pieces, H] exp(A_L)
    int* table;             // [pieces, 2] first row, rows (0: no such piece)
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

// wave per (piece, head)
template <typename T>
__global__ void __launch_bounds__(SD_THREADS) ssd_prep_kernel(SsdArgs a) {
    int lo = 0, n = 0;
    const bool ok = sd_piece(a.cu, a.B, blockIdx.x, &lo, &n);
    if (threadIdx.x == 0 && blockIdx.y == 0) {
        a.table[2 * blockIdx.x] = lo;
        a.table[2 * blockIdx.x + 1] = ok ? n : 0;
    }
    const int h = blockIdx.y * (SD_THREADS / WAVE) + threadIdx.x / WAVE;
    if (!ok || h >= a.H) return;
    const int lane = threadIdx.x % WAVE;
    float d;
    double A;
    sd_decay<T>(a, h, lo, n, lane, &d, &A);
    const double last = __shfl(A, WAVE - 1);
    const long row = (long)blockIdx.x * a.H + h, at = row * SD_L + lane;
    a.logs[at] = A;
    a.steps[at] = d;
    a.tails[at] = d * expf((float)(last - A));
    if (lane == 0) a.fade[row] = expf((float)last);
}

// (piece, head, 128-row x 64-column block of the state); a wave owns two
// 16-row tiles against all the block's columns.
constexpr int SD_NT = 2;
constexpr int SD_NS = SD_NT * 16 * (SD_THREADS / WAVE);

template <typename T, int VT>
__global__ void __launch_bounds__(SD_THREADS)
ssd_states_kernel(SsdArgs a) {
    const int lo = a.table[2 * blockIdx.x], n = a.table[2 * blockIdx.x + 1];
    if (n == 0) return;
    const int h = blockIdx.y, g = h / (a.H / a.G);
    const int vblk = (a.V + SD_L - 1) / SD_L;
    const int lane = threadIdx.x % WAVE;
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
    const int lg = lane >> 4, li = lane & 15;
    const int N = a.N, V = a.V;
    const int n0 = blockIdx.z / vblk * SD_NS + wid * SD_NT * 16;
    const int v0 = blockIdx.z % vblk * SD_L;
    if (n0 >= N) return;                // no workgroup barrier below
    // columns past the end repeat the last one and are not stored
    const T* X = (const T*)a.xbc + (long)h * V;
    const T* Bp = (const T*)a.xbc + (long)a.H * V + (long)g * N;
    int xc[VT], bc[SD_NT];
#pragma unroll
    for (int v = 0; v < VT; ++v) xc[v] = min(v0 + v * 16 + li, V - 1);
#pragma unroll
    for (int i = 0; i < SD_NT; ++i) bc[i] = min(n0 + i * 16 + li, N - 1);
    const float* tail = a.tails + ((long)blockIdx.x * a.H + h) * SD_L;
    f32x4 acc[SD_NT][VT];
#pragma unroll
    for (int i = 0; i < SD_NT; ++i)
#pragma unroll
        for (int v = 0; v < VT; ++v) acc[i][v] = f32x4{0.f, 0.f, 0.f, 0.f};
    // rows past the end repeat the last one; their weight is zero
    const int kend = (n + 15) / 16 * 16;
    for (int k0 = 0; k0 < kend; k0 += 16) {
        float xv[4][VT], bv[4][SD_NT];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int t = k0 + u * 4 + lg;
            const long row = (long)(lo + min(t, n - 1)) * a.xs;
            const float w = tail[t];
#pragma unroll
            for (int v = 0; v < VT; ++v) xv[u][v] = ldf(X + row + xc[v]);
#pragma unroll
            for (int i = 0; i < SD_NT; ++i)
                bv[u][i] = ldf(Bp + row + bc[i]) * w;
        }
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int i = 0; i < SD_NT; ++i)
#pragma unroll
                for (int v = 0; v < VT; ++v)
                    acc[i][v] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                        bv[u][i], xv[u][v], acc[i][v], 0, 0, 0);
    }
    float* out = a.ws + ((long)blockIdx.x * a.H + h) * N * V;
#pragma unroll
    for (int i = 0; i < SD_NT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = n0 + i * 16 + lg * 4 + r;
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const int c = v0 + v * 16 + li;
                if (row < N && c < V) out[(long)row * V + c] = acc[i][v][r];
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

// (piece, head, 64-column block of VT 16-column tiles). First wave w forms the
// decayed C B^T of token rows 16w .. 16w+15 in LDS, in the C layout; then every
// wave owns one column tile of RT = VT row tiles (so a state column is read by
// one wave), reading the LDS tile back as the A operand. SD_MS: its row stride.
constexpr int SD_MS = SD_L + 4;

template <typename T, int VT, bool VEC>
__global__ void __launch_bounds__(SD_THREADS)
ssd_outputs_kernel(SsdArgs a) {
    constexpr int RT = VT;
    static_assert(SD_THREADS / WAVE * RT == 4 * VT, "waves cover the tiles");
    __shared__ __attribute__((aligned(16))) float ms[SD_L * SD_MS];
    const int lo = a.table[2 * blockIdx.x], n = a.table[2 * blockIdx.x + 1];
    if (n == 0) return;
    const int lane = threadIdx.x % WAVE;
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
    const int h = blockIdx.y, g = h / (a.H / a.G);
    const int lg = lane >> 4, li = lane & 15;
    const int N = a.N, V = a.V;
    const long hp = (long)blockIdx.x * a.H + h;
    const T* X = (const T*)a.xbc + (long)h * V;
    const T* Bp = (const T*)a.xbc + (long)a.H * V + (long)g * N;
    const T* Cp = Bp + (long)a.G * N;
    const double* As = a.logs + hp * SD_L;
    const float* ds = a.steps + hp * SD_L;
    // rows past the end repeat the last one and are not stored
    const T *brow[4], *crow[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const long row = (long)(lo + min(j * 16 + li, n - 1)) * a.xs;
        brow[j] = Bp + row;
        crow[j] = Cp + row;
    }
    const int t0 = wid * 16;
    // everything that needs no product yet is fetched ahead: the first step of
    // C S, the wave's columns of X, its rows' log decays
    const float* S = a.ws + hp * N * V;
    const int vt = wid % VT, rt0 = wid / VT * RT;
    // columns past the end repeat the last one and are not stored
    const int c0 = blockIdx.z * SD_L + vt * 16 + li, col = min(c0, V - 1);
    struct Step { Row8<T> c[RT]; float s[8]; };
    auto load = [&](Step& st, int k) {
        const int kc = k + lg * 8;
        // rows of S past the end repeat the last one; C is zero there
#pragma unroll
        for (int e = 0; e < 8; ++e)
            st.s[e] = S[(long)min(kc + e, N - 1) * V + col];
#pragma unroll
        for (int i = 0; i < RT; ++i)
            st.c[i].template load<VEC>(crow[VT == 4 ? i : rt0 + i], kc, N);
    };
    Step cur, nxt;
    load(cur, 0);
    T xr[4][4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e)
            xr[j][e] = X[(long)(lo + min(j * 16 + lg * 4 + e, n - 1)) * a.xs +
                         col];
    if (t0 < n) {
        const T* own = Cp + (long)(lo + min(t0 + li, n - 1)) * a.xs;
        f32x4 cb[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) cb[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        double At[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) At[r] = As[t0 + lg * 4 + r];
        struct Keys { Row8<T> c, b[4]; };
        auto keys = [&](Keys& st, int k) {
            st.c.template load<VEC>(own, k + lg * 8, N);
#pragma unroll
            for (int j = 0; j < 4; ++j)     // tokens after every row: unused
                if (j <= wid)
                    st.b[j].template load<VEC>(brow[j], k + lg * 8, N);
        };
        Keys kc, kn;
        keys(kc, 0);
        for (int k = 0; k < N; k += 32) {
            if (k + 32 < N) keys(kn, k + 32);
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (j <= wid) cb[j] = mma32(kc.c, kc.b[j], cb[j]);
            kc = kn;
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
                ms[t * SD_MS + s] =
                    s <= t ? cb[j][r] * expf((float)(At[r] - Asv)) * d : 0.f;
            }
        }
    }
    f32x4 acc[RT];
#pragma unroll
    for (int i = 0; i < RT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < N; k += 32) {
        if (k + 32 < N) load(nxt, k + 32);
#pragma unroll
        for (int e = 0; e < 8; ++e)
#pragma unroll
            for (int i = 0; i < RT; ++i)
                acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    cur.c[i].get(e), cur.s[e], acc[i], 0, 0, 0);
        cur = nxt;
    }
#pragma unroll
    for (int i = 0; i < RT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r)
            acc[i][r] *= expf((float)As[(rt0 + i) * 16 + lg * 4 + r]);
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        if (j * 16 >= n || j >= rt0 + RT) continue;
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            if (rt0 + i < j || (rt0 + i) * 16 >= n) continue;
            const f32x4 mv = *reinterpret_cast<const f32x4*>(
                ms + ((rt0 + i) * 16 + li) * SD_MS + j * 16 + lg * 4);
#pragma unroll
            for (int e = 0; e < 4; ++e)
                acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    mv[e], ldf(&xr[j][e]), acc[i], 0, 0, 0);
        }
    }
    if (c0 >= V) return;
    const float skip = a.skip[h];
    float* y = a.y + (long)lo * a.H * V + (long)h * V + col;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        // row tile j, whose X rows are the C layout's rows
        if (j < rt0 || j >= rt0 + RT) continue;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = j * 16 + lg * 4 + r;
            if (t < n)
                y[(long)t * a.H * V] =
                    acc[VT == 4 ? j : j - rt0][r] + skip * ldf(&xr[j][r]);
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
    const dim3 gp(pieces, (a.H + SD_THREADS / WAVE - 1) / (SD_THREADS / WAVE));
    hipLaunchKernelGGL((ssd_prep_kernel<T>), gp, dim3(SD_THREADS), 0, s, a);
#define SD_STATES(VT)                                                         \
    hipLaunchKernelGGL((ssd_states_kernel<T, VT>), gs, dim3(SD_THREADS), 0, s, \
                       a)
    if (vt == 1) SD_STATES(1);
    else if (vt == 2) SD_STATES(2);
    else SD_STATES(4);
#undef SD_STATES
    if (cv)
        hipLaunchKernelGGL((ssd_carry_kernel<4>), gc, dim3(SD_THREADS), 0, s,
                           a);
    else
        hipLaunchKernelGGL((ssd_carry_kernel<1>), gc, dim3(SD_THREADS), 0, s,
                           a);
#define SD_OUTPUTS(VT, VC)                                                    \
    hipLaunchKernelGGL((ssd_outputs_kernel<T, VT, VC>), go, dim3(SD_THREADS), \
                       0, s, a)
    const bool v8 = vec && a.N % 8 == 0 && a.V % 8 == 0 && a.xs % 8 == 0;
    if (vt == 1 && v8) SD_OUTPUTS(1, true);
    else if (vt == 1) SD_OUTPUTS(1, false);
    else if (vt == 2 && v8) SD_OUTPUTS(2, true);
    else if (vt == 2) SD_OUTPUTS(2, false);
    else if (v8) SD_OUTPUTS(4, true);
    else SD_OUTPUTS(4, false);
#undef SD_OUTPUTS
    return 0;
}

}  // namespace

extern "C" int ssd_piece_tokens() { return SD_L; }

// pieces 0: token-serial form; else an upper bound of the number of 64-token
// pieces in the batch, ws, logs, steps, tails, fade and table (see SsdArgs)
// sized for it. c: 0 = bf16, 1 = fp32 activations. vec: N, V and xs allow
// 4-element accesses, xbc and state are 16-byte aligned. Returns nonzero when
// the state size is above 512.
extern "C" int launch_ssd_scan(const void* xbc, long xs, const void* dt,
                               long dts, const float* dt_bias,
                               const float* rate, const float* skip,
                               float* state, const int* state_slots,
                               const int* cu, const int* positions, float* y,
                               float* ws, double* logs, float* steps,
                               float* tails, float* fade, int* table,
                               int pieces, int B, int H, int G, int N, int V,
                               int c, int vec, hipStream_t s) {
    if (B == 0) return 0;
    SsdArgs a{xbc, xs, dt, dts, dt_bias, rate, skip, state, state_slots, cu,
              positions, y, ws, logs, steps, tails, fade, table, B, H, G, N,
              V};
    if (c) return ssd_dispatch<float>(a, pieces, vec != 0, s);
    return ssd_dispatch<unsigned short>(a, pieces, vec != 0, s);
}
