// Kernels of decoders that mix a token with the ones right before it ahead of attention or of a
// recurrence, and whose layers take an input of the token's own:
//   conv_norm_store   causal per-channel filter over projected q / k / v, RMS norm per q and k head,
//                     k and v written to their cache slot; the filter's kept inputs
//   shift_mix         h + (previous h - h) mu_i for several vectors mu_i; the kept row
//   relu_squared      max(u, 0)^2
//   token_gate        gelu_tanh(z) times a run of the token's row in a table
// Filters, norms and mixes in fp32.
//
// Sequence layout: `cu_q` [B+1] rows of each sequence (null: row b is sequence b), `positions` [T],
// `slots` [B] state slot per sequence (< 0: unused), `row_seq` [T] the sequence of each row (< 0:
// none; given with cu_q).  A sequence of one row (every row of a decode step) has its kept inputs
// renewed by the kernel itself, whose threads own their channels; longer portions by the tail kernel
// behind it, when every row has read the old ones.
#include "hybrid_conv.h"

using namespace hyb;

// Where row t (the same for every lane of a wave) stands.
struct RowPlace {
    int slot, off, pos;      // state slot (< 0: none), index inside the portion, position
    bool single;             // the only row of its sequence in this step
    RowPlace() = default;
    __device__ __forceinline__ RowPlace(long t, const int* cu_q, const int* positions, const int* slots,
                                        const int* row_seq) {
        const int b = cu_q ? uniform(row_seq[t]) : (int)t;
        slot = b >= 0 ? uniform(slots[b]) : -1;
        pos = uniform(positions[t]);
        off = 0; single = true;
        if (cu_q && b >= 0) {
            const int s0 = uniform(cu_q[b]);
            off = (int)t - s0;
            single = uniform(cu_q[b + 1]) - s0 == 1;
        }
    }
    static __device__ __forceinline__ int uniform(int v) { return __builtin_amdgcn_readfirstlane(v); }
};

struct FilterArgs {
    long x_stride;
    const float* w;          // [C, taps], the last column meets the current token
    float* tail;             // [slots, taps - 1, C]
    const float *qw, *kw;    // [D]
    const int *slot_mapping, *cu_q, *positions, *slots, *row_seq;
    long T_;
    int H, G, D, E, C, taps;
    float eps;
};

// eight elements as they are in memory, widened when they are needed
template <typename T> struct Raw8;
template <> struct Raw8<bf16_t> {
    uint4 v;
    __device__ __forceinline__ void load(const bf16_t* p) { v = *reinterpret_cast<const uint4*>(p); }
    __device__ __forceinline__ void widen(float* o) const {
        const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            o[2 * i] = __uint_as_float(w[i] << 16);
            o[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
        }
    }
};
template <> struct Raw8<float> {
    float4 a, b;
    __device__ __forceinline__ void load(const float* p) {
        a = *reinterpret_cast<const float4*>(p);
        b = *reinterpret_cast<const float4*>(p + 4);
    }
    __device__ __forceinline__ void widen(float* o) const {
        o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w;
        o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
    }
};

// A group of LPH neighbouring lanes owns one head (q heads first, then k, then v), eight channels per
// lane, and walks ROWS rows, whose inputs are all requested ahead, with the filter's window in
// registers: an input is loaded once per group of rows.  grid (row groups, groups of 256 / LPH heads).
template <typename T, int TAPS, int LPH, int ROWS>
__global__ void __launch_bounds__(256)
conv_norm_store_kernel(const T* __restrict__ x, const FilterArgs a, T* __restrict__ q_out,
                       T* __restrict__ k_cache, T* __restrict__ v_cache) {
    const int hd = blockIdx.y * (256 / LPH) + threadIdx.x / LPH, d = (threadIdx.x % LPH) * 8;
    const int H = a.H, G = a.G, D = a.D, E = a.E;
    if (hd >= H + 2 * G) return;                             // (whole groups leave)
    const bool isq = hd < H, isv = hd >= H + G;
    const int n = isv ? E : D;
    const int c = (isv ? (H + G) * D + (hd - H - G) * E : hd * D) + d;
    const bool live = d < n;
    const long t0 = (long)blockIdx.x * ROWS;
    Raw8<T> in[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; ++r)
        if (live && t0 + r < a.T_) in[r].load(x + (t0 + r) * a.x_stride + c);
    RowPlace places[ROWS];
    int rows[ROWS];                                          // cache row of each
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        const long t = min(t0 + r, a.T_ - 1);
        places[r] = RowPlace(t, a.cu_q, a.positions, a.slots, a.row_seq);
        rows[r] = a.slot_mapping ? RowPlace::uniform(a.slot_mapping[t]) : -1;
    }
    float w[8][TAPS], gain[8], hist[TAPS > 1 ? TAPS - 1 : 1][8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        gain[i] = live && !isv ? (isq ? a.qw : a.kw)[d + i] : 0.f;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[i][j] = live ? a.w[(long)(c + i) * TAPS + j] : 0.f;
    }
    bool fresh = true;                                       // the window is not this row's
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        const long t = t0 + r;
        if (t >= a.T_) return;
        const RowPlace& at = places[r];
        if (at.slot < 0) {
            fresh = true;
            if (isq && live) {
                const float zero[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
                store_run8<T>(q_out + (t * H + hd) * (long)D + d, zero);
            }
            continue;
        }
        float* tl = a.tail + (long)at.slot * (TAPS - 1) * a.C + c;
        float cur[8], y[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) cur[i] = 0.f;
        if (live) in[r].widen(cur);
        if (fresh || at.off == 0) {
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) {
                const int back = TAPS - 1 - j;
#pragma unroll
                for (int i = 0; i < 8; ++i) hist[j][i] = 0.f;
                if (!live || at.pos < back) continue;
                if (at.off >= back) load_run<T, 8>(x + (t - back) * a.x_stride + c, hist[j]);
                else load_run<float, 8>(tl + (long)(TAPS - 1 + at.off - back) * a.C, hist[j]);
            }
            fresh = false;
        }
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            float s = cur[i] * w[i][TAPS - 1];
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) s += hist[j][i] * w[i][j];
            y[i] = s;
            ss += s * s;
        }
#pragma unroll
        for (int o = 1; o < LPH; o <<= 1) ss += __shfl_xor(ss, o, kWave);
        if (!isv) {
            const float rr = rsqrtf(ss / (float)n + a.eps);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] *= rr * gain[i];
        }
        if (live) {
            if (isq) store_run8<T>(q_out + (t * H + hd) * (long)D + d, y);
            else {
                const long slot = rows[r];
                if (slot >= 0 && k_cache) {
                    if (isv) store_run8<T>(v_cache + (slot * G + hd - H - G) * (long)E + d, y);
                    else store_run8<T>(k_cache + (slot * G + hd - H) * (long)D + d, y);
                }
            }
        }
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) {
            const float* next = j + 1 < TAPS - 1 ? hist[j + 1 < TAPS - 1 ? j + 1 : 0] : cur;
#pragma unroll
            for (int i = 0; i < 8; ++i) hist[j][i] = next[i];
        }
        if (TAPS > 1 && at.single && live) {
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j) store_run8<float>(tl + (long)j * a.C, hist[j]);
        }
    }
}

// Any sizes, any number of taps: one wave per (row, head), channel by channel; q and k heads are
// filtered twice (once for the sum of squares).  The tail kernel keeps the inputs of every sequence.
template <typename T>
__global__ void __launch_bounds__(256)
conv_norm_store_any_kernel(const T* __restrict__ x, const FilterArgs a, T* __restrict__ q_out,
                           T* __restrict__ k_cache, T* __restrict__ v_cache) {
    const long t = blockIdx.x;
    const int hd = blockIdx.y * 4 + threadIdx.x / kWave, lane = threadIdx.x & (kWave - 1);
    const int H = a.H, G = a.G, D = a.D, E = a.E, taps = a.taps;
    if (hd >= H + 2 * G) return;
    const bool isq = hd < H, isv = hd >= H + G;
    const int n = isv ? E : D;
    const int c0 = isv ? (H + G) * D + (hd - H - G) * E : hd * D;
    const RowPlace at(t, a.cu_q, a.positions, a.slots, a.row_seq);
    T* dst;
    if (isq) dst = q_out + (t * H + hd) * (long)D;
    else {
        const long slot = a.slot_mapping ? a.slot_mapping[t] : -1;
        if (slot < 0 || !k_cache) return;
        dst = isv ? v_cache + (slot * G + hd - H - G) * (long)E : k_cache + (slot * G + hd - H) * (long)D;
    }
    auto filtered = [&](int d) -> float {
        const int c = c0 + d;
        float s = 0.f;
        for (int j = 0; j < taps; ++j) {
            const int back = taps - 1 - j;
            if (at.pos < back) continue;
            const float v = at.off >= back ? ld(x + (t - back) * a.x_stride + c)
                                           : a.tail[((long)at.slot * (taps - 1) + taps - 1 + at.off - back) * a.C + c];
            s += v * a.w[(long)c * taps + j];
        }
        return s;
    };
    if (at.slot < 0) {
        if (isq) for (int d = lane; d < n; d += kWave) st(dst + d, 0.f);
        return;
    }
    if (isv) {
        for (int d = lane; d < n; d += kWave) st(dst + d, filtered(d));
        return;
    }
    float ss = 0.f;
    for (int d = lane; d < n; d += kWave) { const float v = filtered(d); ss += v * v; }
    const float rr = rsqrtf(wave_sum(ss) / (float)n + a.eps);
    const float* gain = isq ? a.qw : a.kw;
    for (int d = lane; d < n; d += kWave) st(dst + d, filtered(d) * rr * gain[d]);
}

// out[i, t, c] = h[t, c] + (prev - h[t, c]) mu[i, c]; a thread owns VEC channels and walks `rows_per`
// rows.  NM > 0: that many mixes, their vectors in registers.
template <typename T, int VEC, int NM>
__global__ void __launch_bounds__(256)
shift_mix_kernel(const T* __restrict__ h, const float* __restrict__ mu, float* __restrict__ tail,
                 const int* __restrict__ cu_q, const int* __restrict__ positions,
                 const int* __restrict__ slots, const int* __restrict__ row_seq, T* __restrict__ out,
                 long T_, int W, int nm, int rows_per) {
    const int c = (blockIdx.y * blockDim.x + threadIdx.x) * VEC;
    if (c >= W) return;
    float m[NM ? NM : 1][VEC];
    if constexpr (NM > 0) {
#pragma unroll
        for (int k = 0; k < NM; ++k)
#pragma unroll
            for (int i = 0; i < VEC; ++i) m[k][i] = mu[(long)k * W + c + i];
    }
    float prev[VEC], cur[VEC];
    bool fresh = true;
    for (int r = 0; r < rows_per; ++r) {
        const long t = (long)blockIdx.x * rows_per + r;
        if (t >= T_) return;
        const RowPlace at(t, cu_q, positions, slots, row_seq);
        float* tl = tail + (long)at.slot * W + c;
        if constexpr (VEC == 8) load_run<T, 8>(h + t * W + c, cur);
        else cur[0] = ld(h + t * W + c);
        if (at.slot < 0 || at.pos == 0) {
#pragma unroll
            for (int i = 0; i < VEC; ++i) prev[i] = 0.f;
        } else if (at.off == 0) {
#pragma unroll
            for (int i = 0; i < VEC; ++i) prev[i] = tl[i];
        } else if (fresh) {
#pragma unroll
            for (int i = 0; i < VEC; ++i) prev[i] = ld(h + (t - 1) * W + c + i);
        }
        fresh = false;
        auto mix = [&](int k, const float* mk) {
            T* dst = out + ((long)k * T_ + t) * W + c;
            float y[VEC];
#pragma unroll
            for (int i = 0; i < VEC; ++i) y[i] = cur[i] + (prev[i] - cur[i]) * mk[i];
            if constexpr (VEC == 8) store_run8<T>(dst, y);
            else st(dst, y[0]);
        };
        if constexpr (NM > 0) {
#pragma unroll
            for (int k = 0; k < NM; ++k) mix(k, m[k]);
        } else {
            for (int k = 0; k < nm; ++k) mix(k, mu + (long)k * W + c);
        }
#pragma unroll
        for (int i = 0; i < VEC; ++i) prev[i] = cur[i];
        if (at.slot >= 0 && at.single) {
#pragma unroll
            for (int i = 0; i < VEC; ++i) tl[i] = cur[i];
        }
    }
}

template <typename T, int VEC>
__global__ void relu_squared_kernel(const T* __restrict__ u, long u_stride, T* __restrict__ act, int n) {
    const long t = blockIdx.y;
    for (int c = (blockIdx.x * blockDim.x + threadIdx.x) * VEC; c < n; c += gridDim.x * blockDim.x * VEC) {
        if constexpr (VEC == 8) {
            float z[8];
            load_run<T, 8>(u + t * u_stride + c, z);
#pragma unroll
            for (int j = 0; j < 8; ++j) { z[j] = fmaxf(z[j], 0.f); z[j] *= z[j]; }
            store_run8<T>(act + t * (long)n + c, z);
        } else {
            const float z = fmaxf(ld(u + t * u_stride + c), 0.f);
            st(act + t * (long)n + c, z * z);
        }
    }
}

// out[t, c] = gelu_tanh(z[t, c]) * table[ids[t], c] (table: already moved to the run's first column)
template <typename T, int VEC>
__global__ void token_gate_kernel(const T* __restrict__ z, long z_stride, const int* __restrict__ ids,
                                  const T* __restrict__ table, long table_stride, T* __restrict__ out,
                                  long T_, int n) {
    const int runs = n / VEC;
    for (long i = blockIdx.x * (long)blockDim.x + threadIdx.x; i < T_ * runs; i += (long)gridDim.x * blockDim.x) {
        const long t = i / runs;
        const int c = (int)(i - t * runs) * VEC;
        const T* zr = z + t * z_stride + c;
        const T* er = table + (long)ids[t] * table_stride + c;
        if constexpr (VEC == 8) {
            float a[8], e[8];
            load_run<T, 8>(zr, a);
            load_run<T, 8>(er, e);
#pragma unroll
            for (int j = 0; j < 8; ++j) a[j] = gelu_tanh_(a[j]) * e[j];
            store_run8<T>(out + t * n + c, a);
        } else {
            st(out + t * n + c, gelu_tanh_(ld(zr)) * ld(er));
        }
    }
}

static inline int threads_for(int n) { return n >= 1024 ? 512 : n >= 256 ? 256 : n > 64 ? 128 : 64; }

template <typename T>
static void launch_tail(const void* x, long x_stride, void* tail, const void* cu_q, const void* positions,
                        const void* slots, int B, int C, int taps, int skip_single, hipStream_t s) {
    const int th = threads_for(C);
    hipLaunchKernelGGL(short_conv_tail_kernel<T>, dim3((C + th - 1) / th, B), dim3(th), 0, s, (const T*)x,
                       x_stride, (float*)tail, (const int*)cu_q, (const int*)positions, (const int*)slots,
                       C, taps, skip_single);
}

extern "C" {

// x [T, >= C] (rows x_stride apart): q (H heads of D), k (G of D), v (G of E) side by side; q_out
// [T, H, D]; caches contiguous [slot, G, D|E]; slot_mapping [T] (< 0: nothing stored).
int hyb_conv_norm_store(const void* x, long x_stride, const void* w, void* tail, const void* qw,
                        const void* kw, float eps, void* q_out, void* k_cache, void* v_cache,
                        const void* slot_mapping, const void* cu_q, const void* positions,
                        const void* slots, const void* row_seq, long T_, int B, int H, int G, int D,
                        int E, int taps, int dt, hipStream_t s) {
    if (T_ <= 0) return 0;
    if (taps < 1 || (cu_q && !row_seq) || (taps > 1 && !tail) || B > 65535 || H <= 0 || G <= 0) return 1;
    if (!cu_q && B < T_) return 1;                           // row b is sequence b
    FilterArgs a{};
    a.x_stride = x_stride; a.w = (const float*)w; a.tail = (float*)tail;
    a.qw = (const float*)qw; a.kw = (const float*)kw; a.slot_mapping = (const int*)slot_mapping;
    a.cu_q = (const int*)cu_q; a.positions = (const int*)positions; a.slots = (const int*)slots;
    a.row_seq = (const int*)row_seq; a.T_ = T_; a.H = H; a.G = G; a.D = D; a.E = E;
    a.C = (H + G) * D + G * E; a.taps = taps; a.eps = eps;
    const int heads = H + 2 * G, longest = D > E ? D : E;
    const size_t align = (size_t)x | (size_t)tail | (size_t)q_out | (size_t)k_cache | (size_t)v_cache;
    const bool runs = D % 8 == 0 && E % 8 == 0 && longest <= 512 && x_stride % 8 == 0 && align % 16 == 0;
    int own = 0;                                             // the kernel keeps single rows' inputs
#define FILTER_ROWS(TAPS, LPH, ROWS)                                                               \
    HYB_DISPATCH(dt, hipLaunchKernelGGL((conv_norm_store_kernel<T, TAPS, LPH, ROWS>),              \
                                        dim3((unsigned)((T_ + ROWS - 1) / ROWS),                   \
                                             (heads + 256 / LPH - 1) / (256 / LPH)), dim3(256), 0, s, \
                                        (const T*)x, a, (T*)q_out, (T*)k_cache, (T*)v_cache))
#define FILTER(TAPS, LPH)                                        \
    do {                                                         \
        if (T_ >= 2048) FILTER_ROWS(TAPS, LPH, 8);               \
        else FILTER_ROWS(TAPS, LPH, 1);                          \
    } while (0)
#define FILTER_TAPS(TAPS)                              \
    do {                                               \
        if (longest <= 64) FILTER(TAPS, 8);            \
        else if (longest <= 128) FILTER(TAPS, 16);     \
        else if (longest <= 256) FILTER(TAPS, 32);     \
        else FILTER(TAPS, 64);                         \
    } while (0)
    if (runs && taps <= 4) {
        own = 1;
        if (taps == 1) FILTER_TAPS(1);
        else if (taps == 2) FILTER_TAPS(2);
        else if (taps == 3) FILTER_TAPS(3);
        else FILTER_TAPS(4);
    } else {
        HYB_DISPATCH(dt, hipLaunchKernelGGL(conv_norm_store_any_kernel<T>, dim3(T_, (heads + 3) / 4),
                                            dim3(256), 0, s, (const T*)x, a, (T*)q_out, (T*)k_cache,
                                            (T*)v_cache));
    }
#undef FILTER_TAPS
#undef FILTER
#undef FILTER_ROWS
    if (hipGetLastError() != hipSuccess) return 2;
    if (taps > 1 && B > 0 && (cu_q || !own))
        HYB_DISPATCH(dt, launch_tail<T>(x, x_stride, tail, cu_q, positions, slots, B, a.C, taps, own, s));
    return HYB_LAUNCH_OK();
}

// h [T, W] contiguous; mu [nm, W]; tail [slots, 1, W]; out [nm, T, W]
int hyb_shift_mix(const void* h, const void* mu, void* tail, const void* cu_q, const void* positions,
                  const void* slots, const void* row_seq, void* out, long T_, int B, int W, int nm,
                  int dt, hipStream_t s) {
    if (T_ <= 0 || nm <= 0) return 0;
    if ((cu_q && !row_seq) || B > 65535 || (!cu_q && B < T_)) return 1;
    const bool vec = W % 8 == 0 && ((size_t)h | (size_t)out) % 16 == 0;
    const int cols = vec ? W / 8 : W, th = cols >= 256 ? 256 : cols > 64 ? 128 : 64;
    const int rows_per = T_ >= 2048 ? 8 : 1;
    const dim3 grid((unsigned)((T_ + rows_per - 1) / rows_per), (cols + th - 1) / th);
#define SHIFT(VEC, NM)                                                                             \
    HYB_DISPATCH(dt, hipLaunchKernelGGL((shift_mix_kernel<T, VEC, NM>), grid, dim3(th), 0, s,      \
                                        (const T*)h, (const float*)mu, (float*)tail, (const int*)cu_q, \
                                        (const int*)positions, (const int*)slots, (const int*)row_seq, \
                                        (T*)out, T_, W, nm, rows_per))
    if (vec && nm == 5) SHIFT(8, 5);
    else if (vec) SHIFT(8, 0);
    else SHIFT(1, 0);
#undef SHIFT
    if (hipGetLastError() != hipSuccess) return 2;
    if (cu_q && B > 0) HYB_DISPATCH(dt, launch_tail<T>(h, W, tail, cu_q, positions, slots, B, W, 2, 1, s));
    return HYB_LAUNCH_OK();
}

int hyb_relu_squared(const void* u, long u_stride, void* act, long T_, int n, int dt, hipStream_t s) {
    if (T_ <= 0 || n <= 0) return 0;
    const bool vec = n % 8 == 0 && u_stride % 8 == 0 && ((size_t)u | (size_t)act) % 16 == 0;
    const int need = (n / (vec ? 8 : 1) + 255) / 256;
    const int bx = need > 64 ? 64 : need;
    for (long t0 = 0; t0 < T_; t0 += 65535) {          // blockIdx.y holds at most 65535 rows
        const long nrow = T_ - t0 < 65535 ? T_ - t0 : 65535;
#define RSQ(VEC)                                                                                   \
        HYB_DISPATCH(dt, hipLaunchKernelGGL((relu_squared_kernel<T, VEC>), dim3(bx, nrow), dim3(256), 0, s, \
                                            (const T*)u + t0 * u_stride, u_stride,                 \
                                            (T*)act + t0 * (long)n, n))
        if (vec) RSQ(8); else RSQ(1);
#undef RSQ
    }
    return HYB_LAUNCH_OK();
}

// table: its rows table_stride elements apart, the run of n starting at column `offset`
int hyb_token_gate(const void* z, long z_stride, const void* ids, const void* table, long table_stride,
                   long offset, void* out, long T_, int n, int dt, hipStream_t s) {
    if (T_ <= 0 || n <= 0) return 0;
    const bool vec = n % 8 == 0 && z_stride % 8 == 0 && table_stride % 8 == 0 && offset % 8 == 0 &&
                     ((size_t)z | (size_t)table | (size_t)out) % 16 == 0;
    const long work = T_ * (n / (vec ? 8 : 1));
    const int blocks = (int)((work + 255) / 256 > 16384 ? 16384 : (work + 255) / 256);
#define TGT(VEC)                                                                                   \
    HYB_DISPATCH(dt, hipLaunchKernelGGL((token_gate_kernel<T, VEC>), dim3(blocks), dim3(256), 0, s, \
                                        (const T*)z, z_stride, (const int*)ids, (const T*)table + offset, \
                                        table_stride, (T*)out, T_, n))
    if (vec) TGT(8); else TGT(1);
#undef TGT
    return HYB_LAUNCH_OK();
}

}  // extern "C"
