// Kernels of decoders with several residual streams and a norm without statistics:
//   hyper_norm          u = sum_s read[s] x_s;  h = tanh(alpha u) * w + b
//   hyper_update_norm   x_b <- sum_a mix[a, b] x_a + write[b] (y + g h'), all streams from the old
//                       ones, then hyper_norm of the new streams (the next sublayer's input)
//   corrected_route     fp32 router: softmax scores, choice by score + correction, weights from the
//                       scores alone, identity experts summed into one column
//   gelu_tanh_glu       gelu_tanh(gate) * up
// Nothing here needs a sum over a row except the router, so the stream kernels are element-wise:
// a thread owns VEC columns of one token, keeps that column of all S streams in registers and makes
// one pass over memory.
#include "hybrid_common.h"

using namespace hyb;

constexpr int MAX_STREAMS = 8;

template <typename T, int VEC>
__device__ __forceinline__ void load_vec(const T* p, float* o) {
    if constexpr (VEC == 4) Vec4<T>::load(p, o);
    else o[0] = ld(p);
}
template <int VEC>
__device__ __forceinline__ void store_f32(float* p, const float* v) {
    if constexpr (VEC == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    else p[0] = v[0];
}
template <typename T, int VEC>
__device__ __forceinline__ void store_vec(T* p, const float* v) {
    if constexpr (VEC == 4 && sizeof(T) == 2) {
        uint32_t w[2];
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            const __bf16 lo = (__bf16)v[2 * i], hi = (__bf16)v[2 * i + 1];
            w[i] = (uint32_t)__builtin_bit_cast(uint16_t, lo) |
                   ((uint32_t)__builtin_bit_cast(uint16_t, hi) << 16);
        }
        *reinterpret_cast<uint2*>(p) = make_uint2(w[0], w[1]);
    } else if constexpr (VEC == 4) {
        *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    } else {
        st(p, v[0]);
    }
}

// xi: streams as read (token stride xi_t, stream stride xi_s: 0 when the S streams are one row);
// xo: streams as written [T, S, W] (may be xi itself), null: nothing is updated.  y [T, W] rows
// y_stride apart; hs [T, W] and gs [T] (stride gs_t): the multiple of the sublayer's input that
// joins y, or null.  read null: no next input; else h [T, W].  Workgroup: `parts` per token row.
template <typename T, int S, int VEC>
__global__ void __launch_bounds__(256)
hyper_kernel(const float* xi, long xi_t, long xi_s, float* xo, const T* __restrict__ y,
             long y_stride, const T* __restrict__ hs, long hs_stride, const float* __restrict__ gs,
             long gs_t, const float* __restrict__ write, const float* __restrict__ mix,
             const float* __restrict__ read, const float* __restrict__ alpha,
             const float* __restrict__ w, const float* __restrict__ b, T* __restrict__ h, int W,
             int parts) {
    const long t = blockIdx.x / parts;
    const int c = ((int)(blockIdx.x - t * parts) * blockDim.x + threadIdx.x) * VEC;
    if (c >= W) return;
    float x[S][VEC];
#pragma unroll
    for (int a = 0; a < S; ++a) load_vec<float, VEC>(xi + t * xi_t + a * xi_s + c, x[a]);
    if (xo) {
        float yv[VEC], nx[S][VEC];
        load_vec<T, VEC>(y + t * y_stride + c, yv);
        if (hs) {
            float hv[VEC];
            load_vec<T, VEC>(hs + t * hs_stride + c, hv);
            const float g = gs[t * gs_t];
#pragma unroll
            for (int i = 0; i < VEC; ++i) yv[i] += g * hv[i];
        }
#pragma unroll
        for (int o = 0; o < S; ++o) {
            const float wo = write[o];
#pragma unroll
            for (int i = 0; i < VEC; ++i) nx[o][i] = wo * yv[i];
#pragma unroll
            for (int a = 0; a < S; ++a) {
                const float m = mix[a * S + o];
#pragma unroll
                for (int i = 0; i < VEC; ++i) nx[o][i] += m * x[a][i];
            }
        }
#pragma unroll
        for (int o = 0; o < S; ++o) {
            store_f32<VEC>(xo + (t * S + o) * (long)W + c, nx[o]);
#pragma unroll
            for (int i = 0; i < VEC; ++i) x[o][i] = nx[o][i];
        }
    }
    if (!read) return;
    float u[VEC], wv[VEC], bv[VEC];
#pragma unroll
    for (int i = 0; i < VEC; ++i) u[i] = 0.f;
#pragma unroll
    for (int a = 0; a < S; ++a) {
        const float r = read[a];
#pragma unroll
        for (int i = 0; i < VEC; ++i) u[i] += r * x[a][i];
    }
    load_vec<float, VEC>(w + c, wv);
    load_vec<float, VEC>(b + c, bv);
    const float al = alpha[0];
#pragma unroll
    for (int i = 0; i < VEC; ++i) u[i] = tanhf(al * u[i]) * wv[i] + bv[i];
    store_vec<T, VEC>(h + t * (long)W + c, u);
}

// sums of N values over a wave, the results spread over the lanes: every exchange halves the number
// of values a lane still carries (N a power of two).  A lane returns the total of value `slot`.
template <int N, int O = kWave / 2>
__device__ __forceinline__ float scatter_sum(float (&v)[N], int lane, int& slot) {
    if constexpr (N == 1) {
        float s = v[0];
#pragma unroll
        for (int o = O; o > 0; o >>= 1) s += __shfl_xor(s, o, kWave);
        return s;
    } else {
        const bool up = lane & O;
        float half[N / 2];
#pragma unroll
        for (int i = 0; i < N / 2; ++i) {
            const float send = up ? v[i] : v[i + N / 2];
            const float keep = up ? v[i + N / 2] : v[i];
            half[i] = keep + __shfl_xor(send, O, kWave);
        }
        slot = slot * 2 + (up ? 1 : 0);
        return scatter_sum<N / 2, O / 2>(half, lane, slot);
    }
}

// One workgroup (4 waves) per TOK token rows: the rows of the router matrix are read once per
// workgroup, eight at a time; then wave k softmaxes and chooses for token k.  z: [TOK][NR] in LDS.
template <typename T, int TOK, int VEC>
__global__ void __launch_bounds__(256)
corrected_route_kernel(const T* __restrict__ h, const float* __restrict__ wr,
                       const float* __restrict__ corr, float* __restrict__ dense, long T_, int W,
                       int NE, int NR, int top, float scale) {
    extern __shared__ float sm[];
    float* z = sm;                               // scores
    float* choice = sm + TOK * NR;
    float* red = choice + TOK * NR;              // [4 waves][8 * TOK]
    const long t0 = (long)blockIdx.x * TOK;
    const int wave = threadIdx.x / kWave, lane = threadIdx.x & (kWave - 1);
    for (int e0 = 0; e0 < NR; e0 += 8) {
        float acc[8 * TOK];
#pragma unroll
        for (int j = 0; j < 8 * TOK; ++j) acc[j] = 0.f;
        for (int c = threadIdx.x * VEC; c < W; c += 256 * VEC) {
            float hv[TOK][VEC];
#pragma unroll
            for (int k = 0; k < TOK; ++k) load_vec<T, VEC>(h + min(t0 + k, T_ - 1) * W + c, hv[k]);
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                float wv[VEC];
                load_vec<float, VEC>(wr + (long)min(e0 + j, NR - 1) * W + c, wv);
#pragma unroll
                for (int k = 0; k < TOK; ++k)
#pragma unroll
                    for (int i = 0; i < VEC; ++i) acc[k * 8 + j] += hv[k][i] * wv[i];
            }
        }
        int slot = 0;
        const float s = scatter_sum<8 * TOK>(acc, lane, slot);
        if ((lane & (kWave / (8 * TOK) - 1)) == 0) red[wave * 8 * TOK + slot] = s;
        __syncthreads();
        if (threadIdx.x < 8 * TOK) {
            const int k = threadIdx.x / 8, j = threadIdx.x & 7;
            if (e0 + j < NR) {
                float sj = 0.f;
                for (int w = 0; w < 4; ++w) sj += red[w * 8 * TOK + threadIdx.x];
                z[k * NR + e0 + j] = sj;
            }
        }
        __syncthreads();
    }
    if (wave >= TOK || t0 + wave >= T_) return;              // (no barrier below)
    float* zr = z + wave * NR;
    float* cr = choice + wave * NR;
    float* row = dense + (t0 + wave) * (NE + 1);
    float m = -INFINITY;
    for (int e = lane; e < NR; e += kWave) m = fmaxf(m, zr[e]);
    m = wave_max(m);
    float sum = 0.f;
    for (int e = lane; e < NR; e += kWave) sum += expf(zr[e] - m);
    sum = wave_sum(sum);
    for (int e = lane; e < NR; e += kWave) {
        const float s = expf(zr[e] - m) / sum;
        zr[e] = s;
        cr[e] = s + corr[e];
        if (e < NE) row[e] = 0.f;
    }
    // the r-th largest choice score not yet taken; every lane walks its own entries (its own LDS
    // words only), the wave agrees on the winner, ties to the lower index
    float total = 0.f, ident = 0.f;
    for (int pass = 0; pass < 2; ++pass) {
        const float f = pass ? scale / (total + 1e-20f) : 0.f;
        for (int r = 0; r < top; ++r) {
            float bv = -INFINITY;
            int be = NR;
            for (int e = lane; e < NR; e += kWave)
                if (cr[e] > bv) { bv = cr[e]; be = e; }
#pragma unroll
            for (int o = kWave / 2; o > 0; o >>= 1) {
                const float ov = __shfl_xor(bv, o, kWave);
                const int oe = __shfl_xor(be, o, kWave);
                if (ov > bv || (ov == bv && oe < be)) { bv = ov; be = oe; }
            }
            if (be >= NR) break;                             // (scores that are not numbers)
            const int owner = be & (kWave - 1);
            const float s = __shfl(lane == owner ? zr[be] : 0.f, owner, kWave);
            if (pass == 0) total += s;
            else if (be >= NE) ident += s * f;
            else if (lane == owner) row[be] = s * f;
            if (lane == owner) cr[be] = -INFINITY;
        }
        if (pass == 0)
            for (int e = lane; e < NR; e += kWave) cr[e] = zr[e] + corr[e];
    }
    if (lane == 0) row[NE] = ident;
}


// gu row = [gate C | up C]; act dense [T, C]; VEC columns per thread (8: aligned 16-byte runs)
template <typename T, int VEC>
__global__ void gelu_tanh_glu_kernel(const T* __restrict__ gu, long gu_stride, T* __restrict__ act,
                                     int C, int parts) {
    const long t = blockIdx.x / parts;
    const int c = ((int)(blockIdx.x - t * parts) * blockDim.x + threadIdx.x) * VEC;
    if (c >= C) return;
    const T* g = gu + t * gu_stride + c;
    if constexpr (VEC == 8) {
        float a[8], u[8];
        load_run<T, 8>(g, a);
        load_run<T, 8>(g + C, u);
#pragma unroll
        for (int j = 0; j < 8; ++j) a[j] = gelu_tanh_(a[j]) * u[j];
        store_run8<T>(act + t * (long)C + c, a);
    } else {
        st(act + t * (long)C + c, gelu_tanh_(ld(g)) * ld(g + C));
    }
}

template <typename T, int VEC>
static int launch_hyper(const void* xi, long xi_t, long xi_s, void* xo, const void* y, long y_stride,
                        const void* hs, long hs_stride, const void* gs, long gs_t, const void* write,
                        const void* mix, const void* read, const void* alpha, const void* w,
                        const void* b, void* h, long T_, int S, int W, hipStream_t s) {
    const int cols = (W + VEC - 1) / VEC;
    const int th = cols >= 256 ? 256 : cols > 128 ? 256 : cols > 64 ? 128 : 64;
    const int parts = (cols + th - 1) / th;
    if (T_ * parts > 0x7fffffffL) return 1;
#define HYPER(NS)                                                                                  \
    case NS:                                                                                       \
        hipLaunchKernelGGL((hyper_kernel<T, NS, VEC>), dim3((unsigned)(T_ * parts)), dim3(th), 0, s, \
                           (const float*)xi, xi_t, xi_s, (float*)xo, (const T*)y, y_stride,        \
                           (const T*)hs, hs_stride, (const float*)gs, gs_t, (const float*)write,   \
                           (const float*)mix, (const float*)read, (const float*)alpha,             \
                           (const float*)w, (const float*)b, (T*)h, W, parts);                     \
        break
    switch (S) {
        HYPER(1); HYPER(2); HYPER(3); HYPER(4); HYPER(5); HYPER(6); HYPER(7); HYPER(8);
        default: return 1;
    }
#undef HYPER
    return HYB_LAUNCH_OK();
}

extern "C" {

// See hyper_kernel.  xo null: hyper_norm alone (then read, alpha, w, b and h are given).
int hyb_hyper_update_norm(const void* xi, long xi_t, long xi_s, void* xo, const void* y,
                          long y_stride, const void* hs, long hs_stride, const void* gs, long gs_t,
                          const void* write, const void* mix, const void* read, const void* alpha,
                          const void* w, const void* b, void* h, long T_, int S, int W, int dt,
                          hipStream_t s) {
    if (T_ <= 0 || W <= 0) return 0;
    if (S < 1 || S > MAX_STREAMS) return 1;
    if ((xo && (!y || !write || !mix)) || (read && (!alpha || !w || !b || !h)) || (!xo && !read)) return 1;
    if (xo == xi && (xi_t != (long)S * W || (S > 1 && xi_s != W))) return 1;
    if (hs && !gs) return 1;
    const bool vec = W % 4 == 0 && xi_t % 4 == 0 && xi_s % 4 == 0 && y_stride % 4 == 0 &&
                     hs_stride % 4 == 0 &&
                     ((size_t)xi | (size_t)xo | (size_t)w | (size_t)b) % 16 == 0 &&
                     ((size_t)y | (size_t)hs | (size_t)h) % (dt == 0 ? 8 : 16) == 0;
#define HYPER_ARGS xi, xi_t, xi_s, xo, y, y_stride, hs, hs_stride, gs, gs_t, write, mix, read, alpha, \
                   w, b, h, T_, S, W, s
    if (vec) HYB_DISPATCH(dt, return (launch_hyper<T, 4>(HYPER_ARGS)));
    HYB_DISPATCH(dt, return (launch_hyper<T, 1>(HYPER_ARGS)));
#undef HYPER_ARGS
}

// h [T, W] contiguous; wr [NR, W], corr [NR] fp32; the last NR - NE rows are identity experts.
// dense [T, NE + 1]: see corrected_route_kernel.
int hyb_corrected_route(const void* h, const void* wr, const void* corr, void* dense, long T_, int W,
                        int NE, int NR, int top, float scale, int dt, hipStream_t s) {
    if (T_ <= 0) return 0;
    if (NE < 0 || NR < NE || NR < 1 || top < 1 || top > NR || NR > 1536) return 1;
    const bool vec = W % 4 == 0 && ((size_t)h | (size_t)wr) % 16 == 0;
#define ROUTE_VEC(TOK, VEC)                                                                        \
    HYB_DISPATCH(dt, hipLaunchKernelGGL((corrected_route_kernel<T, TOK, VEC>),                      \
                                        dim3((unsigned)((T_ + TOK - 1) / TOK)), dim3(256),         \
                                        (2 * TOK * NR + 32 * TOK) * sizeof(float), s, (const T*)h, \
                                        (const float*)wr, (const float*)corr, (float*)dense, T_, W, \
                                        NE, NR, top, scale))
#define ROUTE(TOK) do { if (vec) ROUTE_VEC(TOK, 4); else ROUTE_VEC(TOK, 1); } while (0)
    if (T_ >= 2048) ROUTE(4); else ROUTE(1);
#undef ROUTE
#undef ROUTE_VEC
    return HYB_LAUNCH_OK();
}

int hyb_gelu_tanh_glu(const void* gu, long gu_stride, void* act, long T_, int C, int dt, hipStream_t s) {
    if (T_ <= 0 || C <= 0) return 0;
    const int esize = dt == 0 ? 2 : 4;
    const bool vec = C % 8 == 0 && gu_stride % 8 == 0 && (size_t)gu % 16 == 0 && (size_t)act % 16 == 0;
    const int cols = C / (vec ? 8 : 1);
    const int th = cols > 128 ? 256 : cols > 64 ? 128 : 64;
    const int parts = (cols + th - 1) / th;
    if (T_ * parts > 0x7fffffffL) return 1;
#define GGLU(VEC)                                                                                  \
    HYB_DISPATCH(dt, hipLaunchKernelGGL((gelu_tanh_glu_kernel<T, VEC>), dim3((unsigned)(T_ * parts)), \
                                        dim3(th), 0, s, (const T*)gu, gu_stride, (T*)act, C, parts))
    if (vec) GGLU(8); else GGLU(1);
#undef GGLU
    return HYB_LAUNCH_OK();
}

}  // extern "C"
