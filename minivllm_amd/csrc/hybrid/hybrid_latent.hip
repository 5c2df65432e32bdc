// hipcc-flags: -mllvm -amdgpu-mfma-vgpr-form
// (the flag: results of matrix products stay in ordinary vector registers, where the softmax rescales
// them; query fragments go to the accumulation registers, from which products can read directly.  The
// other way round the compiler keeps the accumulators twice.)
// Causal attention over a paged cache of shared latents, on the matrix cores (bfloat16 cache, fp32
// scores, weights and sums).  A cache row is [c | r]: R numbers that are key part AND value, P
// numbers that are key part only; every query head reads the same rows.  Query row of (token, head)
// = [a | b] with a [R] and b [P] in two tensors.  Optional sink term per head, optional window.
//
// With one row set under all heads a (token, head) pair is just a query row: the n tokens of a
// sequence and its H heads form n * H rows against the same keys, in tiles of 32 per wave, so
// prompt portions and single next tokens run the same tile:
//
//   S^T = K Q^T on v_mfma_f32_32x32x16_bf16 (a lane owns one query row and 16 of the tile's 32
//   keys), softmax with a running reference per lane, O^T += V^T P^T on the same instruction.  The
//   weights stay fp32 as far as the product is concerned: each is cut into a high and a low
//   bfloat16 part (17 bits and more together) that are multiplied one after the other.  The score
//   accumulators are the B operand as they stand, and V^T fragments are transposed LDS reads of
//   the very K tile the scores came from: every cache row is fetched once per workgroup.
//
// Workgroup = 4 waves.  RW = 4 (many rows): a wave per 32 rows, one key tile of 32 at a time for all.
// RW = 2 (many rows, value rows too long for a wave's registers): two waves per 32 rows, each with
// half of the value columns; both form the scores.
// RW = 1 (single next tokens of up to a few dozen heads): all waves share 32 rows; waves 0, 1 / 2, 3
// take the left / right half of the value columns, waves 0, 2 / 1, 3 the even / odd key tiles; the
// two halves of the keys meet in LDS at the end, the context may be split over workgroups too (fp32
// partials in a workspace, folded by the merge kernel).  Key tiles are double-buffered in LDS by
// direct global -> LDS loads, requested a stage ahead.
//
// EP: value columns the accumulators hold (R <= EP, a multiple of 32); DP: key columns of the LDS
// image (R + P <= DP, a multiple of 64).  The image is XOR-swizzled in 16-byte chunks so that both
// the row reads (16 rows, one chunk) and the transposed reads (4 rows, 64 bytes) of a wave fall on
// different banks, for row pitches of 256 bytes and of odd multiples of 128.
#include "hybrid_merge.h"
#include <type_traits>

using namespace hyb;

namespace hyb_latent {

typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((ext_vector_type(8))) short s16x8;

constexpr float LOG2E = 1.4426950408889634f;
constexpr float RESCALE = 6.f;      // log2 units: weights stay <= 64 between rescales

struct LatentArgs {
    const uint16_t* qa; long qa_row, qa_head;      // [rows, heads, R]
    const uint16_t* qb; long qb_row, qb_head;      // [rows, heads, P]
    const uint16_t* cache;                         // [blocks * block_size, R + P]
    const int* tables; int max_blocks, block_size;
    const int* cu_q; const int* positions;         // prompt portions; null: row b is sequence b
    const int* lens;                               // then: its keys, the row's own included
    const float* sink;
    uint16_t* out; long out_row, out_head;         // [rows, heads, R]
    float* ws;                                     // splits > 1: [sequence, head, split][R + 2]
    float scale;
    int H, R, P, window, splits;
};

template <int I, int N, class F>
__device__ __forceinline__ void static_for(F&& f) {
    if constexpr (I < N) {
        f(std::integral_constant<int, I>{});
        static_for<I + 1, N>(f);
    }
}

__device__ __forceinline__ uint16_t bf16_bits(float f) {
    return __builtin_bit_cast(uint16_t, (__bf16)f);
}

// what the chunk number of a row is XORed with (see the header comment)
template <int DP>
__device__ __forceinline__ int swizzle(int row) {
    return DP % 128 == 0 ? ((row & 3) << 2) | ((row >> 2) & 3) : (((row >> 1) & 1) << 2) | ((row >> 2) & 3);
}

template <int EP, int DP, int RW>
__global__ void __launch_bounds__(256, EP >= 256 ? 1 : 2)
latent_attention_kernel(LatentArgs a) {
#ifdef __HIP_DEVICE_COMPILE__       // (the host pass only needs the launch stub)
    static_assert(DP % 64 == 0 && EP % 64 == 0 && EP <= DP && (RW == 4 || RW == 2 || RW == 1));
    constexpr int EW = RW == 4 ? 1 : 2;            // waves along the value columns
    constexpr int KW = 4 / RW / EW;                // key tiles per stage (= waves along the keys)
    constexpr int NB = EP / 32 / EW;               // 32-wide value blocks of a wave
    constexpr int KS = DP / 16;                    // 16-wide steps of the score product
    constexpr int CPR = DP / 8;                    // 16-byte chunks of an LDS row
    constexpr int TILE = 32 * DP * 2;              // bytes
    constexpr int IT = CPR / 8;                    // 16-byte pieces per thread and tile
    constexpr int SW = DP % 128 == 0 ? 16 : 8;     // chunks the swizzle permutes
    extern __shared__ __attribute__((aligned(256))) char smem[];

    const int b = blockIdx.x, split = blockIdx.z;
    const int tile_row0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * (32 * RW);     // longest contexts first
    const int H = a.H, D = a.R + a.P;
    int row0, qlen, start;
    if (a.cu_q) {
        row0 = a.cu_q[b];
        qlen = a.cu_q[b + 1] - row0;
        if (tile_row0 >= qlen * H) return;
        start = a.positions[row0];
    } else {
        row0 = b;
        start = a.lens[b] - 1;
        qlen = start >= 0 ? 1 : 0;
        if (tile_row0 >= qlen * H) return;
    }
    const int* table = a.tables + (long)b * a.max_blocks;
    const int tid = threadIdx.x, lane = tid & 63, half = lane >> 5, l32 = lane & 31;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);      // (scalar: so are its branches)
    const int rw = wave % RW, kw = wave / RW % KW, ew = wave / (RW * KW);

    // ---- this lane's query row
    const int wrow0 = tile_row0 + rw * 32;
    const int qi = wrow0 + l32, n_rows = qlen * H;
    const bool qok = qi < n_rows, wave_live = wrow0 < n_rows;
    const int tok = min(qi, n_rows - 1) / H, head = min(qi, n_rows - 1) - tok * H;
    const int qpos = start + tok;
    bf16x8 qf[KS];
    {
        const uint16_t* pa = a.qa + (long)(row0 + tok) * a.qa_row + (long)head * a.qa_head;
        const uint16_t* pb = a.qb + (long)(row0 + tok) * a.qb_row + (long)head * a.qb_head;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const int d = 16 * s + 8 * half;
            uint4 raw = make_uint4(0, 0, 0, 0);                     // columns from D on: zeros
            if (d < a.R) raw = *reinterpret_cast<const uint4*>(pa + d);
            else if (d < D) raw = *reinterpret_cast<const uint4*>(pb + d - a.R);
            qf[s] = __builtin_bit_cast(bf16x8, raw);
        }
    }

    // ---- the keys this workgroup / this wave needs
    const int wg_last = start + min(n_rows - 1, tile_row0 + 32 * RW - 1) / H;
    const int w_first = start + min(wrow0, n_rows - 1) / H, w_last = start + min(wrow0 + 31, n_rows - 1) / H;
    const int n_keys = wg_last + 1;
    const int wg_lo = a.window > 0 ? max(0, start + tile_row0 / H - a.window + 1) : 0;
    int t_begin = wg_lo >> 5, t_end = (n_keys + 31) >> 5;
    if (a.splits > 1) {
        const int per = ((t_end - t_begin + a.splits - 1) / a.splits + KW - 1) / KW * KW;
        t_begin += split * per;
        t_end = min(t_end, t_begin + per);
    }

    // ---- staging: slot c of a tile's image (row c / CPR, chunk c % CPR) receives the cache chunk
    // that the swizzle puts there; chunks behind the row's end repeat chunk 0 (their queries are 0)
    int s_row[IT], s_off[IT];
#pragma unroll
    for (int i = 0; i < IT; ++i) {
        const int c = i * 256 + tid, row = c / CPR;
        int ch = (c - row * CPR) ^ swizzle<DP>(row);
        if (ch * 8 >= D) ch = 0;
        s_row[i] = row;
        s_off[i] = row * D * 2 + ch * 16;
    }
    const bool uniform_rows = (a.block_size & 31) == 0;             // a tile's rows are consecutive
    // block ids of a stage's tiles, through the scalar unit (the table is read-only here) and a stage
    // early: a vector load would be waited for together with everything else in flight
    int ids[KW];
    auto fetch_ids = [&](int t0) {
        typedef const __attribute__((address_space(4))) int* const_int_p;
#pragma unroll
        for (int k = 0; k < KW; ++k)
            ids[k] = *(const_int_p)(uintptr_t)(table + min((t0 + k) * 32, n_keys - 1) / a.block_size);
    };
    auto stage = [&](int t0, int buf) {
#pragma unroll
        for (int k = 0; k < KW; ++k) {
            const int key0 = (t0 + k) * 32;
            if (key0 >= n_keys) continue;
            char* dst = smem + (buf * KW + k) * TILE + wave * 1024;
            if (uniform_rows) {
                const uint16_t* src = a.cache + ((long)ids[k] * a.block_size + key0 % a.block_size) * D;
                // rows behind the context are out of the buffer's range and read as zeros
                const int bytes = min(32, n_keys - key0) * D * 2;
                const __amdgpu_buffer_rsrc_t rsrc = __builtin_amdgcn_make_buffer_rsrc(
                    const_cast<uint16_t*>(src), 0, bytes, 0x00020000);
#pragma unroll
                for (int i = 0; i < IT; ++i)
                    __builtin_amdgcn_raw_ptr_buffer_load_lds(
                        rsrc, (__attribute__((address_space(3))) void*)(dst + i * 4096), 16, s_off[i], 0, 0, 0);
            } else {
#pragma unroll
                for (int i = 0; i < IT; ++i) {
                    const int key = min(key0 + s_row[i], n_keys - 1);
                    const long row = (long)table[key / a.block_size] * a.block_size + key % a.block_size;
                    const char* src = reinterpret_cast<const char*>(a.cache) + row * D * 2 + (s_off[i] - s_row[i] * D * 2);
                    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src,
                                                     (__attribute__((address_space(3))) void*)(dst + i * 4096), 16, 0, 0);
                }
            }
        }
    };

    // ---- LDS addresses of this wave's fragments inside a buffer (one tile at kw)
    const uint32_t lds0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) const char*)smem + kw * TILE;
    uint32_t k_addr[SW / 2];                        // row l32, chunk 2 s + half: distinct for s < SW / 2
#pragma unroll
    for (int s = 0; s < SW / 2; ++s) k_addr[s] = lds0 + l32 * (DP * 2) + (((2 * s + half) ^ swizzle<DP>(l32)) << 4);
    // transposed reads: 16 lanes take 4 key rows x 16 columns and return 4 keys of one column each
    constexpr int NA = NB < SW / 4 ? NB : SW / 4;   // value blocks with addresses of their own
    const int i16 = lane & 15, tr_row = 4 * half + (i16 >> 2);
    const int tr_chunk = 2 * ((lane >> 4) & 1) + ((i16 & 3) >> 1);
    uint32_t v_addr[NA][2];
#pragma unroll
    for (int n = 0; n < NA; ++n)
#pragma unroll
        for (int hi = 0; hi < 2; ++hi) {
            const int row = tr_row + 8 * hi, ch = 4 * (ew * NB + n) + tr_chunk;
            v_addr[n][hi] = lds0 + row * (DP * 2) + ((ch ^ swizzle<DP>(row)) << 4) + (i16 & 1) * 8;
        }

    f32x16 acc[NB];
#pragma unroll
    for (int n = 0; n < NB; ++n)
#pragma unroll
        for (int e = 0; e < 16; ++e) acc[n][e] = 0.f;
    float m_run = NO_SINK_MAX, l_run = 0.f;         // in log2 units of the scaled scores
    const float sc = a.scale * LOG2E;

    if (t_begin < t_end) {
        fetch_ids(t_begin);
        stage(t_begin, 0);
        if (t_begin + KW < t_end) fetch_ids(t_begin + KW);
    }
    __syncthreads();
    for (int t = t_begin, buf = 0; t < t_end; t += KW, buf ^= 1) {
        const int key0 = (t + kw) * 32;
        const bool live = wave_live && t + kw < t_end && key0 <= w_last &&
                          (a.window <= 0 || key0 + 31 > w_first - a.window);       // (uniform per wave)
        bf16x8 p_hi[2], p_lo[2];
        if (t + KW < t_end) {                           // lands behind this tile's products
            stage(t + KW, buf ^ 1);
            if (t + 2 * KW < t_end) fetch_ids(t + 2 * KW);
        }
        if (live) {
            f32x16 s_acc;
#pragma unroll
            for (int e = 0; e < 16; ++e) s_acc[e] = 0.f;
            // (inline asm as for the value reads below: KA row reads in flight, no more registers)
            constexpr int KA = 4;
            uint32_t ka[SW / 2];
#pragma unroll
            for (int s = 0; s < SW / 2; ++s) ka[s] = k_addr[s] + buf * (KW * TILE);
            s16x8 kf[KS];
            auto read_k = [&](auto ic) {
                constexpr int i = decltype(ic)::value;
                constexpr int off = (i / (SW / 2)) * (SW * 16);
                const uint32_t a0 = ka[i % (SW / 2)];
                s16x8 x;
                asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(x) : "v"(a0), "n"(off));
                kf[i] = x;
            };
            static_for<0, KA>(read_k);
            static_for<0, KS>([&](auto ic) {
                constexpr int i = decltype(ic)::value;
                if constexpr (i + KA < KS) read_k(std::integral_constant<int, i + KA>{});
                constexpr int left = KS - 1 - i < KA ? KS - 1 - i : KA;      // reads still in flight
                s16x8 x = kf[i];
                if constexpr (left == 4) asm volatile("s_waitcnt lgkmcnt(4)" : "+v"(x));
                else if constexpr (left == 3) asm volatile("s_waitcnt lgkmcnt(3)" : "+v"(x));
                else if constexpr (left == 2) asm volatile("s_waitcnt lgkmcnt(2)" : "+v"(x));
                else if constexpr (left == 1) asm volatile("s_waitcnt lgkmcnt(1)" : "+v"(x));
                else asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(x));
                s_acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, x), qf[i], s_acc, 0, 0, 0);
                __builtin_amdgcn_sched_barrier(0);    // (products sunk below later reads cost registers)
            });
            // lane: query row l32, keys key0 + (e & 3) + 8 (e >> 2) + 4 half
            const bool all_seen = key0 + 31 <= w_first && (a.window <= 0 || w_last - key0 < a.window);
            const int oldest = a.window > 0 ? qpos - a.window : -1;
            if (!all_seen) {                             // (one uniform branch, not one per score)
#pragma unroll
                for (int e = 0; e < 16; ++e) {
                    const int key = key0 + (e & 3) + 8 * (e >> 2) + 4 * half;
                    s_acc[e] = ((key > qpos) | (key <= oldest)) ? -INFINITY : s_acc[e] * sc;
                }
            } else {
#pragma unroll
                for (int e = 0; e < 16; ++e) s_acc[e] *= sc;
            }
            float mt = -INFINITY;
#pragma unroll
            for (int e = 0; e < 16; ++e) mt = fmaxf(mt, s_acc[e]);
            mt = fmaxf(mt, __shfl_xor(mt, 32, kWave));
            // the reference of the exponentials only moves when some row outgrows it by RESCALE
            if (!__all(mt - m_run <= RESCALE)) {
                const float m_new = fmaxf(m_run, mt);
                const float f = __builtin_amdgcn_exp2f(m_run - m_new);
                l_run *= f;
#pragma unroll
                for (int n = 0; n < NB; ++n) acc[n] *= f;
                m_run = m_new;
            }
#pragma unroll
            for (int s = 0; s < 2; ++s) {
                s16x8 hi, lo;
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const float p = __builtin_amdgcn_exp2f(s_acc[8 * s + j] - m_run);
                    l_run += p;
                    const uint16_t h = bf16_bits(p);
                    hi[j] = (short)h;
                    lo[j] = (short)bf16_bits(p - __uint_as_float((uint32_t)h << 16));
                }
                p_hi[s] = __builtin_bit_cast(bf16x8, hi);
                p_lo[s] = __builtin_bit_cast(bf16x8, lo);
            }
        }
        if (live) {
            // transposed reads as inline asm: through the builtin the compiler would wait for the
            // stage's loads in flight ahead of the first one.  Step i (value block i / 2, keys 16
            // (i & 1) ..) is requested AHEAD steps early; LDS returns in order.
            constexpr int STEPS = 2 * NB, AHEAD = STEPS < 4 ? STEPS : 4;
            s16x4 lo4[STEPS], hi4[STEPS];
            uint32_t va[NA][2];
#pragma unroll
            for (int n = 0; n < NA; ++n) {
                va[n][0] = v_addr[n][0] + buf * (KW * TILE);
                va[n][1] = v_addr[n][1] + buf * (KW * TILE);
            }
            auto read = [&](auto ic) {
                constexpr int i = decltype(ic)::value, n = i >> 1, s = i & 1;
                constexpr int off = (n / NA) * NA * 64 + s * 16 * DP * 2;
                const uint32_t a0 = va[n % NA][0], a1 = va[n % NA][1];
                s16x4 x, y;
                asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(x) : "v"(a0), "n"(off));
                asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(y) : "v"(a1), "n"(off));
                lo4[i] = x;
                hi4[i] = y;
            };
            static_for<0, AHEAD>(read);
            static_for<0, STEPS>([&](auto ic) {
                constexpr int i = decltype(ic)::value, n = i >> 1, s = i & 1;
                if constexpr (i + AHEAD < STEPS) read(std::integral_constant<int, i + AHEAD>{});
                constexpr int left = STEPS - 1 - i < AHEAD ? STEPS - 1 - i : AHEAD;   // steps still in flight
                s16x4 x = lo4[i], y = hi4[i];
                if constexpr (left >= 4) asm volatile("s_waitcnt lgkmcnt(8)" : "+v"(x), "+v"(y));
                else if constexpr (left == 3) asm volatile("s_waitcnt lgkmcnt(6)" : "+v"(x), "+v"(y));
                else if constexpr (left == 2) asm volatile("s_waitcnt lgkmcnt(4)" : "+v"(x), "+v"(y));
                else if constexpr (left == 1) asm volatile("s_waitcnt lgkmcnt(2)" : "+v"(x), "+v"(y));
                else asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(x), "+v"(y));
                const s16x8 v = {x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]};
                const bf16x8 vf = __builtin_bit_cast(bf16x8, v);
                acc[n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, p_hi[s], acc[n], 0, 0, 0);
                acc[n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, p_lo[s], acc[n], 0, 0, 0);
                __builtin_amdgcn_sched_barrier(0);
            });
        }
        __syncthreads();
    }
    l_run += __shfl_xor(l_run, 32, kWave);

    if constexpr (KW == 2) {                         // odd key tiles' part -> LDS -> even's
        float* o = reinterpret_cast<float*>(smem) + ew * (NB * 16 + 2) * 64 + lane;
        if (kw == 1) {
#pragma unroll
            for (int n = 0; n < NB; ++n)
#pragma unroll
                for (int e = 0; e < 16; ++e) o[(n * 16 + e) * 64] = acc[n][e];
            o[NB * 16 * 64] = m_run;
            o[(NB * 16 + 1) * 64] = l_run;
        }
        __syncthreads();
        if (kw == 1) return;
        const float m2 = o[NB * 16 * 64], l2 = o[(NB * 16 + 1) * 64];
        const float m_new = fmaxf(m_run, m2);
        const float f1 = __builtin_amdgcn_exp2f(m_run - m_new), f2 = __builtin_amdgcn_exp2f(m2 - m_new);
        l_run = l_run * f1 + l2 * f2;
        m_run = m_new;
#pragma unroll
        for (int n = 0; n < NB; ++n)
#pragma unroll
            for (int e = 0; e < 16; ++e) acc[n][e] = acc[n][e] * f1 + o[(n * 16 + e) * 64] * f2;
    }
    const int e0 = ew * NB * 32;
    if (a.splits > 1) {
        if (!qok) return;
        float* w = a.ws + (((long)(row0 + tok) * H + head) * a.splits + split) * (a.R + 2);
        if (ew == 0 && half == 0) { w[0] = m_run / LOG2E; w[1] = l_run; }
#pragma unroll
        for (int n = 0; n < NB; ++n)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int e = e0 + 32 * n + 8 * r + 4 * half;
                if (e < a.R) {
                    float2* d = reinterpret_cast<float2*>(w + 2 + e);
                    d[0] = make_float2(acc[n][4 * r], acc[n][4 * r + 1]);
                    d[1] = make_float2(acc[n][4 * r + 2], acc[n][4 * r + 3]);
                }
            }
        return;
    }
    float f;
    if (a.sink) {
        const float sk = a.sink[head] * LOG2E, M = fmaxf(m_run, sk);
        f = __builtin_amdgcn_exp2f(m_run - M);
        f = f / (l_run * f + __builtin_amdgcn_exp2f(sk - M));
    } else {
        f = 1.f / l_run;
    }
    // both halves of the wave hold every second run of four columns of a row: swapped so that a
    // lane stores eight neighbouring ones
    uint16_t* op = a.out + (long)(row0 + tok) * a.out_row + (long)head * a.out_head + e0;
#pragma unroll
    for (int n = 0; n < NB; ++n)
#pragma unroll
        for (int r = 0; r < 4; r += 2) {
            uint32_t w[4];
#pragma unroll
            for (int k = 0; k < 4; ++k)
                w[k] = (uint32_t)bf16_bits(acc[n][4 * r + 2 * k] * f) |
                       ((uint32_t)bf16_bits(acc[n][4 * r + 2 * k + 1] * f) << 16);
            const uint32_t s0 = half ? w[0] : w[2], s1 = half ? w[1] : w[3];
            const uint32_t g0 = __shfl_xor(s0, 32, kWave), g1 = __shfl_xor(s1, 32, kWave);
            const uint4 v = half ? make_uint4(g0, g1, w[2], w[3]) : make_uint4(w[0], w[1], g0, g1);
            const int e = 32 * n + 8 * r + 8 * half;
            if (qok && e0 + e < a.R) *reinterpret_cast<uint4*>(op + e) = v;
        }
#endif
}

template <int EP, int DP>
int launch(const LatentArgs& a, int nseq, int max_rows, bool wide, hipStream_t s) {
    constexpr int tile = 32 * DP * 2;
#define LATENT(RW)                                                                                 \
    do {                                                                                           \
        constexpr int lds = 2 * (RW == 1 ? 2 : 1) * tile;                                          \
        static_assert(lds <= 160 * 1024 && (RW > 1 || (EP / 2 + 4) * 256 <= lds));                  \
        if (lds > 64 * 1024) {                                                                     \
            static const hipError_t once = hipFuncSetAttribute(                                    \
                (const void*)latent_attention_kernel<EP, DP, RW>,                                  \
                hipFuncAttributeMaxDynamicSharedMemorySize, lds);                                  \
            if (once != hipSuccess) return 2;                                                      \
        }                                                                                          \
        const dim3 grid(nseq, (max_rows + 32 * RW - 1) / (32 * RW), a.splits);                     \
        hipLaunchKernelGGL((latent_attention_kernel<EP, DP, RW>), grid, dim3(256), lds, s, a);      \
    } while (0)
    if (!wide) LATENT(1); else if constexpr (EP > 256) LATENT(2); else LATENT(4);
#undef LATENT
    return HYB_LAUNCH_OK();
}

int dispatch(const LatentArgs& a, int nseq, int max_rows, bool wide, hipStream_t s) {
    const int R = a.R, D = a.R + a.P;
#define PICK(EP, DP) if (R <= EP && D <= DP) return launch<EP, DP>(a, nseq, max_rows, wide, s)
    PICK(64, 128);
    PICK(128, 128);
    PICK(128, 192);
    PICK(128, 256);
    PICK(256, 320);
    PICK(256, 384);
    PICK(512, 576);
    PICK(512, 640);
#undef PICK
    return 1;
}

}  // namespace hyb_latent

using namespace hyb_latent;

extern "C" {

// 1 when there is an instance for latents of R numbers and key parts of P more
int hyb_latent_attention_ok(int R, int P) {
    if (R < 8 || P < 0 || R % 8 || P % 8) return 0;
    const int D = R + P;
    return (R <= 128 && D <= 256) || (R <= 256 && D <= 384) || (R <= 512 && D <= 640);
}

// Prompt portions (cu_q / positions given: sequence b owns rows cu_q[b] .. cu_q[b + 1], max_q: the
// longest portion) or single next tokens (cu_q null: row b is sequence b with lens[b] keys).
// splits > 1 (single tokens only): ws holds nseq * H * splits * (R + 2) floats.
int hyb_latent_attention(const void* qa, long qa_row, long qa_head, const void* qb, long qb_row,
                         long qb_head, const void* cache, const void* tables, int max_blocks,
                         int block_size, const void* cu_q, const void* positions, const void* lens,
                         const void* sink, void* out, long out_row, long out_head, void* ws,
                         float scale, int nseq, int max_q, int H, int R, int P, int window,
                         int splits, hipStream_t s) {
    if (nseq <= 0 || max_q <= 0) return 0;
    if (!hyb_latent_attention_ok(R, P) || H <= 0 || block_size <= 0 || splits < 1) return 1;
    if (cu_q ? (!positions || splits != 1) : (!lens || max_q != 1)) return 1;
    if (splits > 1 && !ws) return 1;
    if (((size_t)qa | (size_t)qb | (size_t)cache | (size_t)out) % 16) return 1;
    if (qa_row % 8 || qa_head % 8 || qb_row % 8 || qb_head % 8 || out_row % 8 || out_head % 8) return 1;
    if ((long)max_q * H > 0x3fffffffL) return 1;
    LatentArgs a{(const uint16_t*)qa, qa_row, qa_head, (const uint16_t*)qb, qb_row, qb_head,
                 (const uint16_t*)cache, (const int*)tables, max_blocks, block_size,
                 (const int*)cu_q, (const int*)positions, (const int*)lens, (const float*)sink,
                 (uint16_t*)out, out_row, out_head, (float*)ws, scale, H, R, P, window, splits};
    const int rc = dispatch(a, nseq, max_q * H, max_q * H > 64, s);
    if (rc || splits == 1) return rc;
    hipLaunchKernelGGL(sink_attention_merge_kernel<bf16_t>, dim3(nseq * H), dim3(R >= 128 ? 128 : 64), 0, s,
                       (const float*)ws, (const float*)sink, (const bf16_t*)nullptr, 0L,
                       (const int*)lens, (bf16_t*)out, H, R, splits);
    return HYB_LAUNCH_OK();
}

}  // extern "C"
