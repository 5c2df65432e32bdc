// What a causal filter over time keeps of a sequence from step to step: its last taps - 1 inputs in
// tail [slots, taps - 1, C] fp32, the newest last.
#pragma once
#include "hybrid_common.h"

namespace hyb {

// The kept inputs after the step: grid (channel chunks, sequences); runs after every row has read.
// skip_single: sequences of one row are passed over (the kernel ahead has kept their input itself).
template <typename T>
__global__ void short_conv_tail_kernel(const T* __restrict__ x, long x_stride, float* __restrict__ tail,
                                       const int* __restrict__ cu_q, const int* __restrict__ positions,
                                       const int* __restrict__ slots, int C, int taps,
                                       int skip_single) {
    const int b = blockIdx.y;
    const int c = blockIdx.x * blockDim.x + threadIdx.x;
    if (c >= C) return;
    const int slot = slots[b];
    if (slot < 0) return;
    const long s0 = cu_q ? cu_q[b] : b, e0 = cu_q ? cu_q[b + 1] : b + 1;
    const int n = (int)(e0 - s0);
    if (n <= 0 || (skip_single && n == 1)) return;
    const int p0 = positions[s0], keep = taps - 1;
    float* tl = tail + (long)slot * keep * C + c;
    for (int i = 0; i < keep; ++i) {                  // ascending: reads never trail the writes
        const int off = n - keep + i;                 // row offset inside the step
        float v;
        if (off >= 0) v = ld(x + (s0 + off) * x_stride + c);
        else v = (p0 + off >= 0) ? tl[(long)(i + n) * C] : 0.f;
        tl[(long)i * C] = v;
    }
}

}  // namespace hyb
