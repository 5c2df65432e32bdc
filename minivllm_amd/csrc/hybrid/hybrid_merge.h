// The last step of attention whose context is split over workgroups: per (row, head) the splits'
// partial results {running maximum, sum, weighted value sum [E]} in a fp32 workspace are folded
// together with the sink term and the optional gate.
#pragma once
#include "hybrid_common.h"

namespace hyb {

// running maximum of a softmax that has seen nothing and has no sink: large, negative and FINITE,
// so that no path forms inf - inf
constexpr float NO_SINK_MAX = -1e30f;

template <typename T>
__global__ void sink_attention_merge_kernel(const float* __restrict__ ws,
                                            const float* __restrict__ sink,
                                            const T* __restrict__ gate, long gate_row,
                                            const int* __restrict__ context_lens,
                                            T* __restrict__ out, int H, int E, int splits) {
    const int b = blockIdx.x / H, h = blockIdx.x % H;
    if (context_lens[b] <= 0) return;
    const int PS = E + 2;
    const float* p = ws + ((long)b * H + h) * splits * PS;
    float M = sink ? sink[h] : NO_SINK_MAX;
    for (int s = 0; s < splits; ++s) M = fmaxf(M, p[s * PS]);
    float L = sink ? expf(sink[h] - M) : 0.f;
    for (int s = 0; s < splits; ++s) L += p[s * PS + 1] * expf(p[s * PS] - M);
    float f = 1.f / L;
    if (gate) f *= sigmoidf_(ld(gate + b * gate_row + h));
    for (int e = threadIdx.x; e < E; e += blockDim.x) {
        float v = 0.f;
        for (int s = 0; s < splits; ++s) v += p[s * PS + 2 + e] * expf(p[s * PS] - M);
        st(out + ((long)b * H + h) * E + e, v * f);
    }
}

}  // namespace hyb
