// vec_input.h -- how a decode workgroup stages its input vector in LDS (device), and the expert choice.
#pragma once
#include "bf16_util.h"
#include "device_util.h"
#include "linear.h"

namespace mg {

// Element i of a staged vector of nc8 chunks of 8: two planes of float4, so that neighbouring lanes (which own
// neighbouring chunks) read 16 bytes apart.
__device__ __forceinline__ int plane_index(int i, int nc8) { return ((((i >> 2) & 1) * nc8 + (i >> 3)) << 2) + (i & 3); }

// Stages in.src (transformed as VecInput says) as Kp floats, zero past in.n; ends with a barrier.  store: this
// workgroup writes normOut / out.
__device__ __forceinline__ void stage_vector(const VecInput& in, float* act, int Kp, bool store, float* red) {
    const int nc8 = Kp >> 3;
    const int n = in.n;
    float ss = 0.f;
    for (int i = threadIdx.x; i < Kp; i += WG) {
        const float v = i < n ? in.src[i] : 0.f;
        act[plane_index(i, nc8)] = v;
        ss = fmaf(v, v, ss);
    }
    if (in.gain) {
        const float rs = 1.0f / sqrtf(block_sum(ss, red) / (float)n + in.eps);
        float ss2 = 0.f;
        for (int i = threadIdx.x; i < n; i += WG) {
            float v = act[plane_index(i, nc8)] * rs * in.gain[i];
            if (store && in.normOut) in.normOut[i] = v;
            if (in.part) v = fmaf(in.coef, v, in.part[i]);
            if (store && in.out) in.out[i] = v;
            act[plane_index(i, nc8)] = v;
            ss2 = fmaf(v, v, ss2);
        }
        if (in.gain2) {
            const float r2 = 1.0f / sqrtf(block_sum(ss2, red) / (float)n + in.eps);
            for (int i = threadIdx.x; i < n; i += WG) act[plane_index(i, nc8)] *= r2 * in.gain2[i];
        }
    }
    __syncthreads();
}

constexpr int MAX_EXPERTS = 512;
constexpr int MAX_TOP = 32;

// The `top` largest of E logits (the lower index on ties) and their softmax over all E, by one full wave.
// ids / w: LDS or global, written by lane 0.
__device__ __forceinline__ void choose_experts(const float* z, int E, int top, int* ids, float* w) {
    const int lane = threadIdx.x & 63;
    float v[MAX_EXPERTS / 64];
    float m = -INFINITY;
#pragma unroll
    for (int k = 0; k < MAX_EXPERTS / 64; k++) {
        const int e = k * 64 + lane;
        v[k] = e < E ? z[e] : -INFINITY;
        m = fmaxf(m, v[k]);
    }
    m = wave_max(m);
    float sum = 0.f;
#pragma unroll
    for (int k = 0; k < MAX_EXPERTS / 64; k++) sum += expf(v[k] - m);
    sum = wave_sum(sum);
    for (int s = 0; s < top; s++) {
        float bv = -INFINITY;
        int bi = INT_MAX;
#pragma unroll
        for (int k = 0; k < MAX_EXPERTS / 64; k++)
            if (v[k] > bv) { bv = v[k]; bi = k * 64 + lane; }
        wave_argmax(bv, bi);
        if (bi >= E) bi = 0;                      // (only with non-finite logits)
#pragma unroll
        for (int k = 0; k < MAX_EXPERTS / 64; k++)
            if (bi == k * 64 + lane) v[k] = -INFINITY;
        if (lane == 0) { ids[s] = bi; w[s] = expf(bv - m) / sum; }
    }
}

}  // namespace mg
