// side_jobs.h -- device code of the decode step's side jobs (row_ops.h).
#pragma once
#include "bf16_util.h"
#include "device_util.h"
#include "row_ops.h"

namespace mg {

// Element d of the rotated part at a position: pairs (2i, 2i+1) below ropeDims turned, the rest as they are.
__device__ __forceinline__ float rotated_element(const float* v, int d, int ropeDims, const float* c, const float* s) {
    if (d >= ropeDims) return v[d];
    const float u = v[d & ~1], w = v[d | 1];
    return (d & 1) ? w * c[d >> 1] + u * s[d >> 1] : u * c[d >> 1] - w * s[d >> 1];
}

// One cache row from the raw projection, by a whole workgroup of WG threads.
template <typename CT>
__device__ __forceinline__ void write_latent_row(const LatentCache& c, const float* z, const float* gain, float eps, int pos, float* red) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < c.rank; i += WG) ss = fmaf(z[i], z[i], ss);
    const float rs = 1.0f / sqrtf(block_sum(ss, red) / (float)c.rank + eps);
    CT* row = static_cast<CT*>(c.rows) + (size_t)pos * c.stride;
    for (int i = threadIdx.x; i < c.rank; i += WG) store_act(row + i, z[i] * rs * gain[i]);
    const size_t t = (size_t)pos * (c.ropeDims >> 1);
    for (int d = threadIdx.x; d < c.rot; d += WG)
        store_act(row + c.rankPad + d, rotated_element(z + c.rank, d, c.ropeDims, c.cosTab + t, c.sinTab + t));
}

__device__ __forceinline__ void run_side_job(const SideJobs& j, int wg, float* red) {
    if (j.z) {
        if (wg == 0) {
            if (j.cache.f32) write_latent_row<float>(j.cache, j.z, j.gain, j.eps, j.state->pos, red);
            else write_latent_row<bf16_t>(j.cache, j.z, j.gain, j.eps, j.state->pos, red);
            return;
        }
        wg--;
    }
    const int i = wg * WG + threadIdx.x;
    if (i >= j.n) return;
    float v = j.coef[0] * j.first[i];
    for (int t = 1; t < j.terms; t++) v = fmaf(j.coef[t], j.hist[(size_t)(t - 1) * j.histStride + i], v);
    j.part[i] = v;
}

}  // namespace mg
