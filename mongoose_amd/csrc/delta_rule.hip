// delta_rule.hip -- the generalized delta rule (delta_rule.h), everything in fp32.
#include "delta_rule.h"
#include "activations.h"
#include "bf16_util.h"
#include "device_util.h"
#include "side_jobs.h"

namespace mg {

constexpr float LOG_DECAY = -0.60653065971263342f;      // -exp(-1/2)
constexpr float UNIT_EPS = 1e-6f;

// ---------------------------------------------------------------------------
// decode: one workgroup a head; thread = (value column, group of key channels)
// ---------------------------------------------------------------------------
__global__ __launch_bounds__(WG) void delta_step_kernel(DeltaStep p) {
    extern __shared__ float sh[];
    __shared__ float red[4];
    const int H = p.d.heads, D = p.d.dim, h = blockIdx.x;
    if (h >= H) { run_side_job(p.side, h - H, red); return; }
    const int HD = H * D;
    float* th = sh;                       // tanh(W1 h) [rank]
    float* r = th + pad_to(p.d.rank, 64);
    float* k = r + D;
    float* u = k + D;
    float* w = u + D;
    float* au = w + D;
    float* part = au + D;                 // [groups][D]
    const float* z = p.z;
    const bool fresh = p.state->pos == 0;
    for (int i = threadIdx.x; i < p.d.rank; i += WG) th[i] = tanhf(z[(size_t)5 * HD + i]);
    float kk = 0.f;
    for (int i = threadIdx.x; i < D; i += WG) {
        r[i] = z[h * D + i];
        const float x = z[HD + h * D + i];
        k[i] = x;
        kk = fmaf(x, x, kk);
    }
    const float inv = 1.0f / sqrtf(block_sum(kk, red) + UNIT_EPS);       // (its barriers also publish th, r, k)
    for (int i = threadIdx.x; i < D; i += WG) {
        const int c = h * D + i;
        const unsigned short* w2 = p.d.w2.w + (size_t)c * p.d.w2.ld;
        float e = p.d.w0[c];
        for (int j = 0; j < p.d.rank; j++) e = fmaf(bf16_to_f32(w2[j]), th[j], e);
        w[i] = expf(LOG_DECAY * sigmoid_f(e));
        u[i] = k[i] * inv;
        au[i] = sigmoid_f(z[(size_t)4 * HD + c] + p.d.aBias[c]) * u[i];
    }
    __syncthreads();
    const int cols = D < WG ? D : WG, groups = WG / cols;     // threads past groups * cols idle
    const int g = threadIdx.x / cols, j0 = threadIdx.x % cols;
    const bool on = g < groups;
    const int per = (D + groups - 1) / groups, i0 = g * per, i1 = min(i0 + per, D);
    float* S = p.S + (size_t)h * D * D;
    float ss = 0.f;
    for (int jb = 0; jb < D; jb += cols) {                    // (one pass up to 256 columns)
        const int j = jb + j0;
        const bool in = on && j < D;
        float dot = 0.f;
        if (in && !fresh)
            for (int i = i0; i < i1; i++) dot = fmaf(u[i], S[(size_t)i * D + j], dot);
        if (in) part[g * cols + j0] = dot;
        __syncthreads();
        float d = 0.f;
        if (in) for (int q = 0; q < groups; q++) d += part[q * cols + j0];
        __syncthreads();
        float o = 0.f;
        if (in) {
            const float v = z[2 * HD + h * D + j];
            for (int i = i0; i < i1; i++) {
                const float old = fresh ? 0.f : S[(size_t)i * D + j];
                const float s = fmaf(k[i], v, fmaf(w[i], old, -au[i] * d));
                S[(size_t)i * D + j] = s;
                o = fmaf(r[i], s, o);
            }
            part[g * cols + j0] = o;
        }
        __syncthreads();
        if (in && g == 0) {
            o = 0.f;
            for (int q = 0; q < groups; q++) o += part[q * cols + j0];
            p.y[h * D + j] = o;
            ss = fmaf(o, o, ss);
        }
        __syncthreads();
    }
    const float rs = 1.0f / sqrtf(block_sum(ss, red) / (float)D + p.d.eps);
    if (g == 0)
        for (int j = j0; j < D; j += cols) {                  // (each thread rewrites what it wrote)
            const int c = h * D + j;
            p.y[c] = p.y[c] * rs * p.d.norm[c] * sigmoid_f(z[3 * HD + c]);
        }
}
hipError_t launch_delta_step(const DeltaStep& p, hipStream_t s) {
    const int D = p.d.dim;
    if (!delta_supported(D) || p.d.heads < 1 || p.d.rank < 1 || p.d.w2.ld < p.d.rank) return hipErrorInvalidValue;
    const size_t lds = ((size_t)pad_to(p.d.rank, 64) + 5 * (size_t)D + WG) * 4;
    if (lds > (60u << 10)) return hipErrorInvalidValue;
    hipLaunchKernelGGL(delta_step_kernel, dim3(p.d.heads + p.side.wgs()), dim3(WG), lds, s, p);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------
// many rows
// ---------------------------------------------------------------------------
__global__ void delta_tanh_kernel(DeltaRows p, int ldw) {
    const int t = blockIdx.x;
    const float* z = p.z + (size_t)t * p.ldz + (size_t)5 * p.d.heads * p.d.dim;
    for (int i = threadIdx.x; i < ldw; i += blockDim.x) p.w1[(size_t)t * ldw + i] = i < p.d.rank ? tanhf(z[i]) : 0.f;
}

// decay, unit key and removal of one (row, head); one wave
__global__ __launch_bounds__(64) void delta_gates_kernel(DeltaRows p) {
    const int h = blockIdx.x, t = blockIdx.y, D = p.d.dim, HD = p.d.heads * D;
    const float* z = p.z + (size_t)t * p.ldz;
    float kk = 0.f;
    for (int i = threadIdx.x; i < D; i += 64) { const float x = z[HD + h * D + i]; kk = fmaf(x, x, kk); }
    const float inv = 1.0f / sqrtf(wave_sum(kk) + UNIT_EPS);
    for (int i = threadIdx.x; i < D; i += 64) {
        const int c = h * D + i;
        const size_t o = (size_t)t * HD + c;
        const float un = z[HD + c] * inv;
        p.u[o] = un;
        p.au[o] = sigmoid_f(z[(size_t)4 * HD + c] + p.d.aBias[c]) * un;
        p.dec[o] = expf(LOG_DECAY * sigmoid_f(p.dec[o] + p.d.w0[c]));
    }
}

// The recurrence itself.  The value columns of a state do not touch each other: 16 lanes (one DPP row) own a column,
// CPL key channels each; a workgroup 16 columns of one head.  Tokens go through LDS in chunks of TC.
template <int CPL>
__global__ __launch_bounds__(WG) void delta_scan_kernel(DeltaRows p) {
    constexpr int DP = 16 * CPL, TC = CPL >= 16 ? 8 : 16;
    __shared__ __attribute__((aligned(16))) float vec[5][TC][DP];       // decay, a u, u, k, r (zero past dim)
    __shared__ float vv[TC][16], oo[TC][16];
    const int h = blockIdx.x, D = p.d.dim, HD = p.d.heads * D;
    const int lane = threadIdx.x & 63, sub = lane & 15, col = (threadIdx.x >> 4);
    const int j = blockIdx.y * 16 + col;
    const bool in = j < D;
    float S[CPL];
    float* Sg = p.S + (size_t)h * D * D;
#pragma unroll
    for (int c = 0; c < CPL; c++) {
        const int i = sub * CPL + c;
        S[c] = in && i < D && p.pos0 > 0 ? Sg[(size_t)i * D + j] : 0.f;
    }
    for (int t0 = 0; t0 < p.T; t0 += TC) {
        const int n = min(TC, p.T - t0);
        __syncthreads();
        for (int x = threadIdx.x; x < n * DP; x += WG) {
            const int t = x / DP, i = x % DP;
            const bool ok = i < D;
            const size_t a = (size_t)(t0 + t) * HD + h * D + i, zb = (size_t)(t0 + t) * p.ldz + h * D + i;
            vec[0][t][i] = ok ? p.dec[a] : 0.f;
            vec[1][t][i] = ok ? p.au[a] : 0.f;
            vec[2][t][i] = ok ? p.u[a] : 0.f;
            vec[3][t][i] = ok ? p.z[zb + HD] : 0.f;
            vec[4][t][i] = ok ? p.z[zb] : 0.f;
        }
        for (int x = threadIdx.x; x < n * 16; x += WG) {
            const int t = x >> 4, c = blockIdx.y * 16 + (x & 15);
            vv[t][x & 15] = c < D ? p.z[(size_t)(t0 + t) * p.ldz + 2 * HD + h * D + c] : 0.f;
        }
        __syncthreads();
        for (int t = 0; t < n; t++) {
            float dot = 0.f;
#pragma unroll
            for (int c = 0; c < CPL; c++) dot = fmaf(vec[2][t][sub * CPL + c], S[c], dot);
            dot = row_sum16(dot);
            const float v = vv[t][col];
            float o = 0.f;
#pragma unroll
            for (int c = 0; c < CPL; c++) {
                const int i = sub * CPL + c;
                S[c] = fmaf(vec[3][t][i], v, fmaf(vec[0][t][i], S[c], -vec[1][t][i] * dot));
                o = fmaf(vec[4][t][i], S[c], o);
            }
            o = row_sum16(o);
            if (sub == 0) oo[t][col] = o;
        }
        __syncthreads();
        for (int x = threadIdx.x; x < n * 16; x += WG) {
            const int t = x >> 4, c = blockIdx.y * 16 + (x & 15);
            if (c < D) p.o[(size_t)(t0 + t) * HD + h * D + c] = oo[t][x & 15];
        }
    }
    if (in)
#pragma unroll
        for (int c = 0; c < CPL; c++) {
            const int i = sub * CPL + c;
            if (i < D) Sg[(size_t)i * D + j] = S[c];
        }
}

template <typename AT>
__global__ __launch_bounds__(64) void delta_output_kernel(DeltaRows p) {
    const int h = blockIdx.x, t = blockIdx.y, D = p.d.dim, HD = p.d.heads * D;
    const float* o = p.o + (size_t)t * HD + h * D;
    float ss = 0.f;
    for (int i = threadIdx.x; i < D; i += 64) ss = fmaf(o[i], o[i], ss);
    const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)D + p.d.eps);
    for (int i = threadIdx.x; i < D; i += 64) {
        const int c = h * D + i;
        store_act(static_cast<AT*>(p.yAct) + (size_t)t * p.ldAct + c, o[i] * rs * p.d.norm[c] * sigmoid_f(p.z[(size_t)t * p.ldz + 3 * HD + c]));
    }
}

bool delta_supported(int dim) { return dim >= 1 && dim <= 256; }

hipError_t launch_delta_rows(const DeltaRows& p, hipStream_t s) {
    if (p.T <= 0) return hipSuccess;
    const int D = p.d.dim, H = p.d.heads, ldw = p.d.w2.ld;
    if (!delta_supported(D) || p.T > 65535 || p.d.rank > ldw || ldw % 64) return hipErrorInvalidValue;
    hipLaunchKernelGGL(delta_tanh_kernel, dim3(p.T), dim3(64), 0, s, p, ldw);
    Gemm g;
    g.A = p.w1; g.f32 = 1; g.lda = ldw; g.M = p.T;
    g.W = p.d.w2.w; g.ldw = ldw; g.N = H * D; g.K = ldw;
    g.mode = GEMM_F32; g.out = p.dec; g.ldc = H * D;
    hipError_t e = launch_gemm_bf16w(g, s);
    if (e != hipSuccess) return e;
    hipLaunchKernelGGL(delta_gates_kernel, dim3(H, p.T), dim3(64), 0, s, p);
    const dim3 grid(H, (D + 15) / 16);
    const int cpl = (D + 15) / 16;
    if (cpl <= 1) hipLaunchKernelGGL(delta_scan_kernel<1>, grid, dim3(WG), 0, s, p);
    else if (cpl <= 2) hipLaunchKernelGGL(delta_scan_kernel<2>, grid, dim3(WG), 0, s, p);
    else if (cpl <= 4) hipLaunchKernelGGL(delta_scan_kernel<4>, grid, dim3(WG), 0, s, p);
    else if (cpl <= 8) hipLaunchKernelGGL(delta_scan_kernel<8>, grid, dim3(WG), 0, s, p);
    else hipLaunchKernelGGL(delta_scan_kernel<16>, grid, dim3(WG), 0, s, p);
    if (p.actF32) hipLaunchKernelGGL(delta_output_kernel<float>, dim3(H, p.T), dim3(64), 0, s, p);
    else hipLaunchKernelGGL(delta_output_kernel<bf16_t>, dim3(H, p.T), dim3(64), 0, s, p);
    return hipGetLastError();
}

}  // namespace mg
