// latent_attn.h -- attention over a cache of latents shared by all heads (latent_attn.hip).
//
// score(i, j) = (q_i . W_uk c_j + qr_i . kr_j) * scale per head, over the keys j <= i of a sliding window (window 0: all
// of them); output per head: softmax-weighted sum of W_uv c_j.
//   absorbed form: W_uk^T q_i is a vector of the latent's size, so scores and weighted sums run on the cache rows
//     themselves and W_uv is applied to the summed latent.  Everything in fp32.  Decode, fp32 models, few rows.
//   expanded form: keys and values of the visible range are made once by two matrix products, then a tiled softmax
//     attention on the matrix cores.  Many rows of a bf16 model.
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include "row_ops.h"

namespace mg {

struct LatentDecode {
    const float* qlat = nullptr;     // [T, heads, rankPad]: W_uk^T q (past rank any finite value: cache rows are zero there)
    const float* q = nullptr;        // [T, heads, headW]: the rotated part (not turned yet) from column ropeOff of a head
    int headW = 0, ropeOff = 0;
    LatentCache cache;
    int heads = 0, window = 0;
    float scale = 0.f;
    const StepState* state = nullptr;    // position (T = 1), or NULL: pos0 + t
    int pos0 = 0, T = 1;
    int splits = 1, splitLen = 0;    // split s sees keys first + s * splitLen ..
    float* pacc = nullptr;           // [T, heads, splits, rankPad]
    float* pm = nullptr;             // [T, heads, splits]
    float* pl = nullptr;
};
// Splits for a span of at most `span` keys and T rows.
void latent_decode_splits(int span, int heads, int T, int* splits, int* splitLen);
bool latent_decode_supported(int rank, int rot);
hipError_t launch_latent_decode(const LatentDecode& p, hipStream_t s);

struct LatentPrefill {
    const unsigned short* q = nullptr;   // bf16 [T, ldq]: heads of [dimPad | turned rotated part, zero up to headW]
    int ldq = 0, headW = 0, dimPad = 0;
    const unsigned short* k = nullptr;   // bf16 [keys, heads * dimPad] of positions kBase ..
    const unsigned short* vt = nullptr;  // bf16 [heads * vPad, ldv]: values of positions kBase .., transposed
    int ldv = 0, vPad = 0;
    LatentCache cache;                   // rotated key parts
    int kBase = 0;
    int heads = 0, window = 0;
    float scale = 0.f;
    int T = 0, pos0 = 0;
    unsigned short* out = nullptr;       // bf16 [T, ldo], heads of vPad
    int ldo = 0;
};
// Padded sizes the kernel has variants for: headW for dim and rot (0: none), vPad for vdim (0: none).
int latent_prefill_head_width(int dimPad, int rot);
int latent_prefill_value_width(int vdim);
bool latent_prefill_supported(int headW, int vPad);
hipError_t launch_latent_prefill(const LatentPrefill& p, hipStream_t s);

}  // namespace mg
