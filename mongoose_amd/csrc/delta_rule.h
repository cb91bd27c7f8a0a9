// delta_rule.h -- the generalized delta rule (delta_rule.hip): per head a state S [dim key channels, dim value channels]
// in fp32,
//   S <- diag(w) S - (a u)(u^T S) + k v^T  (both terms from the old state),   o = S^T r,
// with u = k / sqrt(sum k^2 + 1e-6), w = exp(-exp(-1/2) sigmoid(W2 tanh(W1 h) + w0)), a = sigmoid(Wa h + b); then
// y = o / rms(o) * norm * sigmoid(Wg h).
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include "linear.h"
#include "row_ops.h"

namespace mg {

// The projections of a token lie in one row z = [r | k | v | g | a | w1 h], each but the last heads * dim wide.
struct DeltaParams {
    int heads = 0, dim = 0, rank = 0;
    const float* aBias = nullptr;    // [heads * dim]
    const float* w0 = nullptr;
    const float* norm = nullptr;
    Bf16Mat w2;                      // [heads * dim, rank]
    float eps = 0.f;
};

struct DeltaStep {
    DeltaParams d;
    const float* z = nullptr;
    float* S = nullptr;              // [heads, dim, dim]
    const StepState* state = nullptr;    // at position 0 the state counts as zero
    float* y = nullptr;              // [heads * dim]
    SideJobs side;
};
hipError_t launch_delta_step(const DeltaStep& p, hipStream_t s);

struct DeltaRows {
    DeltaParams d;
    const float* z = nullptr;        // [T, ldz]
    int ldz = 0, T = 0, pos0 = 0;
    float* S = nullptr;
    float* w1 = nullptr;             // work: [T, rank padded to 64] tanh(W1 h); zero past rank
    float* dec = nullptr;            // work: [T, heads * dim] W2 tanh(..) , then the decay
    float* au = nullptr;             // work: a u
    float* u = nullptr;              // work
    float* o = nullptr;              // work: [T, heads * dim]
    float* chunks = nullptr;         // work: delta_chunk_floats() floats, or NULL: always token by token
    void* yAct = nullptr;            // [T, ldAct]
    int actF32 = 0, ldAct = 0;
};
constexpr int DELTA_CHUNK_MIN_ROWS = 64;     // fewer rows go token by token
// Workspace of the chunked form for T rows; 0 where it is not used.
size_t delta_chunk_floats(int heads, int dim, int T);
bool delta_supported(int dim);
hipError_t launch_delta_rows(const DeltaRows& p, hipStream_t s);

}  // namespace mg
