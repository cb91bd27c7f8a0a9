// context.hip -- DecodeContext (token loops, graphs, timing over any model class) and the mg_* C entry points that
// every model class has.  Host code only (no kernels here); compiled with hipcc for the runtime API.
#include "context.h"
#include "../../include/mongoose_hip.h"

#include <algorithm>
#include <cmath>
#include <cstring>

namespace mg {

static thread_local std::string g_err;
void set_error(const std::string& s) { g_err = s; }
const std::string& get_error() { return g_err; }

int Slab::init(size_t bytes) {
    release();
    void* v = nullptr;
    HIPCHK(hipMalloc(&v, bytes ? bytes : 256));
    base = static_cast<char*>(v); size = bytes; used = 0;
    return MG_OK;
}
void* Slab::take(size_t bytes) {
    size_t off = alignUp256(used);
    if (!base || off + bytes > size) return nullptr;
    used = off + bytes;
    return base + off;
}
void Slab::release() {
    if (base) (void)hipFree(base);
    base = nullptr; size = used = 0;
}

int DecodeContext::initTokenState(size_t extraBytes) {
    HIPCHK(hipStreamCreateWithFlags(&stream, hipStreamNonBlocking));
    HIPCHK(hipEventCreate(&ev0));
    HIPCHK(hipEventCreate(&ev1));
    amaxParts = 4096;
    const size_t words = (size_t)2 * dim + vocabSize + 2 * (size_t)amaxParts + 2 * ((size_t)maxSeq + 1) + 16;
    const size_t bytes = words * 4 + 16 * 256 + extraBytes;
    int rc = scratch.init(bytes);
    if (rc) return rc;
    HIPCHK(hipMemsetAsync(scratch.base, 0, bytes, stream));
    HIPCHK(hipStreamSynchronize(stream));
    auto takeF = [&](float*& p, size_t n) { p = static_cast<float*>(scratch.take(n * 4)); return p != nullptr; };
    auto takeI = [&](int*& p, size_t n) { p = static_cast<int*>(scratch.take(n * 4)); return p != nullptr; };
    bool ok = takeF(hidden[0], dim) && takeF(hidden[1], dim) && takeF(logits, vocabSize) && takeF(amaxVal, amaxParts) &&
              takeI(amaxIdx, amaxParts) && takeI(dHistory, (size_t)maxSeq + 1) && takeI(dPrompt, (size_t)maxSeq + 1);
    if (ok) { dState = static_cast<StepState*>(scratch.take(sizeof(StepState))); ok = dState != nullptr; }
    if (!ok) { set_error("scratch slab too small"); return MG_E_STATE; }
    void* hp = nullptr;
    HIPCHK(hipHostMalloc(&hp, sizeof(StepState), hipHostMallocDefault));
    hState = static_cast<StepState*>(hp);
    HIPCHK(hipHostMalloc(&hp, 64, hipHostMallocCoherent | hipHostMallocMapped));
    hGate = static_cast<int*>(hp);
    *hGate = 1;
    HIPCHK(hipHostMalloc(&hp, sizeof(int) * ((size_t)maxSeq + 1), hipHostMallocDefault));
    hTokens = static_cast<int*>(hp);
    return MG_OK;
}

DecodeContext::~DecodeContext() {
    if (stream) (void)hipStreamSynchronize(stream);
    if (execFull) (void)hipGraphExecDestroy(execFull);
    if (execPrompt) (void)hipGraphExecDestroy(execPrompt);
    if (graphFull) (void)hipGraphDestroy(graphFull);
    if (graphPrompt) (void)hipGraphDestroy(graphPrompt);
    scratch.release();
    if (embedTable) (void)hipFree(embedTable);
    if (hState) (void)hipHostFree(hState);
    if (hGate) (void)hipHostFree(hGate);
    if (hTokens) (void)hipHostFree(hTokens);
    for (hipEvent_t e : profEvents) (void)hipEventDestroy(e);
    if (ev0) (void)hipEventDestroy(ev0);
    if (ev1) (void)hipEventDestroy(ev1);
    if (stream) (void)hipStreamDestroy(stream);
}

int DecodeContext::invalidateGraphs() {
    graphGeneration++;
    graphsInvalidated();
    if (execFull) { (void)hipGraphExecDestroy(execFull); execFull = nullptr; }
    if (execPrompt) { (void)hipGraphExecDestroy(execPrompt); execPrompt = nullptr; }
    if (graphFull) { (void)hipGraphDestroy(graphFull); graphFull = nullptr; }
    if (graphPrompt) { (void)hipGraphDestroy(graphPrompt); graphPrompt = nullptr; }
    return MG_OK;
}

// While the instrumented graph is being captured: an event before the launch
// of class `cls` (the previous launch's end).  No-op otherwise.
int DecodeContext::mark(int cls) {
    if (!profiling) return MG_OK;
    // an event opens the interval of a wanted class and closes the interval of the one before it
    const bool opens = cls >= 0 && cls < 8 && ((profMask >> cls) & 1);
    const bool closes = profLast >= 0 && profLast < 8 && ((profMask >> profLast) & 1);
    profLast = cls;
    if (!opens && !closes) return MG_OK;
    if (!opens) cls = 8;                      // interval that follows is not measured
    hipEvent_t e = nullptr;
    HIPCHK(hipEventCreate(&e));
    profEvents.push_back(e);
    profClass.push_back(cls);
    HIPCHK(hipEventRecord(e, stream));
    return MG_OK;
}

// Sets the device-resident step state.
int DecodeContext::setState(int pos, int token, int count, int nPrompt) {
    HIPCHK(launch_set_state(dState, pos, token, count, nPrompt, ropeRef(), stream));
    statePosHost = pos;
    return MG_OK;
}

int DecodeContext::decodeRun(int nTokens, bool useGraph) {
    for (int i = 0; i < nTokens; i++) {
        statePosHost = -1;                          // (advanced on the device by launches that do not tell the host)
        if (useGraph) HIPCHK(hipGraphLaunch(execFull, stream));
        else { int rc = enqueueToken(true); if (rc) return rc; }
    }
    return MG_OK;
}

int DecodeContext::ExportHidden(float* out) {
    if (!built) return MG_E_NOT_BUILT;
    ARGCHK(out, "ExportHidden: NULL out");
    HIPCHK(hipStreamSynchronize(stream));
    HIPCHK(hipMemcpy(out, hidden[hiddenIdx], (size_t)dim * 4, hipMemcpyDeviceToHost));
    return finishRun();
}

int DecodeContext::DecodeToken(int token, int pos, int* nextToken, float* logitsOut) {
    if (!built) return MG_E_NOT_BUILT;
    ARGCHK(pos >= 0 && pos < maxSeq && token >= 0 && token < vocabSize, "DecodeToken: token or pos out of range");
    int rc = checkReady();
    if (rc) return rc;
    rc = checkPosition(pos);
    if (rc) return rc;
    { int rcs = setState(pos, token, 0, 0); if (rcs) return rcs; }
    rc = hostPositions() ? enqueueTokenAt(pos) : enqueueToken(true);
    if (rc) return rc;
    HIPCHK(hipMemcpyAsync(hTokens, dHistory, sizeof(int), hipMemcpyDeviceToHost, stream));
    HIPCHK(hipStreamSynchronize(stream));
    steppedTo(pos + 1);
    if (nextToken) *nextToken = hTokens[0];
    if (logitsOut) HIPCHK(hipMemcpy(logitsOut, logits, (size_t)vocabSize * 4, hipMemcpyDeviceToHost));
    return finishRun();
}

// Two whole-token graphs: with the lm_head and argmax, and for prompt positions without them.  The kernels read
// position and token from device memory, so one capture serves every position.
int DecodeContext::GraphCapture() {
    if (!built) return MG_E_NOT_BUILT;
    int rc = checkReady();
    if (rc) return rc;
    if (execFull && execPrompt && captureCurrent()) return MG_OK;
    invalidateGraphs();
    rc = beforeCapture();                           // allocations and uploads come before the capture
    if (rc) return rc;
    HIPCHK(hipStreamSynchronize(stream));
    statePosHost = -1;                              // a captured launch is replayed at any position: the variant that covers all
    for (int which = 0; which < 2; which++) {
        HIPCHK(hipStreamBeginCapture(stream, hipStreamCaptureModeRelaxed));
        fuseEmbed = true;
        rc = enqueueToken(which == 0);
        fuseEmbed = false;
        hipGraph_t g = nullptr;
        hipError_t e = hipStreamEndCapture(stream, &g);
        if (rc) { if (g) (void)hipGraphDestroy(g); return rc; }
        HIPCHK(e);
        hipGraphExec_t ex = nullptr;
        HIPCHK(hipGraphInstantiate(&ex, g, nullptr, nullptr, 0));
        if (which == 0) { graphFull = g; execFull = ex; } else { graphPrompt = g; execPrompt = ex; }
    }
    return MG_OK;
}

int DecodeContext::GraphLaunch(int token, int pos, int* nextToken) {
    if (!built) return MG_E_NOT_BUILT;
    ARGCHK(pos >= 0 && pos < maxSeq && token >= 0 && token < vocabSize, "GraphLaunch: token or pos out of range");
    int rc = GraphCapture();
    if (rc) return rc;
    rc = checkPosition(pos);
    if (rc) return rc;
    { int rcs = setState(pos, token, 0, 0); if (rcs) return rcs; }
    rc = primeGraph();
    if (rc) return rc;
    statePosHost = -1;
    HIPCHK(hipGraphLaunch(execFull, stream));
    HIPCHK(hipMemcpyAsync(hTokens, dHistory, sizeof(int), hipMemcpyDeviceToHost, stream));
    HIPCHK(hipStreamSynchronize(stream));
    steppedTo(pos + 1);
    if (nextToken) *nextToken = hTokens[0];
    return finishRun();
}

int DecodeContext::GraphValidate(int token, int pos, float* maxAbsDiff) {
    if (!built) return MG_E_NOT_BUILT;
    std::vector<float> a(vocabSize), b(vocabSize);
    int t0 = -1, t1 = -1;
    int rc = checkPosition(pos);
    if (rc == MG_OK) rc = saveSequence();
    if (rc) return rc;
    const int saved = setHostPositions(-1);  // launches with host positions are not captured: compare the graph with the fused launches
    rc = DecodeToken(token, pos, &t0, a.data());
    setHostPositions(saved);
    if (rc == MG_OK) rc = restoreSequence();
    if (rc) return rc;
    rc = GraphLaunch(token, pos, &t1);
    if (rc) return rc;
    HIPCHK(hipMemcpy(b.data(), logits, (size_t)vocabSize * 4, hipMemcpyDeviceToHost));
    float md = 0.f;
    for (int i = 0; i < vocabSize; i++) md = std::fmax(md, std::fabs(a[i] - b[i]));
    if (t0 != t1) md = std::fmax(md, 1.0f);
    if (maxAbsDiff) *maxAbsDiff = md;
    return MG_OK;
}

int DecodeContext::Generate(const int* prompt, int nPrompt, int nDecode, int* outTokens, bool useGraph) {
    if (!built) return MG_E_NOT_BUILT;
    ARGCHK(prompt && nPrompt >= 1 && nDecode >= 0 && outTokens, "Generate: bad arguments");
    ARGCHK(nPrompt + nDecode <= maxSeq + 1 && nPrompt <= maxSeq, "Generate: prompt + decode exceeds maxSeq");
    for (int i = 0; i < nPrompt; i++) ARGCHK(prompt[i] >= 0 && prompt[i] < vocabSize, "Generate: prompt token out of range");
    int rc = checkReady();
    if (rc) return rc;
    rc = checkPosition(0);
    if (rc) return rc;
    if (hostPositions()) {
        // per-op mode: host-driven loop, one synchronisation per token
        int tok = prompt[0];
        for (int pos = 0; pos < nPrompt - 1 + nDecode; pos++) {
            int next = -1;
            rc = DecodeToken(tok, pos, &next, nullptr);
            if (rc) return rc;
            if (pos + 1 < nPrompt) tok = prompt[pos + 1];
            else { outTokens[pos + 1 - nPrompt] = next; tok = next; }
        }
        return MG_OK;
    }
    // (where runs of tokens go into one launch no graph is needed: the prompt steps are launched one by one)
    const bool graphs = useGraph && !runsInLaunch(useGraph);
    if (graphs) { rc = GraphCapture(); if (rc) return rc; }
    HIPCHK(hipStreamSynchronize(stream));
    HIPCHK(hipMemcpy(dPrompt, prompt, sizeof(int) * (size_t)nPrompt, hipMemcpyHostToDevice));
    { int rcs = setState(0, prompt[0], 0, nPrompt); if (rcs) return rcs; }
    if (graphs) { rc = primeGraph(); if (rc) return rc; }
    for (int i = 0; i < nPrompt - 1; i++) {
        if (graphs) HIPCHK(hipGraphLaunch(execPrompt, stream));
        else { rc = enqueueToken(false); if (rc) return rc; }
    }
    statePosHost = nPrompt - 1;                     // one position a prompt step since setState(0, ..)
    steppedTo(-1);                                  // (until the run is known to have ended)
    rc = decodeRun(nDecode, useGraph);
    if (rc) return rc;
    if (nDecode > 0) HIPCHK(hipMemcpyAsync(hTokens, dHistory, sizeof(int) * (size_t)nDecode, hipMemcpyDeviceToHost, stream));
    HIPCHK(hipStreamSynchronize(stream));
    for (int i = 0; i < nDecode; i++) outTokens[i] = hTokens[i];
    steppedTo(nPrompt - 1 + nDecode);
    return finishRun();
}

int DecodeContext::TimedDecode(int token, int pos, int steps, bool useGraph, float* elapsedMs) {
    if (!built) return MG_E_NOT_BUILT;
    ARGCHK(steps >= 1 && pos >= 0 && pos + steps <= maxSeq && token >= 0 && token < vocabSize, "TimedDecode: bad arguments");
    int rc = checkReady();
    if (rc) return rc;
    const bool graphs = useGraph && !runsInLaunch(useGraph);
    if (graphs) { rc = GraphCapture(); if (rc) return rc; }
    rc = prepareRun();                              // (allocations before the timed region)
    if (rc) return rc;
    // measurements may start anywhere; the sequence the caches and states held is given up unless this continues it
    const bool continues = checkPosition(pos) == MG_OK;
    steppedTo(-1);
    { int rcs = setState(pos, token, 0, 0); if (rcs) return rcs; }
    if (graphs) { rc = primeGraph(); if (rc) return rc; }
    HIPCHK(hipStreamSynchronize(stream));
    HIPCHK(hipEventRecord(ev0, stream));
    rc = decodeRun(steps, useGraph);
    if (rc) return rc;
    HIPCHK(hipEventRecord(ev1, stream));
    HIPCHK(hipEventSynchronize(ev1));
    float ms = 0.f;
    HIPCHK(hipEventElapsedTime(&ms, ev0, ev1));
    if (elapsedMs) *elapsedMs = ms;
    if (continues) steppedTo(pos + steps);
    return finishRun();
}

// Per-launch-class durations inside a token.  Events cannot be read back from
// graph nodes, so the same launches are issued eagerly with an event between
// every two of them -- behind a gate kernel that holds the stream until the
// host has queued the whole batch, so the GPU never waits for the host.
// classMs[c] = mean milliseconds from the end of the previous launch to the
// end of a launch of class c (0 embed, 1 norm+QKV, 2 attention, 3 Wo,
// 4 gate/up, 5 down, 6 lm_head, 7 argmax finish); classLaunches[c] = launches per token.
int DecodeContext::ProfileDecode(int token, int pos, int steps, unsigned classMask, float* classMs, int* classLaunches) {
    if (!built) return MG_E_NOT_BUILT;
    ARGCHK(steps >= 1 && steps <= 64 && pos >= 0 && pos + steps <= maxSeq && token >= 0 && token < vocabSize &&
           classMs && classLaunches, "ProfileDecode: bad arguments (1 <= steps <= 64)");
    int rc = checkReady();
    if (rc) return rc;
    HIPCHK(hipStreamSynchronize(stream));
    for (hipEvent_t e : profEvents) (void)hipEventDestroy(e);
    profEvents.clear(); profClass.clear();
    const bool continues = checkPosition(pos) == MG_OK;
    steppedTo(-1);
    int* gate = hGate;
    *reinterpret_cast<volatile int*>(gate) = 0;
    { int rcs = setState(pos, token, 0, 0); if (rcs) return rcs; }
    HIPCHK(launch_gate(gate, 100LL * 1000 * 500, stream));   // at most 0.5 s
    profiling = true;
    profMask = classMask ? classMask : 0xffu;
    profLast = -1;
    for (int i = 0; i < steps && rc == 0; i++) {
        rc = enqueueToken(true);
        if (rc == 0) rc = mark(8);
    }
    profiling = false;
    *reinterpret_cast<volatile int*>(gate) = 1;
    HIPCHK(hipStreamSynchronize(stream));
    if (rc) return rc;
    double acc[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    int cnt[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    for (size_t k = 0; k + 1 < profEvents.size(); k++) {
        int c = profClass[k];
        if (c < 0 || c >= 8) continue;
        float ms = 0.f;
        HIPCHK(hipEventElapsedTime(&ms, profEvents[k], profEvents[k + 1]));
        acc[c] += ms; cnt[c]++;
    }
    for (int c = 0; c < 8; c++) {
        classMs[c] = cnt[c] ? (float)(acc[c] / cnt[c]) : 0.f;
        classLaunches[c] = cnt[c] / steps;
    }
    for (hipEvent_t e : profEvents) (void)hipEventDestroy(e);
    profEvents.clear(); profClass.clear();
    if (continues) steppedTo(pos + steps);
    return MG_OK;
}

// Prompt through the GEMM path, then nDecode - 1 graph replays from the device state it left.
int DecodeContext::GeneratePrefill(const int* prompt, int nPrompt, int nDecode, int* outTokens) {
    if (!built) return MG_E_NOT_BUILT;
    ARGCHK(prompt && nPrompt >= 1 && nDecode >= 1 && outTokens, "GeneratePrefill: bad arguments");
    ARGCHK(nPrompt + nDecode <= maxSeq + 1, "GeneratePrefill: prompt + decode exceeds maxSeq");
    const bool graphs = !runsInLaunch(true);
    int rc = graphs ? GraphCapture() : MG_OK;
    if (rc) return rc;
    rc = Prefill(prompt, nPrompt, 0, nullptr, nullptr, nullptr);
    if (rc) return rc;
    if (nDecode > 1 && graphs) { rc = primeGraph(); if (rc) return rc; }
    steppedTo(-1);
    rc = decodeRun(nDecode - 1, true);
    if (rc) return rc;
    HIPCHK(hipMemcpyAsync(hTokens, dHistory, sizeof(int) * (size_t)nDecode, hipMemcpyDeviceToHost, stream));
    HIPCHK(hipStreamSynchronize(stream));
    for (int i = 0; i < nDecode; i++) outTokens[i] = hTokens[i];
    steppedTo(nPrompt - 1 + nDecode);
    return finishRun();
}

}  // namespace mg

// ---------------------------------------------------------------------------
// C entry points of every model class
// ---------------------------------------------------------------------------
#define CTX(c) if (!(c) || !(c)->f) { mg::set_error("NULL context"); return MG_E_NOT_BUILT; } mg::DecodeContext* f = (c)->f

extern "C" {

const char* mg_last_error(void) { return mg::get_error().c_str(); }
void mg_destroy(mg_ctx* c) {
    if (!c) return;
    if (c->dropGraphs) c->dropGraphs(c);
    delete c->f;
    delete c;
}
int mg_reset_kv(mg_ctx* c) { CTX(c); return f->ResetKV(); }
int mg_export_hidden(mg_ctx* c, float* out) { CTX(c); return f->ExportHidden(out); }
int mg_read_hidden(mg_ctx* c, float* out) { CTX(c); return f->ExportHidden(out); }
int mg_hidden_idx(mg_ctx* c) { CTX(c); return f->hiddenIdx; }
int mg_decode_token(mg_ctx* c, int token, int pos, int* next, float* logitsOut) { CTX(c); return f->DecodeToken(token, pos, next, logitsOut); }
int mg_generate(mg_ctx* c, const int* prompt, int nPrompt, int nDecode, int* out, int useGraph) {
    CTX(c); return f->Generate(prompt, nPrompt, nDecode, out, useGraph != 0);
}
int mg_graph_capture(mg_ctx* c) { CTX(c); return f->GraphCapture(); }
int mg_graph_launch(mg_ctx* c, int token, int pos, int* next) { CTX(c); return f->GraphLaunch(token, pos, next); }
int mg_graph_validate(mg_ctx* c, int token, int pos, float* md) { CTX(c); return f->GraphValidate(token, pos, md); }
int mg_has_graph_kernel(void) { return 1; }
int mg_timed_decode(mg_ctx* c, int token, int pos, int steps, int useGraph, float* ms) {
    CTX(c); return f->TimedDecode(token, pos, steps, useGraph != 0, ms);
}
int mg_profile_decode(mg_ctx* c, int token, int pos, int steps, unsigned classMask, float* classMs, int* classLaunches) {
    CTX(c); return f->ProfileDecode(token, pos, steps, classMask, classMs, classLaunches);
}
int mg_prefill(mg_ctx* c, const int* tokens, int nTokens, int pos0, int* next, float* logitsOut, float* ms) {
    CTX(c); return f->Prefill(tokens, nTokens, pos0, next, logitsOut, ms);
}
int mg_prefill_logits(mg_ctx* c, const int* tokens, int nTokens, int pos0, const int* want, int nWant, float* logitsOut) {
    CTX(c); return f->PrefillLogits(tokens, nTokens, pos0, want, nWant, logitsOut);
}
int mg_generate_prefill(mg_ctx* c, const int* prompt, int nPrompt, int nDecode, int* out) {
    CTX(c); return f->GeneratePrefill(prompt, nPrompt, nDecode, out);
}
uint64_t mg_weight_bytes_per_token(const mg_ctx* c) { return c && c->f ? c->f->WeightBytesPerToken() : 0; }
uint64_t mg_kv_bytes_at(const mg_ctx* c, int pos) { return c && c->f ? c->f->KVBytesAt(pos) : 0; }

}  // extern "C"
