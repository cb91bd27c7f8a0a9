// context.h -- DecodeContext: what every model class of the library shares.  It owns the stream, the
// device-resident step state, the token history, the captured token graphs and the loops over tokens (decode,
// greedy generation, timed and instrumented runs); a model class supplies the launches of one token, the
// multi-token prefill, its weights and its cache or state.
#pragma once
#include "kernels.h"

#include <cstdint>
#include <string>
#include <vector>

namespace mg {

inline size_t alignUp256(size_t v) { return (v + 255) & ~(size_t)255; }

// One device allocation handed out in 256-byte aligned pieces.
struct Slab {
    char* base = nullptr;
    size_t size = 0, used = 0;
    int init(size_t bytes);
    void* take(size_t bytes);
    void release();
};

void set_error(const std::string& s);
const std::string& get_error();

#define HIPCHK(expr)                                                                      \
    do {                                                                                  \
        hipError_t e_ = (expr);                                                           \
        if (e_ != hipSuccess) {                                                           \
            set_error(std::string(#expr) + ": " + hipGetErrorString(e_));                 \
            (void)hipGetLastError();                                                      \
            return MG_E_HIP;                                                              \
        }                                                                                 \
    } while (0)

#define ARGCHK(cond, msg)                                                                 \
    do {                                                                                  \
        if (!(cond)) { set_error(msg); return MG_E_ARG; }                                 \
    } while (0)

class DecodeContext {
public:
    virtual ~DecodeContext();

    int DecodeToken(int token, int pos, int* nextToken, float* logitsOut);
    int Generate(const int* prompt, int nPrompt, int nDecode, int* outTokens, bool useGraph);
    int GraphCapture();                                                           // cuda_graph.go:315
    int GraphLaunch(int token, int pos, int* nextToken);                          // cuda_graph.go:663
    int GraphValidate(int token, int pos, float* maxAbsDiff);                     // cuda_graph.go:554
    int TimedDecode(int token, int pos, int steps, bool useGraph, float* elapsedMs);
    int ProfileDecode(int token, int pos, int steps, unsigned classMask, float* classMs, int* classLaunches);
    int GeneratePrefill(const int* prompt, int nPrompt, int nDecode, int* outTokens);
    virtual int ExportHidden(float* out);                                                 // cuda_fused_infer.go:235
    // nTokens positions starting at pos0 in one pass: fills the caches and states, leaves the last position's
    // hidden state, logits and greedy token, and the device step state ready for the decode that follows.
    virtual int Prefill(const int* tokens, int nTokens, int pos0, int* nextToken, float* logitsOut, float* elapsedMs) = 0;
    // The same with the logits of chosen rows (indices into tokens) instead of the last one's: logitsOut [nWant, vocab].
    virtual int PrefillLogits(const int* tokens, int nTokens, int pos0, const int* want, int nWant, float* logitsOut) = 0;
    // Forget the sequence: caches and states as before the first token.
    virtual int ResetKV() = 0;
    virtual uint64_t WeightBytesPerToken() const = 0;
    virtual uint64_t KVBytesAt(int pos) const = 0;

    // shape
    int dim = 0, vocabSize = 0, nLayers = 0, maxSeq = 0;
    float eps = 0.f;
    hipStream_t stream = nullptr;
    float* hidden[2] = {nullptr, nullptr};
    int hiddenIdx = 0;
    float* logits = nullptr;
    int statePosHost = -1;                    // the device state's position where the host knows it, else -1

protected:
    DecodeContext() = default;
    // Stream, events, pinned words and the scratch slab (extraBytes for the model class) with the token-level
    // buffers taken from it.  maxSeq, dim and vocabSize are set.
    int initTokenState(size_t extraBytes);
    int invalidateGraphs();
    int mark(int cls);
    int primeGraph() { return enqueueEmbed(); }

    // ---- what a model class supplies ----
    virtual int checkReady() = 0;                         // weights and caches complete
    virtual int enqueueEmbed() = 0;                       // hidden <- embedding of the device state's token
    virtual int enqueueToken(bool withHead) = 0;          // embed -> layers -> final(+argmax) / advance, all from device state
    virtual RopeCur ropeRef() const { return RopeCur{}; }
    // May a step run at this position now?  (A recurrent state only continues where it stopped.)
    virtual int checkPosition(int pos) { (void)pos; return MG_OK_; }
    virtual void steppedTo(int pos) { (void)pos; }        // the sequence now holds positions 0 .. pos - 1 (-1: unknown)
    virtual int setState(int pos, int token, int count, int nPrompt);
    virtual int decodeRun(int nTokens, bool useGraph);    // nTokens decode steps from the device state
    virtual bool runsInLaunch(bool useGraph) const { (void)useGraph; return false; }   // ... as runs of tokens inside one launch
    virtual int prepareRun() { return MG_OK_; }           // allocations before a timed region / a run in the launch
    virtual bool hostPositions() const { return false; }  // launches that take their position from the host (never captured)
    virtual int enqueueTokenAt(int pos) { (void)pos; return enqueueToken(true); }
    virtual int setHostPositions(int mode) { (void)mode; return 0; }   // exec mode switch around GraphValidate
    virtual bool captureCurrent() const { return true; }  // the captured graphs still fit how tokens are launched
    virtual int beforeCapture() { return MG_OK_; }
    virtual int finishRun() { return MG_OK_; }            // after a synchronisation: did a launch report an error?
    virtual int saveSequence() { return MG_OK_; }         // GraphValidate runs one step twice
    virtual int restoreSequence() { return MG_OK_; }
    virtual void graphsInvalidated() {}

    static constexpr int MG_OK_ = 0;
    bool built = false;
    bool fuseEmbed = false;      // set while the graphs are captured
    Slab scratch;
    // embedding table (optional for models whose lm_head is tied)
    int embedKind = -1;       // kinds of launch_embed_token
    void* embedTable = nullptr;
    // token-level state
    StepState* dState = nullptr;
    StepState* hState = nullptr;    // pinned mirror
    int* hGate = nullptr;           // pinned flag the timing gate kernel polls
    float* amaxVal = nullptr;
    int* amaxIdx = nullptr;
    int amaxParts = 0;
    int* dHistory = nullptr;
    int* dPrompt = nullptr;
    int* hTokens = nullptr;         // pinned
    unsigned graphGeneration = 0;     // bumped by whatever makes captured graphs stale (weights, caches, modes)
    hipGraph_t graphFull = nullptr, graphPrompt = nullptr;
    hipGraphExec_t execFull = nullptr, execPrompt = nullptr;
    hipEvent_t ev0 = nullptr, ev1 = nullptr;
    // instrumented run: an event between every two launches of a token
    std::vector<hipEvent_t> profEvents;
    std::vector<int> profClass;       // class of the launch that follows event i
    bool profiling = false;
    unsigned profMask = 0xffu;
    int profLast = -1;
};

class HIPFusedInference;
class LayeredInference;

}  // namespace mg

// The opaque handle of the C ABI.  f is the model; fused / layered is the same object where it is of that class.
struct mg_layer_graph;
struct mg_ctx {
    mg::DecodeContext* f = nullptr;
    mg::HIPFusedInference* fused = nullptr;
    mg::LayeredInference* layered = nullptr;
    std::vector<mg_layer_graph*> layerGraphs;      // live graph objects: they outlive the context as dead handles
    void (*dropGraphs)(mg_ctx*) = nullptr;         // set by who creates layer graphs
};
