// The model object behind the forge_hip_model handle: what every network shares (the step function with its graph, the
// position, sampling state, prompt chunks, profiling) and the interface a network implements (llama.hip, block_model.hip).
#pragma once

#include <algorithm>
#include <memory>
#include <vector>

#include "common.h"

namespace fh {

constexpr uint32_t PREFILL_CHUNK = 4096;   // rows of scratch for batched prefill

struct DevBuf {
    void* p = nullptr;
    DevBuf() = default;
    DevBuf(const DevBuf&) = delete;
    DevBuf& operator=(const DevBuf&) = delete;
    ~DevBuf() { if (p) (void)hipFree(p); }
    int32_t alloc(size_t n) {
        FH_HIP(hipMalloc(&p, n < 16 ? 16 : n));
        return FORGE_HIP_OK;
    }
    template <typename T> T* as() const { return reinterpret_cast<T*>(p); }
};

// Stage ids of forward_profile / prefill_profile (the order of FORGE_HIP_STAGE_* in forge_hip.h).
enum Stage { ST_EMBED = 0, ST_RMSNORM, ST_QKV, ST_ROPE, ST_ATTN, ST_QUANT, ST_O, ST_GATE_UP, ST_SILU, ST_DOWN, ST_LM_HEAD,
             ST_ARGMAX, ST_COUNT };
static_assert(ST_COUNT == FORGE_HIP_NUM_STAGES, "stage table out of step with forge_hip.h");

}  // namespace fh

struct forge_hip_model {
    forge_hip_config cfg{};              // shared code reads vocab, max_seq and layers; the rest belongs to the network
    hipStream_t stream = nullptr;
    fh::DevBuf logits, state, argmax_ws;
    fh::DevBuf counts;                   // u32 [vocab]: how often each token id has been fed since the last reset
    fh::DevBuf ptok;                     // token ids of one prompt chunk
    float repeat_penalty = 1.0f;         // > 1: forward_greedy picks the maximum of the penalised logits
    uint32_t chunk_rows = 0;             // rows of a prompt chunk
    // pinned host staging: [0] token, [1] next token, [2] position
    uint32_t* h_stage = nullptr;
    float* h_logits = nullptr;           // pinned: logits come home at PCIe speed and are copied to the caller's (pageable) buffer from here
    int64_t pos = 0;
    bool use_graph = true;
    hipGraphExec_t decode_graph = nullptr;
    // forward_profile / prefill_profile: one event pair per kernel launch, tagged with the stage of the
    // enclosing StageMark (ST_COUNT = outside any stage, not measured)
    int prof_cur = 0;
    std::vector<hipEvent_t> prof_ev;
    std::vector<int> prof_stage;
    size_t prof_used = 0;

    uint32_t* d_pos() const { return state.as<uint32_t>(); }
    uint32_t* d_token() const { return state.as<uint32_t>() + 1; }
    uint32_t* d_next() const { return state.as<uint32_t>() + 2; }

    virtual ~forge_hip_model();
    // Stream, pinned staging, decode state and sampling state for cfg (set before the call).
    int32_t init_shared();
    // Last maximum of `logits` -> d_next() (+ position and token advance when `advance`).
    void enqueue_argmax(bool penalise, bool advance);

    // ---- the network -----------------------------------------------------------------------------
    // One decode step: the token *d_token() at position *d_pos(), logits, argmax, advance.  Captured into a graph.
    virtual void enqueue_decode_step() = 0;
    // `rows` tokens of a prompt (ptok) at positions base_pos..; fills the cache and leaves the rows' residual stream.
    virtual int32_t enqueue_prompt_rows(uint32_t rows, uint32_t base_pos) = 0;
    // Logits of row `row` of the last chunk (and their argmax) as they follow a prompt.
    virtual void enqueue_row_logits(uint32_t row) = 0;
    // How many rows enqueue_rows_logits takes at once; more than one: [n][vocab] floats in `logits`.
    virtual uint32_t logits_rows_max() const { return 1; }
    virtual void enqueue_rows_logits(const uint32_t* rows, uint32_t n) { (void)n; enqueue_row_logits(rows[0]); }
    // false: only the last row of a chunk is still there when the chunk is done
    virtual bool keeps_rows() const { return true; }
    virtual int32_t decode_launches() const = 0;

    // ---- optional parts ------------------------------------------------------------------------------
    // A step that is one resident kernel: it takes the token with the launch and hands the next one over through host memory.
    virtual bool resident() const { return false; }
    virtual int32_t resident_enqueue(bool profile, uint32_t token) { (void)profile; (void)token; return FORGE_HIP_OK; }
    virtual bool resident_wait_token(uint32_t* next) { (void)next; return false; }
    virtual int32_t resident_after_sync(uint32_t abort_flag) { (void)abort_flag; return FORGE_HIP_OK; }
    virtual int32_t resident_profile(float* stage_ms, uint32_t* stage_launches) { (void)stage_ms; (void)stage_launches; return FORGE_HIP_OK; }
    virtual int32_t repeat_penalty_changed(float penalty) { (void)penalty; return FORGE_HIP_OK; }
    virtual void poll_limit_changed(uint32_t polls) { (void)polls; }
    virtual int32_t set_kv_pages(uint32_t page_rows, const uint32_t* table, uint32_t n_pages);
    virtual int32_t read_kv(uint32_t layer, uint32_t which, uint16_t* out_host);
    // Residual stream after every layer run for `rows` tokens (ptok) of an empty cache, [runs][rows][hidden] on the host.
    virtual uint32_t layer_runs() const { return cfg.layers; }
    virtual int32_t prompt_residuals(uint32_t rows, float* out_host);
};

namespace fh {

// While the model is profiling, names the stage that the launches of one scope are counted under.
struct StageMark {
    forge_hip_model* m;
    int saved;
    StageMark(forge_hip_model* model, int stage) : m(model), saved(model->prof_cur) { m->prof_cur = stage; }
    ~StageMark() { m->prof_cur = saved; }
};

}  // namespace fh
