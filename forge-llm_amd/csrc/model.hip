// extern "C" surface, part 2: the model handle (MetalModel::{forward, forward_prefill_batch, reset}, metal:5070-5981;
// model::{forward, forward_prefill_batched}, emit.rs:4029-5486) on one GPU, for every network: the step function, prompts in
// chunks, position, sampling state and profiling.  What a step computes is the network's part (llama.hip, block_model.hip).
//
// The decode step is captured once into a HIP graph (position and token live in device
// memory so the graph never changes) and replayed per token.
#include "model.h"

#include <string.h>

using namespace fh;

forge_hip_model::~forge_hip_model() {
    if (decode_graph) (void)hipGraphExecDestroy(decode_graph);
    for (hipEvent_t e : prof_ev) (void)hipEventDestroy(e);
    if (h_stage) (void)hipHostFree(h_stage);
    if (h_logits) (void)hipHostFree(h_logits);
    if (stream) (void)hipStreamDestroy(stream);
}

int32_t forge_hip_model::init_shared() {
    const char* genv = getenv("FORGE_HIP_GRAPH");
    use_graph = !(genv && genv[0] == '0');
    FH_HIP(hipStreamCreateWithFlags(&stream, hipStreamNonBlocking));
    FH_HIP(hipHostMalloc((void**)&h_stage, 64, hipHostMallocDefault));
    FH_HIP(hipHostMalloc((void**)&h_logits, (size_t)cfg.vocab * 4 * logits_rows_max(), hipHostMallocDefault));
    chunk_rows = std::min(PREFILL_CHUNK, cfg.max_seq);
    int32_t rc;
    if ((rc = logits.alloc((size_t)cfg.vocab * 4 * logits_rows_max())) || (rc = state.alloc(64)) || (rc = argmax_ws.alloc(ARGMAX_BLOCKS * 8)) ||
        (rc = counts.alloc((size_t)cfg.vocab * 4)) || (rc = ptok.alloc((size_t)chunk_rows * 4)))
        return rc;
    FH_HIP(hipMemset(state.p, 0, 64));
    FH_HIP(hipMemset(counts.p, 0, (size_t)cfg.vocab * 4));
    return FORGE_HIP_OK;
}

void forge_hip_model::enqueue_argmax(bool penalise, bool advance) {
    StageMark t(this, ST_ARGMAX);
    const bool pen = penalise && repeat_penalty > 1.0f;
    launch_argmax(logits.as<float>(), cfg.vocab, d_next(), argmax_ws.p, advance ? d_pos() : nullptr, advance ? d_token() : nullptr,
                  pen ? counts.as<uint32_t>() : nullptr, repeat_penalty, stream);
}

int32_t forge_hip_model::set_kv_pages(uint32_t page_rows, const uint32_t*, uint32_t) {
    FH_CHECK(page_rows == 0, "set_kv_pages: this network keeps a flat cache");
    return FORGE_HIP_OK;
}

int32_t forge_hip_model::read_kv(uint32_t, uint32_t, uint16_t*) {
    return fail(FORGE_HIP_ERR_INVALID, "read_kv: this network has no fp16 K/V cache");
}

int32_t forge_hip_model::prompt_residuals(uint32_t, float*) {
    return fail(FORGE_HIP_ERR_INVALID, "prefill_residuals: not available for this network");
}

namespace {

// Hands every kernel launch of a profiled pass its own pair of events (fh::launch attaches them to the
// dispatch) and remembers the stage it belongs to.
struct ModelProbe : LaunchProbe {
    forge_hip_model* m;
    explicit ModelProbe(forge_hip_model* model) : m(model) {
        m->prof_used = 0; m->prof_stage.clear(); m->prof_cur = ST_COUNT;
        launch_probe() = this;
    }
    ~ModelProbe() override { launch_probe() = nullptr; }
    bool next(hipEvent_t* start, hipEvent_t* stop) override {
        if (m->prof_cur == ST_COUNT) return false;
        if (m->prof_used + 2 > m->prof_ev.size()) {
            for (int i = 0; i < 2; i++) {
                hipEvent_t e = nullptr;
                if (hipEventCreate(&e) != hipSuccess) return false;
                m->prof_ev.push_back(e);
            }
        }
        *start = m->prof_ev[m->prof_used];
        *stop = m->prof_ev[m->prof_used + 1];
        m->prof_stage.push_back(m->prof_cur);
        m->prof_used += 2;
        return true;
    }
};

// Sum the kernels' device times per stage (milliseconds) after the stream has drained.
int32_t collect_profile(forge_hip_model* m, float* stage_ms, uint32_t* stage_launches) {
    for (int i = 0; i < ST_COUNT; i++) { stage_ms[i] = 0.f; if (stage_launches) stage_launches[i] = 0; }
    for (size_t i = 0; i * 2 < m->prof_used; i++) {
        float ms = 0.f;
        FH_HIP(hipEventElapsedTime(&ms, m->prof_ev[2 * i], m->prof_ev[2 * i + 1]));
        stage_ms[m->prof_stage[i]] += ms;
        if (stage_launches) stage_launches[m->prof_stage[i]] += 1;
    }
    return FORGE_HIP_OK;
}

int32_t run_decode_step(forge_hip_model* m, uint32_t token) {
    if (m->resident()) return m->resident_enqueue(false, token);   // the token rides with the launch
    m->h_stage[0] = token;
    FH_HIP(hipMemcpyAsync(m->d_token(), &m->h_stage[0], 4, hipMemcpyHostToDevice, m->stream));
    if (m->use_graph && !m->decode_graph) {
        hipGraph_t g = nullptr;
        FH_HIP(hipStreamBeginCapture(m->stream, hipStreamCaptureModeThreadLocal));
        m->enqueue_decode_step();
        hipError_t e = hipStreamEndCapture(m->stream, &g);
        if (e != hipSuccess || !g) return fail(FORGE_HIP_ERR_HIP, std::string("graph capture failed: ") + hipGetErrorString(e));
        e = hipGraphInstantiate(&m->decode_graph, g, nullptr, nullptr, 0);
        (void)hipGraphDestroy(g);
        if (e != hipSuccess) { m->decode_graph = nullptr; return fail(FORGE_HIP_ERR_HIP, std::string("graph instantiate failed: ") + hipGetErrorString(e)); }
    }
    if (m->decode_graph) FH_HIP(hipGraphLaunch(m->decode_graph, m->stream));
    else { m->enqueue_decode_step(); FH_HIP(hipGetLastError()); }
    return FORGE_HIP_OK;
}

// Reads back {next token, abort flag} after a decode step and waits for the stream.
int32_t finish_decode_step(forge_hip_model* m) {
    FH_HIP(hipMemcpyAsync(&m->h_stage[4], m->d_next(), 8, hipMemcpyDeviceToHost, m->stream));
    FH_HIP(hipStreamSynchronize(m->stream));
    if (m->resident()) return m->resident_after_sync(m->h_stage[5]);
    return FORGE_HIP_OK;
}

// Enqueues a decode step.  The position is counted as advanced here; a step that turns out not to have happened (the
// resident kernel gave up) is taken back by step_failed().
int32_t forward_common(forge_hip_model* m, uint32_t token) {
    FH_CHECK(m, "model is null");
    if (m->pos >= (int64_t)m->cfg.max_seq) return fail(FORGE_HIP_ERR_POSITION, "KV cache is full (pos == max_seq)");
    if (token >= m->cfg.vocab) return fail(FORGE_HIP_ERR_POSITION, "token id out of range");
    int32_t rc = run_decode_step(m, token);
    if (rc) return rc;
    m->pos += 1;
    return FORGE_HIP_OK;
}

// finish_decode_step() with the host's view put back in line with the device's when the step failed: the device position
// was not advanced, so neither is the host's, and the same token can be fed again.
int32_t finish_or_undo(forge_hip_model* m) {
    const int32_t rc = finish_decode_step(m);
    if (rc && m->pos > 0) m->pos -= 1;
    return rc;
}

// A prompt of n tokens in chunks; logits of the rows want[0..n_want) into logits_host [n_want][vocab].
int32_t prefill_rows(forge_hip_model* m, const uint32_t* tokens, uint64_t n, const uint64_t* want, uint64_t n_want, float* logits_host) {
    FH_CHECK(m && tokens, "prefill_batch: null pointer");
    FH_CHECK(n >= 1, "prefill_batch: empty token list");
    if ((uint64_t)m->pos + n > m->cfg.max_seq)
        return fail(FORGE_HIP_ERR_POSITION, "prompt does not fit the KV cache (pos + n > max_seq)");
    for (uint64_t i = 0; i < n; i++)
        if (tokens[i] >= m->cfg.vocab) return fail(FORGE_HIP_ERR_POSITION, "token id out of range");
    for (uint64_t i = 0; i < n_want; i++) FH_CHECK(want[i] < n, "prefill: a wanted row lies past the tokens");
    hipStream_t s = m->stream;
    const size_t vocab = m->cfg.vocab;
    uint64_t done = 0;
    std::vector<uint32_t> rows_w;
    std::vector<uint64_t> slot_w;
    while (done < n) {
        uint32_t rows = (uint32_t)std::min<uint64_t>(m->chunk_rows, n - done);
        if (!m->keeps_rows())
            for (uint64_t i = 0; i < n_want; i++)
                if (want[i] >= done && want[i] + 1 < done + rows) rows = (uint32_t)(want[i] + 1 - done);
        // pageable source: the copy is complete (staged) when the call returns
        FH_HIP(hipMemcpyAsync(m->ptok.p, tokens + done, (size_t)rows * 4, hipMemcpyHostToDevice, s));
        const int32_t rc = m->enqueue_prompt_rows(rows, (uint32_t)(m->pos + done));
        if (rc) return rc;
        FH_HIP(hipGetLastError());
        rows_w.clear();
        slot_w.clear();
        for (uint64_t i = 0; i < n_want; i++)
            if (want[i] >= done && want[i] < done + rows) { rows_w.push_back((uint32_t)(want[i] - done)); slot_w.push_back(i); }
        for (size_t i = 0; i < rows_w.size();) {
            const uint32_t k = (uint32_t)std::min<size_t>(m->logits_rows_max(), rows_w.size() - i);
            m->enqueue_rows_logits(rows_w.data() + i, k);
            FH_HIP(hipGetLastError());
            FH_HIP(hipMemcpyAsync(m->h_logits, m->logits.p, vocab * 4 * k, hipMemcpyDeviceToHost, s));
            FH_HIP(hipStreamSynchronize(s));
            for (uint32_t j = 0; j < k; j++) memcpy(logits_host + slot_w[i + j] * vocab, m->h_logits + j * vocab, vocab * 4);
            i += k;
        }
        done += rows;
    }
    m->pos += (int64_t)n;
    m->h_stage[2] = (uint32_t)m->pos;
    FH_HIP(hipMemcpyAsync(m->d_pos(), &m->h_stage[2], 4, hipMemcpyHostToDevice, s));
    FH_HIP(hipStreamSynchronize(s));
    return FORGE_HIP_OK;
}

}  // namespace

extern "C" {

const char* forge_hip_last_error(void) { return last_error_cstr(); }

int32_t forge_hip_device_count(void) {
    int n = 0;
    if (hipGetDeviceCount(&n) != hipSuccess) return 0;
    return n;
}

void forge_hip_model_destroy(forge_hip_model* m) {
    if (!m) return;
    if (m->stream) (void)hipStreamSynchronize(m->stream);
    delete m;
}

int32_t forge_hip_forward(forge_hip_model* m, uint32_t token, float* logits_host) {
    FH_CHECK(logits_host, "forward: null logits");
    int32_t rc = forward_common(m, token);
    if (rc) return rc;
    FH_HIP(hipMemcpyAsync(m->h_logits, m->logits.p, (size_t)m->cfg.vocab * 4, hipMemcpyDeviceToHost, m->stream));
    rc = finish_or_undo(m);
    if (rc) return rc;
    memcpy(logits_host, m->h_logits, (size_t)m->cfg.vocab * 4);
    return FORGE_HIP_OK;
}

int32_t forge_hip_forward_greedy(forge_hip_model* m, uint32_t token, uint32_t* next_token_host) {
    FH_CHECK(next_token_host, "forward_greedy: null out");
    int32_t rc = forward_common(m, token);
    if (rc) return rc;
    // the resident kernel hands the token over through host memory as soon as it is final
    if (m->resident() && m->resident_wait_token(next_token_host)) return FORGE_HIP_OK;
    rc = finish_or_undo(m);
    if (rc) return rc;
    *next_token_host = m->h_stage[4];
    return FORGE_HIP_OK;
}

int32_t forge_hip_prefill_batch(forge_hip_model* m, const uint32_t* tokens, uint64_t n, float* logits_host) {
    const uint64_t last = n - 1;
    return prefill_rows(m, tokens, n, &last, logits_host && n ? 1 : 0, logits_host);
}

int32_t forge_hip_prefill_logits(forge_hip_model* m, const uint32_t* tokens, uint64_t n, const uint64_t* want, uint64_t n_want, float* logits_host) {
    FH_CHECK(n_want == 0 || (want && logits_host), "prefill_logits: null pointer");
    return prefill_rows(m, tokens, n, want, n_want, logits_host);
}

int32_t forge_hip_prefill_residuals(forge_hip_model* m, const uint32_t* tokens, uint64_t n, float* out_host) {
    FH_CHECK(m && tokens && out_host, "prefill_residuals: null pointer");
    FH_CHECK(m->pos == 0, "prefill_residuals: the cache must be empty (after create or reset)");
    FH_CHECK(n >= 1 && n <= m->chunk_rows, "prefill_residuals: the tokens must fit one prompt chunk");
    for (uint64_t i = 0; i < n; i++)
        if (tokens[i] >= m->cfg.vocab) return fail(FORGE_HIP_ERR_POSITION, "token id out of range");
    FH_HIP(hipMemcpyAsync(m->ptok.p, tokens, (size_t)n * 4, hipMemcpyHostToDevice, m->stream));
    const int32_t rc = m->prompt_residuals((uint32_t)n, out_host);
    FH_HIP(hipStreamSynchronize(m->stream));
    return rc ? rc : forge_hip_reset(m);
}

uint32_t forge_hip_model_layer_runs(const forge_hip_model* m) { return m ? m->layer_runs() : 0; }

int32_t forge_hip_model_config(const forge_hip_model* m, forge_hip_config* out) {
    FH_CHECK(m && out, "model_config: null pointer");
    *out = m->cfg;
    return FORGE_HIP_OK;
}

int32_t forge_hip_forward_profile(forge_hip_model* m, uint32_t token, float* stage_ms, uint32_t* stage_launches) {
    FH_CHECK(m && stage_ms, "forward_profile: null pointer");
    if (m->pos >= (int64_t)m->cfg.max_seq) return fail(FORGE_HIP_ERR_POSITION, "KV cache is full (pos == max_seq)");
    if (token >= m->cfg.vocab) return fail(FORGE_HIP_ERR_POSITION, "token id out of range");
    if (m->resident()) {
        // one kernel: the stages are its phases, timed by the kernel's own clock stamps
        int32_t rc = m->resident_enqueue(true, token);
        if (rc) return rc;
        rc = finish_decode_step(m);
        if (rc) return rc;
        m->pos += 1;
        return m->resident_profile(stage_ms, stage_launches);
    }
    m->h_stage[0] = token;
    FH_HIP(hipMemcpyAsync(m->d_token(), &m->h_stage[0], 4, hipMemcpyHostToDevice, m->stream));
    {
        ModelProbe probe(m);
        m->enqueue_decode_step();        // eager launches, each carrying its own pair of events
    }
    FH_HIP(hipGetLastError());
    FH_HIP(hipStreamSynchronize(m->stream));
    m->pos += 1;
    return collect_profile(m, stage_ms, stage_launches);
}

int32_t forge_hip_prefill_profile(forge_hip_model* m, const uint32_t* tokens, uint64_t n, float* stage_ms,
                                  uint32_t* stage_launches) {
    FH_CHECK(m && stage_ms, "prefill_profile: null pointer");
    int32_t rc;
    {
        ModelProbe probe(m);
        rc = forge_hip_prefill_batch(m, tokens, n, nullptr);
    }
    if (rc) return rc;
    FH_HIP(hipStreamSynchronize(m->stream));
    return collect_profile(m, stage_ms, stage_launches);
}

int32_t forge_hip_model_decode_launches(const forge_hip_model* m) { return m ? m->decode_launches() : -1; }

int32_t forge_hip_reset(forge_hip_model* m) {
    FH_CHECK(m, "reset: model is null");
    m->pos = 0;
    m->h_stage[2] = 0;
    FH_HIP(hipMemcpyAsync(m->d_pos(), &m->h_stage[2], 4, hipMemcpyHostToDevice, m->stream));
    FH_HIP(hipMemsetAsync(m->counts.p, 0, (size_t)m->cfg.vocab * 4, m->stream));      // recent_tokens starts empty again
    FH_HIP(hipStreamSynchronize(m->stream));
    return FORGE_HIP_OK;
}

int32_t forge_hip_model_set_repeat_penalty(forge_hip_model* m, float penalty) {
    FH_CHECK(m, "set_repeat_penalty: model is null");
    FH_CHECK(penalty == penalty && penalty > 0.0f, "set_repeat_penalty: the penalty must be a positive number");
    if (penalty == m->repeat_penalty) return FORGE_HIP_OK;
    FH_HIP(hipStreamSynchronize(m->stream));
    const int32_t rc = m->repeat_penalty_changed(penalty);
    if (rc) return rc;
    m->repeat_penalty = penalty;
    // the captured kernel sequence carries the old value in its launch arguments: capture again at the next step
    if (m->decode_graph) { (void)hipGraphExecDestroy(m->decode_graph); m->decode_graph = nullptr; }
    return FORGE_HIP_OK;
}

int32_t forge_hip_model_set_poll_limit(forge_hip_model* m, uint32_t polls) {
    FH_CHECK(m, "set_poll_limit: model is null");
    FH_HIP(hipStreamSynchronize(m->stream));
    m->poll_limit_changed(polls);
    return FORGE_HIP_OK;
}

int64_t forge_hip_model_pos(const forge_hip_model* m) { return m ? m->pos : -1; }

int32_t forge_hip_model_set_kv_pages(forge_hip_model* m, uint32_t page_rows, const uint32_t* page_table_host, uint32_t n_pages) {
    FH_CHECK(m, "set_kv_pages: model is null");
    FH_CHECK(m->pos == 0, "set_kv_pages: the cache layout can only change while the cache is empty (after create or reset)");
    FH_HIP(hipStreamSynchronize(m->stream));
    const int32_t rc = m->set_kv_pages(page_rows, page_table_host, n_pages);
    if (rc) return rc;
    // the captured kernel sequence carries the old layout in its launch arguments: capture again at the next step
    if (m->decode_graph) { (void)hipGraphExecDestroy(m->decode_graph); m->decode_graph = nullptr; }
    return FORGE_HIP_OK;
}

int32_t forge_hip_model_read_kv(forge_hip_model* m, uint32_t layer, uint32_t which, uint16_t* out_host) {
    FH_CHECK(m && out_host, "read_kv: null pointer");
    FH_CHECK(layer < m->cfg.layers && which <= 1, "read_kv: layer or selector out of range");
    FH_HIP(hipStreamSynchronize(m->stream));
    return m->read_kv(layer, which, out_host);
}

}  // extern "C"
