/* tk_decoder.hip — see tk_decoder.h */
#include "tk_decoder.h"

#include <stdio.h>
#include <stdlib.h>
#include <string.h>

#include <chrono>

#define HIPQ(expr)                                                                              \
    do {                                                                                        \
        hipError_t e__ = (expr);                                                                \
        if (e__ != hipSuccess) {                                                                \
            char b__[256];                                                                      \
            snprintf(b__, sizeof b__, "%s failed: %s (%s:%d)", #expr, hipGetErrorString(e__), __FILE__, __LINE__); \
            error = b__;                                                                        \
            return false;                                                                       \
        }                                                                                       \
    } while (0)

std::mutex& tk_capture_mutex() {
    static std::mutex mu;
    return mu;
}

bool TkDecodeSession::graphs_enabled() {
    /* TK_MI355X_NO_GRAPH=1: eager launches, for profilers that cannot follow hipGraphLaunch */
    const char* ng = getenv("TK_MI355X_NO_GRAPH");
    return !(ng && ng[0] == '1');
}

bool TkDecodeSession::init_tables(int device, int vocab, int row_cap, size_t extra, int32_t** extra_tab) {
    device_ = device;
    vocab_ = vocab;
    row_cap_ = row_cap;
    HIPQ(hipSetDevice(device));
    HIPQ(hipStreamCreateWithFlags(&stream, hipStreamNonBlocking));
    const size_t ints = 3 * (size_t)row_cap + extra;
    HIPQ(hipMalloc((void**)&d_block_, ints * 4));
    HIPQ(hipMemset(d_block_, 0, ints * 4));
    d_seq = d_block_;
    d_pos = d_seq + row_cap;
    d_tok = d_pos + row_cap;
    if (extra_tab) *extra_tab = d_tok + row_cap;
    HIPQ(hipMalloc((void**)&logits, (size_t)TK_MAX_ROWS * vocab * 4));
    HIPQ(hipMalloc((void**)&d_nsteps, TK_MAX_ROWS * 4));
    HIPQ(hipMemset(d_nsteps, 0, TK_MAX_ROWS * 4));
    hist_cap = max_ctx;
    HIPQ(hipMalloc((void**)&d_hist, (size_t)hist_cap * TK_MAX_ROWS * 4));
    HIPQ(hipMalloc((void**)&d_mask, (size_t)TK_MAX_ROWS * (((size_t)vocab + 31) / 32) * 4));
    HIPQ(hipMalloc((void**)&d_mask_row, TK_MAX_ROWS * 4));
    HIPQ(hipMemset(d_mask_row, 0xFF, TK_MAX_ROWS * 4));
    mask_rows_dirty = false;
    HIPQ(hipMalloc((void**)&d_samp, TK_MAX_ROWS * sizeof(TkSampleRow)));
    HIPQ(hipMemset(d_samp, 0, TK_MAX_ROWS * sizeof(TkSampleRow))); /* temp 0: every row samples greedily */
    samp_dirty = false;
    return true;
}

TkDecodeSession::~TkDecodeSession() {
    if (!stream && !d_block_) return;
    (void)hipSetDevice(device_);
    void* ptrs[] = {d_block_, logits, d_nsteps, d_hist, d_mask, d_mask_row, d_samp};
    for (void* p : ptrs) if (p) (void)hipFree(p);
    if (stream) (void)hipStreamDestroy(stream);
}

bool TkDecodeSession::reset() {
    HIPQ(hipSetDevice(device_));
    HIPQ(hipMemsetAsync(d_nsteps, 0, TK_MAX_ROWS * 4, stream));
    HIPQ(hipStreamSynchronize(stream));
    return true;
}

bool TkDecodeSession::rows_in_range(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok) {
    for (int r = 0; r < nrows; ++r)
        if (seq[r] < 0 || seq[r] >= max_seq || pos[r] < 0 || pos[r] >= max_ctx || tok[r] < 0 || tok[r] >= vocab_) {
            error = "row out of range (sequence id, position or token id)";
            return false;
        }
    return true;
}

bool TkDecodeSession::stage_sampling(int n, const int32_t* rows, const uint32_t* const* row_masks, const TkSampleRow* row_samp) {
    /* per-row sampling masks: the masks of the constrained rows, compacted, + the row -> mask table the arg max kernel reads */
    int32_t rowtab[TK_MAX_ROWS];
    int nmask = 0;
    const size_t words = ((size_t)vocab_ + 31) / 32;
    for (int r = 0; r < TK_MAX_ROWS; ++r) rowtab[r] = -1;
    for (int i = 0; i < n; ++i) {
        const int r = rows ? rows[i] : i;
        if (row_masks && row_masks[r]) {
            HIPQ(hipMemcpyAsync(d_mask + (size_t)nmask * words, row_masks[r], words * 4, hipMemcpyHostToDevice, stream));
            rowtab[i] = nmask++;
        }
    }
    if (nmask > 0 || mask_rows_dirty) {
        HIPQ(hipMemcpyAsync(d_mask_row, rowtab, TK_MAX_ROWS * 4, hipMemcpyHostToDevice, stream)); /* whole table (a wider pass may have left entries); pageable source: staged before the call returns */
        mask_rows_dirty = nmask > 0;
    }
    /* per-row sampling state (temp <= 0: greedy): data of the pass like the masks, so sampled and greedy rows share passes and graphs */
    bool any_samp = false;
    for (int i = 0; i < n && row_samp; ++i) any_samp = any_samp || row_samp[rows ? rows[i] : i].temp > 0.0f;
    if (any_samp) {
        if (vocab_ > 65536) { error = "stochastic sampling supports vocabularies of at most 65536 tokens"; return false; }
        TkSampleRow tab[TK_MAX_ROWS] = {};
        for (int i = 0; i < n; ++i) tab[i] = row_samp[rows ? rows[i] : i];
        HIPQ(hipMemcpyAsync(d_samp, tab, sizeof tab, hipMemcpyHostToDevice, stream));
        samp_dirty = true;
    } else if (samp_dirty) {
        HIPQ(hipMemsetAsync(d_samp, 0, TK_MAX_ROWS * sizeof(TkSampleRow), stream));
        samp_dirty = false;
    }
    return true;
}

bool TkDecodeSession::capture(hipGraphExec_t* slot, const std::function<void()>& enqueue) {
    if (*slot) return true;
    const auto t_cap = std::chrono::steady_clock::now();
    struct Tally { TkDecodeSession* s; std::chrono::steady_clock::time_point t0; ~Tally() { s->n_captures++; s->capture_ms += std::chrono::duration<double, std::milli>(std::chrono::steady_clock::now() - t0).count(); } } tally{this, t_cap};
    std::lock_guard<std::mutex> lk(tk_capture_mutex());
    hipGraph_t g = nullptr;
    HIPQ(hipStreamBeginCapture(stream, hipStreamCaptureModeRelaxed));
    launch_error.clear();
    enqueue();
    /* from here on the stream must leave capture mode and the graph must be freed whatever fails */
    const hipError_t e_end = hipStreamEndCapture(stream, &g);
    hipError_t e_inst = hipSuccess;
    if (e_end == hipSuccess && launch_error.empty()) e_inst = hipGraphInstantiate(slot, g, nullptr, nullptr, 0);
    if (g) (void)hipGraphDestroy(g);
    if (e_end != hipSuccess || e_inst != hipSuccess || !launch_error.empty()) {
        if (*slot && e_inst != hipSuccess) { (void)hipGraphExecDestroy(*slot); }
        *slot = nullptr;
        (void)hipGetLastError();
        error = !launch_error.empty() ? launch_error
                : std::string("graph capture of a pass failed: ") + hipGetErrorString(e_end != hipSuccess ? e_end : e_inst);
        return false;
    }
    return true;
}

bool TkDecodeSession::decode(int nrows, int n_steps, int32_t* out_tokens_host) {
    if (nrows <= 0 || nrows > TK_MAX_ROWS) { error = "nrows must be in [1,256]"; return false; }
    if (n_steps <= 0 || n_steps > hist_cap) { error = "n_steps exceeds the session context"; return false; }
    HIPQ(hipSetDevice(device_));
    /* positions must stay inside the cache for the whole loop */
    int32_t hpos[TK_MAX_ROWS];
    HIPQ(hipMemcpyAsync(hpos, d_pos, nrows * 4, hipMemcpyDeviceToHost, stream));
    HIPQ(hipStreamSynchronize(stream));
    for (int r = 0; r < nrows; ++r)
        if (hpos[r] + n_steps > max_ctx) { error = "decode would run past max_ctx"; return false; }
    if (!begin_decode(nrows, hpos, n_steps)) return false;
    const bool use_graph = graphs_enabled();
    int top0 = 0;
    for (int r = 0; r < nrows; ++r) top0 = hpos[r] > top0 ? hpos[r] : top0;
    HIPQ(hipMemsetAsync(d_nsteps, 0, TK_MAX_ROWS * 4, stream));
    if (mask_rows_dirty) { HIPQ(hipMemsetAsync(d_mask_row, 0xFF, TK_MAX_ROWS * 4, stream)); mask_rows_dirty = false; } /* the loop samples unconstrained */
    hipEvent_t e0, e1;
    HIPQ(hipEventCreate(&e0));
    HIPQ(hipEventCreate(&e1));
    HIPQ(hipEventRecord(e0, stream));
    int done = 0;
    bool ok = true;
    launch_error.clear();
    for (; done < n_steps && ok; ++done) {
        hipGraphExec_t* slot = decode_slot(nrows, top0 + done); /* positions advance on the device; the host knows where the loop stands */
        if (use_graph) {
            ok = capture(slot, [&] { enqueue_decode(nrows); });
            if (ok && hipGraphLaunch(*slot, stream) != hipSuccess) { error = "graph launch of a decode step failed"; ok = false; }
        } else {
            enqueue_decode(nrows);
            if (!launch_error.empty()) { error = launch_error; ok = false; }
        }
        if (!ok) break;
    }
    end_decode(nrows, done);
    launch_error.clear();
    if (!ok) { (void)hipStreamSynchronize(stream); (void)hipEventDestroy(e0); (void)hipEventDestroy(e1); return false; }
    HIPQ(hipGetLastError());
    HIPQ(hipEventRecord(e1, stream));
    if (out_tokens_host) HIPQ(hipMemcpyAsync(out_tokens_host, d_hist, (size_t)n_steps * TK_MAX_ROWS * 4, hipMemcpyDeviceToHost, stream));
    HIPQ(hipStreamSynchronize(stream));
    float ms = 0.0f;
    HIPQ(hipEventElapsedTime(&ms, e0, e1));
    last_step_ms = ms / n_steps;
    (void)hipEventDestroy(e0);
    (void)hipEventDestroy(e1);
    return true;
}
