/*
 * tk_decoder.h — what every decoder of the library shares behind the runner API: a model that opens sessions, and a session that runs passes of
 * (sequence, position, token) rows.  The base owns what does not depend on the architecture — the stream, the row tables, the sampling tables and
 * the token history, the device-driven decode loop, hipGraph capture — and the scheduler (tk_llm_batcher.h) and the C-ABI drive this interface.
 *   TkLlmModel / TkLlmSession       GGUF Mistral-class checkpoints (tk_llm_engine.h)
 *   TkLayeredModel / TkLayeredSession   decoders described layer by layer in config.json (tk_layered.h)
 */
#ifndef TK_DECODER_H
#define TK_DECODER_H

#include <hip/hip_runtime.h>
#include <stdint.h>

#include <functional>
#include <memory>
#include <string>

#include "../common/tk_sample.h"
#include "tk_llm_layout.h"

class TkDecodeSession;

class TkDecoderModel {
public:
    int device = 0;
    std::string error;
    virtual ~TkDecoderModel() {}
    virtual int vocab_size() const = 0;
    /* matrix bytes a decode step streams */
    virtual uint64_t step_weight_bytes() const = 0;
    /* max_seq sequences of at most max_ctx positions; pool_tokens: positions all live sequences hold together (0: max_seq x max_ctx; models whose
     * cache is not paged take it as a promise only).  null with *err on failure */
    virtual std::unique_ptr<TkDecodeSession> open_session(int max_seq, int max_ctx, int pool_tokens, std::string* err) = 0;
};

class TkDecodeSession {
public:
    int max_seq = 0, max_ctx = 0;
    std::string error;
    hipStream_t stream = nullptr;
    /* average ms of one step of the last decode(), HIP events */
    float last_step_ms = 0.0f;
    uint64_t n_captures = 0; /* passes recorded into a graph so far, and the host time that took (diagnostics: TK_MI355X_BATCHER_TRACE) */
    double capture_ms = 0.0;

    virtual ~TkDecodeSession();
    /* one pass; host arrays.  row_masks (optional): row_masks[r] = nullptr or the (vocab + 31) / 32 words whose bit t says token t may be
     * sampled for row r: grammar-constrained greedy sampling, per row, so constrained and unconstrained rows share passes (and the captured
     * graphs).  row_samp (optional): [nrows] sampling state, temp > 0 = the default stochastic chain for that row, else greedy.
     * out_rows (optional): the n_out rows, ascending, whose logits / ids are wanted; logits_host and argmax_host then hold n_out entries in that
     * order.  Without it every row is wanted. */
    virtual bool forward(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, float* logits_host, int32_t* argmax_host, bool lm_head = true,
                         const uint32_t* const* row_masks = nullptr, const TkSampleRow* row_samp = nullptr, int n_out = 0, const int32_t* out_rows = nullptr) = 0;
    /* prompts of equal length for sequences 0..nseq-1 (tokens[nseq][n_prompt]); leaves row r = sequence r holding the first sampled token so
     * decode() can follow; first_tokens_host[nseq] optional */
    virtual bool prefill(int nseq, int n_prompt, const int32_t* tokens, int32_t* first_tokens_host) = 0;
    /* greedy decode loop, on-device feedback, hipGraph replay.  Starts from the rows' current (tok, pos) state left by the previous
     * forward()/decode(); out_tokens[n_steps][TK_MAX_ROWS]. */
    bool decode(int nrows, int n_steps, int32_t* out_tokens_host);
    bool reset();
    /* rows one forward() takes */
    virtual int row_capacity() const { return TK_MAX_ROWS; }
    /* what a sequence holds in the cache is given back.  Thread-safe against the thread that runs passes. */
    virtual void release_sequence(int seq) { (void)seq; }
    /* (pages in use, pages) of a paged cache, (0, 0) otherwise */
    virtual void cache_usage(int* used, int* total) { *used = *total = 0; }

protected:
    int device_ = 0, vocab_ = 0, row_cap_ = 0;
    int32_t *d_seq = nullptr, *d_pos = nullptr, *d_tok = nullptr, *d_nsteps = nullptr, *d_hist = nullptr;
    float* logits = nullptr;        /* [TK_MAX_ROWS][vocab] */
    uint32_t* d_mask = nullptr;     /* [TK_MAX_ROWS][(vocab + 31) / 32] allowed-token bits of the masked rows of the current pass */
    int32_t* d_mask_row = nullptr;  /* [TK_MAX_ROWS] index into d_mask, -1 = the row samples unconstrained */
    bool mask_rows_dirty = true;    /* d_mask_row holds something other than all -1 */
    TkSampleRow* d_samp = nullptr;  /* [TK_MAX_ROWS] sampling state of the rows of the current pass (temp 0 = greedy); decode() continues from it */
    bool samp_dirty = false;        /* d_samp holds a stochastic row */
    int hist_cap = 0;
    std::string launch_error; /* set by enqueue functions when a launcher refuses its arguments (no HIP error is raised for that) */

    /* stream, row tables for row_cap rows followed by `extra` ints (returned in *extra_tab), sampling tables, history of max_ctx steps */
    bool init_tables(int device, int vocab, int row_cap, size_t extra, int32_t** extra_tab);
    /* sampling tables of a pass that samples rows[0 .. n): masks and states are indexed by the pass's rows */
    bool stage_sampling(int n, const int32_t* rows, const uint32_t* const* row_masks, const TkSampleRow* row_samp);
    /* records what `enqueue` launches into *slot (kept when it is there already) */
    bool capture(hipGraphExec_t* slot, const std::function<void()>& enqueue);
    static bool graphs_enabled();
    bool rows_in_range(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok);

    /* hooks of decode(): before the loop (host positions of the rows), then per step, `top` = the step's highest position: the graph slot the step
     * replays, and the launches it consists of */
    virtual bool begin_decode(int nrows, const int32_t* pos, int n_steps) { (void)nrows; (void)pos; (void)n_steps; return true; }
    virtual void end_decode(int nrows, int steps_done) { (void)nrows; (void)steps_done; }
    virtual hipGraphExec_t* decode_slot(int nrows, int top) = 0;
    virtual void enqueue_decode(int nrows) = 0;

private:
    int32_t* d_block_ = nullptr;
};

/* capture is one at a time per process: other host threads keep calling allocation and copy APIs meanwhile (relaxed mode) */
#include <mutex>
std::mutex& tk_capture_mutex();

#endif
