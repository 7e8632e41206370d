/*
 * tk_layered.h — decoders described layer by layer (tk_layer_spec.h) behind the shared decoder interface (tk_decoder.h).
 *
 * Model: a folder with config.json and model.safetensors.  At load every product's weights become one operand image (nn/tk_gemm_image.h): all
 * projections that read a layer's input side by side (one launch), the branches' output projections side by side in k (their sum is one
 * product; a branch's scale is applied to its activations), gate and up interleaved, an expert's matrices behind one another.
 *
 * A layer may run another layer's tensors (TkLayerSpec::weights_of): the model holds them once, the session keeps a cache and a state for each.
 *
 * Session: keys and values in pages of 64 positions shared by all sequences (one page table for all layers), recurrent state in two copies per
 * sequence and layer: a pass reads one and writes the other, so the last pass of a sequence can be taken back (the scheduler's run-ahead rows)
 * and nothing is copied.  A pass is any mix of runs of consecutive positions, one run per sequence; each run continues where its sequence
 * stands, or starts at position 0.
 */
#ifndef TK_LAYERED_H
#define TK_LAYERED_H

#include <map>
#include <mutex>
#include <string>
#include <vector>

#include "../nn/tk_gemm_image.h"
#include "tk_decoder.h"
#include "tk_layer_spec.h"
#include "tk_mixer_kernels.h"

/* a weight image; N and K padded */
struct TkMat { void* img = nullptr; int N = 0, K = 0, rows = 0, cols = 0; size_t bytes = 0; };

struct TkLayeredBranch {
    int col = 0;    /* first projection column */
    int out_k0 = 0; /* first k of the output projection */
    /* attention */
    float *bias = nullptr, *q_norm = nullptr, *k_norm = nullptr;
    /* delta rule; the convolution may be attention's too */
    float *conv = nullptr, *a_log = nullptr, *dt_bias = nullptr, *norm = nullptr;
    int rank_a = 0, rank_g = 0, low_a = 0, low_g = 0;
};

struct TkLayeredLayer {
    std::vector<TkLayeredBranch> branches;
    TkMat in, low, out, gate_up, down, router; /* gate_up, down: of all experts when the layer has experts (bytes = one expert's) */
    int low_col = 0, low_cols = 0;             /* projection columns that feed `low` */
    uint64_t bytes = 0;                        /* of the matrices */
    float* out_bias = nullptr;
    TkNorm pre1{}, norm1{}, pre2{}, norm2{}; /* on the sublayers' inputs (w null: none) and outputs */
};

class TkLayeredModel : public TkDecoderModel {
public:
    TkLayeredConfig cfg;
    int type = TK_IMG_BF16; /* element type of weights' and activations' images and of the cache */
    uint16_t* embed = nullptr; /* [vocab][width] bf16 */
    TkMat head;
    TkNorm final_norm{};
    std::vector<TkLayeredLayer> layers;

    ~TkLayeredModel() override;
    /* folder with config.json and model.safetensors; dtype "bfloat16" or "float32" (everything in 32-bit) */
    bool load(const std::string& dir, const std::string& dtype, int device);
    /* random weights of the described shape, made on the device; rank: inner size of the low-rank gates */
    bool fill_synthetic(const std::string& config_json, const std::string& dtype, int device, uint64_t seed, int rank);
    int vocab_size() const override { return cfg.vocab; }
    uint64_t step_weight_bytes() const override { return matrix_bytes_; }
    std::unique_ptr<TkDecodeSession> open_session(int max_seq, int max_ctx, int pool_tokens, std::string* err) override;

private:
    struct Source;
    bool begin(const std::string& config_json, const std::string& dtype, int device);
    bool build(Source& src);
    bool alloc(void** p, size_t bytes);
    bool mat(TkMat* m, int rows, int cols, int copies = 1);
    std::vector<void*> owned_;
    uint64_t matrix_bytes_ = 0;
};

class TkLayeredSession : public TkDecodeSession {
public:
    ~TkLayeredSession() override;
    bool init(TkLayeredModel* m, int max_seq, int max_ctx, int pool_tokens);
    bool forward(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, float* logits_host, int32_t* argmax_host, bool lm_head = true,
                 const uint32_t* const* row_masks = nullptr, const TkSampleRow* row_samp = nullptr, int n_out = 0, const int32_t* out_rows = nullptr) override;
    bool prefill(int nseq, int n_prompt, const int32_t* tokens, int32_t* first_tokens_host) override;
    int row_capacity() const override { return row_cap_; }
    void release_sequence(int seq) override;
    void cache_usage(int* used, int* total) override;
    /* a pass whose residual stream after every layer is copied out: [layers][nrows][width] */
    bool forward_streams(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, float* streams_host);

protected:
    bool begin_decode(int nrows, const int32_t* pos, int n_steps) override;
    void end_decode(int nrows, int steps_done) override;
    hipGraphExec_t* decode_slot(int nrows, int top) override;
    void enqueue_decode(int nrows) override;

private:
    struct Seq { int len = 0, prev = -1, side = 0; std::vector<int32_t> pages; };
    struct Pass { int nrows = 0, nseg = 0, ntiles = 0, nblocks = 0, nsums = 0; bool single = true, singles = true; }; /* all segments, or any, are single rows */
    TkLayeredModel* m_ = nullptr;
    std::mutex mu_; /* seqs_, free_pages_, host page table */
    std::vector<Seq> seqs_;
    std::vector<int32_t> free_pages_, h_pages_;
    bool pages_dirty_ = true;
    int n_pages_ = 0, max_pages_ = 0;
    std::vector<int32_t> live_; /* sequences of rows 0 .. of the last pass decode() may continue from */
    std::vector<void*> owned_;
    int32_t *h_tab_ = nullptr, *d_tab_ = nullptr, *d_pages_ = nullptr, *d_out_rows_ = nullptr, *d_tiles_ = nullptr, *d_blocks_ = nullptr, *d_otok_ = nullptr;
    int ret_heads_ = 0; /* most heads of a retention layer (0: none) */
    int retention_rows(int nrows) const;
    size_t tab_ints_ = 0;
    TkPassTab tab_{};
    float *x_ = nullptr, *proj_ = nullptr, *low_ = nullptr, *y_ = nullptr, *router_ = nullptr, *scratch_ = nullptr;
    float* sums_ = nullptr;
    float *dq_ = nullptr, *dk_ = nullptr, *dv_ = nullptr, *dg_ = nullptr, *db_ = nullptr, *do_ = nullptr;
    void *img_x_ = nullptr, *img_low_ = nullptr, *img_mix_ = nullptr, *img_ff_ = nullptr, *img_gather_ = nullptr, *img_head_ = nullptr, *q_ = nullptr;
    TkMoeTab moe_{};
    struct Rope { float *c, *s; };
    std::map<std::pair<int, double>, Rope> rope_;
    struct BranchState { TkKvPool kv{}; float *conv = nullptr, *state = nullptr, *decay = nullptr; Rope rope{}; int splits_pages = 1; };
    std::vector<std::vector<BranchState>> st_;
    hipGraphExec_t graphs_[TK_MAX_ROWS + 1] = {};
    float* streams_ = nullptr; /* forward_streams(): destination of the layers' streams */

    bool alloc(void** p, size_t bytes, bool zero = false);
    bool rotation(int dims, double base, Rope* out);
    bool describe(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, Pass* p);
    void commit(int nrows, const int32_t* seq, const int32_t* pos);
    void need_pages(Seq& s, int seq, int last_pos);
    void give_back(Seq& s);
    bool upload_pages();
    void gemm(const TkImgGemm& g, int* slabs = nullptr);
    size_t y_floats_ = 0;
    void enqueue_layers(const Pass& p);
    void enqueue_head(int n, const int32_t* d_rows, int32_t* tok, int32_t* pos);
    void enqueue_moe(const TkLayerSpec& s, const TkLayeredLayer& L, int nrows);
    bool run(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, float* logits_host, int32_t* argmax_host, bool head,
             const uint32_t* const* row_masks, const TkSampleRow* row_samp, int n_out, const int32_t* out_rows);
};

#endif
