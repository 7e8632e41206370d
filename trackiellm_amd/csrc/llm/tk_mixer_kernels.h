/*
 * tk_mixer_kernels.h — launch wrappers of the layer-list decoders' kernels (tk_layered.h): paged attention with a sliding window and kept first
 * positions, or with chunks, the gated delta rule and retention, short convolutions, norms around the residual stream, the grouped sigmoid router.
 * Sizes and constants are arguments throughout.  Wrappers only enqueue on `s`.
 *
 * Activations that feed a matrix product are operand images (nn/tk_gemm_image.h) of the session's element type; everything else — projections'
 * results, the residual stream, gates, decays, recurrent state — is f32.
 */
#ifndef TK_MIXER_KERNELS_H
#define TK_MIXER_KERNELS_H

#include <hip/hip_runtime.h>
#include <stdint.h>

#include "../nn/tk_gemm_image.h"
#include "tk_layer_spec.h"

#define TK_PAGE 64 /* positions of a cache page */

/* device tables of one pass.  A segment is a run of consecutive rows that hold consecutive positions of one sequence. */
struct TkPassTab {
    const int32_t *seq, *pos, *tok; /* [rows] */
    const int32_t* seg;             /* [rows] */
    const int32_t *seg_row0, *seg_n; /* [segments] */
    int32_t *seg_in, *seg_out;      /* [segments] state copies read (-1: the sequence starts here) and written; never the same copy */
    const int32_t* page_of;         /* [sequences][max_pages] page ids */
    int max_pages;
};

/* keys [page][kv head][TK_PAGE][dim_pad], values transposed [page][kv head][vdim_pad][TK_PAGE]; dim_pad = image k padding, vdim_pad = 16s */
struct TkKvPool { void *k, *v; int dim_pad, vdim_pad; };

struct TkAttnArgs {
    int heads, kv_heads, dim, vdim, rot_dims, window, keep_first, chunk;
    float scale, softcap, out_scale, eps;
    int col;                          /* first column of q | k | v in the projections */
    int taps;                         /* > 0: a causal convolution on every channel of q | k | v, before the rotation (no biases and norms then) */
    const float* conv;                /* [channels][taps] */
    float* conv_state;                /* [copies][channels][taps - 1] */
    const float *bias;                /* q | k | v biases or null */
    const float *q_norm, *k_norm;     /* null: no norm */
    const float *rope_cos, *rope_sin; /* [max_ctx][rot_dims / 2] */
    void* q;                          /* [rows][heads][dim_pad] */
    TkKvPool kv;
    void* out_img;                    /* next product's image; head h at k = out_k0 + h * vdim */
    int out_k0, out_ktiles;
};

struct TkDeltaArgs {
    int heads, kv_heads, dim, vdim, taps;
    float out_scale, eps, unit_eps;
    int col;                          /* first column of q | k | v | b in the projections */
    const float *conv;                /* [2 kv_heads dim + heads vdim][taps] */
    const float *a_log, *dt_bias, *norm;
    const float* low;                 /* [rows][low_ld]: decay inputs (heads x dim) from column low_a on, gate inputs (heads x vdim) from low_g */
    int low_ld, low_a, low_g;
    float *q, *k, *v, *g, *beta, *o;  /* [rows][kv_heads dim], same, [rows][heads vdim], [rows][heads dim], [rows][heads], [rows][heads vdim] */
    float* conv_state;                /* [copies][channels][taps - 1] */
    float* state;                     /* [copies][heads][dim][vdim padded to 4] */
    void* out_img;
    int out_k0, out_ktiles;
};

/* linear attention with one constant decay per head: S <- decay S + k v^T, o = S^T q; q and k rotated, k times dim^-1/2; o over its root mean square,
 * times silu(gate) */
#define TK_RETENTION_BLOCK 64 /* rows of a scan's blocks are multiples of this */
struct TkRetentionArgs {
    int heads, dim, vdim, rot_dims;
    float out_scale, eps;
    int col;                          /* first column of q | k | v | gate in the projections */
    const float *rope_cos, *rope_sin; /* [max_ctx][rot_dims / 2] */
    const float* decay;               /* [heads][TK_RETENTION_BLOCK + 1] powers 0 .. TK_RETENTION_BLOCK */
    float* state;                     /* [copies][heads][dim][vdim padded to 4] */
    float* sums;                      /* [slots][heads][dim][vdim padded to 4] what a block of rows adds to the state */
    void* out_img;
    int out_k0, out_ktiles;
};

/* a norm's tensors; w null: no norm.  layer: mean taken off, b added; otherwise over the root mean square */
struct TkNorm { const float *w, *b; int layer; };

/* x = table[tok] * scale; the image of next(x) */
void tk_launch_layer_embed(int type, const uint16_t* table, int width, float scale, const int32_t* tok, int nrows, float* x, const TkNorm& next, float eps, void* img, int ktiles, hipStream_t s);

/* everything between the projections and the mixers: biases, per-head norms, rotation, cache append; convolutions, unit norms, decays, step sizes */
void tk_launch_mixer_prep(int type, const float* proj, int ld, const TkAttnArgs* attn, const TkDeltaArgs* delta, const TkPassTab& t, int nrows, hipStream_t s);

/* tiles: [2 * n_tiles] = first row, rows (<= 64) of a run of consecutive positions; every head of every tile is one workgroup */
void tk_launch_attn_tiles(int type, const TkAttnArgs& a, const TkPassTab& t, const int32_t* tiles, int n_tiles, hipStream_t s);
/* one row at a time (decoding): `splits` workgroups per (row, group of query heads) share the row's pages; scratch for splits > 1 */
void tk_launch_attn_rows(int type, const TkAttnArgs& a, const TkPassTab& t, int nrows, int splits, float* scratch, hipStream_t s);
int tk_attn_rows_splits(const TkAttnArgs& a, int pages, int nrows); /* for at most `pages` visible pages */
size_t tk_attn_rows_scratch_floats(const TkAttnArgs& a, int nrows, int splits);

/* the recurrence over every segment, token by token, and the gated per-head norm of its output */
void tk_launch_delta_scan(int type, const TkDeltaArgs& d, const TkPassTab& t, int n_segments, int nrows, hipStream_t s);
/* the same for passes whose segments are single rows: one launch */
void tk_launch_delta_step(int type, const TkDeltaArgs& d, const TkPassTab& t, int nrows, hipStream_t s);

/* blocks: [n_blocks] runs of rows of one segment; every block but a segment's last has the same number of rows, a multiple of TK_RETENTION_BLOCK.
 * n_sums: how many of them are followed by another block of their segment (their own share of the state goes through args.sums) */
struct TkRetentionBlock { int32_t row0, n, seg, slot0, index, last; }; /* slot0: of the segment's first block in args.sums; index: of the block in its segment */
void tk_launch_retention_scan(int type, const TkRetentionArgs& d, const float* proj, int ld, const TkPassTab& t, const TkRetentionBlock* blocks, int n_blocks, int n_sums, hipStream_t s);
/* the segments that are single rows (others are left alone) */
void tk_launch_retention_step(int type, const TkRetentionArgs& d, const float* proj, int ld, const TkPassTab& t, int n_segments, hipStream_t s);

/* tk_launch_attn_rows and tk_launch_delta_step in one launch, side by side; false (nothing launched): sizes it has no form for */
bool tk_launch_mixers_step(int type, const TkAttnArgs& a, const TkDeltaArgs& d, const TkPassTab& t, int nrows, hipStream_t s);

/* where a sublayer's output comes from: a product's rows, or the chosen experts' rows, weighted */
struct TkSubOut {
    const float* y; int ld;
    int slabs; size_t slab_floats; /* partial results of a product split over k, added in order (1: whole) */
    const float* bias; float bias_scale; /* bias may be null */
    const int32_t* slot; const float* weight; int top; /* top > 0: y[slot[row * top + j]] * weight[row * top + j] summed over j */
};
/* x += norm(output); the image of next(x), the next sublayer's input */
void tk_launch_post_norm(int type, const TkSubOut& o, const TkNorm& norm, const TkNorm& next, float eps, int width, int nrows, float* x, void* img, int ktiles, hipStream_t s);
/* norm of the listed rows (null: rows 0 .. n - 1) as an image */
void tk_launch_rows_norm(int type, const float* x, const int32_t* rows, int n, const TkNorm& norm, float eps, int width, void* img, int ktiles, hipStream_t s);

struct TkMoeTab {
    int32_t* count;      /* [experts], zero between passes */
    int32_t* expert;     /* [rows * top] */
    int32_t* rank;       /* [rows * top] place among the expert's rows */
    float* weight;       /* [rows * top] */
    int32_t* tile0;      /* [experts] first 16-row tile */
    int32_t* slot;       /* [rows * top] row in the gathered image */
    TkImgBlock* blocks;
    int32_t* n_blocks;
};
/* router logits -> chosen experts, weights, ranks, first tiles and row blocks of at most block_tiles tiles */
void tk_launch_moe_select(const float* logits, int ld, int experts, int top, int groups, int keep, int nrows, int block_tiles, const TkMoeTab& t, hipStream_t s);
void tk_launch_moe_gather(const void* img, void* gathered, int ktiles, int top, int nrows, const TkMoeTab& t, hipStream_t s);

/* end of a pass in a device-driven loop: every single-row segment reads next what it has just written */
void tk_launch_swap_state(const TkPassTab& t, int n, hipStream_t s);

/* LDS opt-in on the current device; nullptr or an error string */
const char* tk_mixer_prepare_device();

#endif
