/*
 * tk_gemm_image.h — C[rows][N] = A[rows][K] x W[N][K]^T with both operands held as "operand images": the element order in which one 16-byte
 * load per lane IS a matrix-core operand, so neither operand is ever shuffled on its way to the MFMA.
 *
 *   Image of a matrix [R][K], element type T (bf16 or f32): tiles of 16 rows x KT k (KT = 32 for bf16, 16 for f32), 1 KiB each, tiles of one
 *   16-row group contiguous over k.  Inside a tile lane l = (r = l % 16, g = l / 16) owns 16 bytes: k = KT * tile + (KT / 4) * g + 0 ..
 *   KT/4 - 1 of row r.  K is padded to a multiple of 2 KT with zeros, R to a multiple of 16.
 *
 *   bf16: one v_mfma_f32_16x16x32_bf16 per tile pair.  f32: four v_mfma_f32_16x16x4_f32 (true 32-bit products and sums; the four k of one
 *   instruction are element t of the four lane groups on both sides, an order of the same sum).
 *
 * Two kernels: a skinny one (up to 64 rows per block: the waves of a workgroup split K and stream the weights once from HBM to registers) and a
 * wide one (128 rows x 32 .. 128 columns per workgroup, both operands through a double-buffered LDS image filled by LDS-DMA).  Either can take
 * its row blocks from a table that names a weight matrix per block (mixture of experts: one launch over all experts).
 */
#ifndef TK_GEMM_IMAGE_H
#define TK_GEMM_IMAGE_H

#include <hip/hip_runtime.h>
#include <stdint.h>

enum TkImgType { TK_IMG_BF16 = 0, TK_IMG_F32 = 1 };

static inline int tk_img_kt(int type) { return type == TK_IMG_F32 ? 16 : 32; }
/* k of the padded image */
static inline int tk_img_pad_k(int type, int K) { const int m = 2 * tk_img_kt(type); return (K + m - 1) / m * m; }
static inline size_t tk_img_bytes(int type, int64_t rows, int K) {
    return (size_t)((rows + 15) / 16) * (size_t)(tk_img_pad_k(type, K) / tk_img_kt(type)) * 1024;
}

/* row blocks of a grouped launch: {weight matrix, first 16-row tile of A, tiles in this block, 0} */
struct TkImgBlock { int32_t group, tile0, ntiles, pad; };

struct TkImgGemm {
    int type;            /* TkImgType of both operands */
    const void* w;       /* image [N][K] */
    const void* a;       /* image [rows][K]; allocated for rows rounded up to 128 */
    int K;               /* padded */
    int N;               /* rows of the weight image, padded to 16 (32 with swiglu) */
    int nrows;           /* rows of A (grouped: unused) */
    /* f32 output: out[row][n], n < n_valid; columns [copy0, copy1) are also written, as T, to the image copy_img at k = n - copy0 */
    float* out;
    int ldc, n_valid;
    /* K-split (wide kernel, f32 output without copied columns): up to max_slabs partial results, slab i at out + i * slab_floats, which the
     * consumer adds in ascending order; the launcher reports how many it wrote.  0 / 1: none. */
    int max_slabs;
    size_t slab_floats;
    void* copy_img;
    int copy0, copy1, copy_ktiles;
    /* swiglu: the weight image alternates 16 gate rows and 16 up rows; silu(gate) * up goes, as T, to the image act_img [rows][N / 2].
     * act_clamped: g = min(gate, limit), u = clamp(up, -limit, limit), then g * sigmoid(act_slope * g) * (u + act_shift) instead */
    int swiglu, act_clamped;
    float act_limit, act_slope, act_shift;
    void* act_img;
    int act_ktiles, act_valid; /* columns >= act_valid are not stored */
    /* grouped: row blocks from a device table of at most max_blocks entries, *n_blocks of them live; block_tiles = the largest ntiles (<= 8) */
    const TkImgBlock* blocks;
    const int32_t* n_blocks;
    int max_blocks, block_tiles;
    size_t group_bytes;  /* between the weight images of two groups */
};

/* nullptr, or why the arguments are refused (nothing is launched then) */
const char* tk_launch_gemm_image(const TkImgGemm& g, hipStream_t s, int* slabs = nullptr);

/* opts the kernels into their dynamic LDS on the calling thread's current device; nullptr or an error string.  Idempotent, thread-safe. */
const char* tk_gemm_image_prepare_device();

/* src: row-major [N][K] (device), bf16 (src_f32 = 0) or f32 -> rows n0 .. and columns k0 .. of an image with `ktiles` k tiles.  Row n of the
 * source lands in row  (n0 + n) of the image, or, with interleave = 0 or 1, in 16-row group 2 * (n / 16) + interleave (gate / up). */
void tk_launch_put_image(int type, const void* src, int src_f32, int64_t N, int64_t K, void* img, int ktiles, int64_t n0, int64_t k0, int interleave, hipStream_t s);

#endif
