/* tk_gemm_image.hip — see tk_gemm_image.h */
#include "tk_gemm_image.h"

#include <atomic>
#include <mutex>

#include "tk_image_device.h"

namespace {

__device__ __forceinline__ tk_v4u ldg16(const uint8_t* p) { return *(const tk_v4u*)p; }
__device__ __forceinline__ tk_v4u ldg16_stream(const uint8_t* p) { return __builtin_nontemporal_load((const tk_v4u*)p); }

/* one accumulator tile (lane: row = l % 16 of the M-tile, columns n .. n + 3) to its f32 destination */
template <typename T>
__device__ __forceinline__ void store_f32(const TkImgGemm& a, int64_t row, int n, tk_v4f v) {
    float* o = a.out + row * a.ldc + n;
    if (n + 3 < a.n_valid && (a.ldc & 3) == 0) *(tk_v4f*)o = v;
    else
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (n + r < a.n_valid) o[r] = v[r];
    if (a.copy_img && n + 3 >= a.copy0 && n < a.copy1)
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (n + r >= a.copy0 && n + r < a.copy1) tk_img_put((T*)a.copy_img, row, n + r - a.copy0, a.copy_ktiles, v[r]);
}

/* gate and up tiles of the same 16 columns -> the gated activation in the next product's operand image */
template <typename T>
__device__ __forceinline__ void store_act(const TkImgGemm& a, int64_t row, int n, tk_v4f gate, tk_v4f up) {
    tk_v4f h;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        float y;
        if (a.act_clamped) {
            const float g = fminf(gate[r], a.act_limit), u = fminf(fmaxf(up[r], -a.act_limit), a.act_limit);
            y = g * tk_sigmoid32(a.act_slope * g) * (u + a.act_shift);
        } else {
            y = tk_silu32(gate[r]) * up[r];
        }
        h[r] = n + r < a.act_valid ? y : 0.0f;
    }
    if (n < a.act_valid) tk_img_put4((T*)a.act_img, row, n, a.act_ktiles, h);
}

/* ---- skinny: MT M-tiles of rows, NT column tiles per workgroup, K interleaved over the waves in pieces of U tiles ---- */
template <typename T, int MT, int NT, int WAVES, bool SWIGLU, bool GROUPED>
__global__ __launch_bounds__(64 * WAVES) void k_gemm_skinny(TkImgGemm a) {
    constexpr int U = MT >= 4 ? 2 : 4;
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int ktiles = a.K / TkImg<T>::KT;
    int m0 = blockIdx.y * MT, mlive = (a.nrows + 15) / 16 - m0;
    const uint8_t* wbase = (const uint8_t*)a.w;
    if (GROUPED) {
        if ((int)blockIdx.y >= *a.n_blocks) return;
        const TkImgBlock b = a.blocks[blockIdx.y];
        m0 = b.tile0; mlive = b.ntiles;
        wbase += (size_t)b.group * a.group_bytes;
    }
    if (mlive > MT) mlive = MT;
    const int ntot = a.N / 16, n0 = blockIdx.x * NT;
    const uint8_t* wp[NT];
    const uint8_t* ap[MT];
#pragma unroll
    for (int n = 0; n < NT; ++n) wp[n] = wbase + (size_t)(n0 + n < ntot ? n0 + n : ntot - 1) * ktiles * 1024 + lane * 16;
#pragma unroll
    for (int m = 0; m < MT; ++m) ap[m] = (const uint8_t*)a.a + (size_t)(m0 + (m < mlive ? m : 0)) * ktiles * 1024 + lane * 16;
    tk_v4f acc[NT][MT];
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < MT; ++m) acc[n][m] = tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
    const tk_v4u zero = {0, 0, 0, 0};
    tk_v4u wq[U][NT], aq[U][MT];
    /* tiles past the end re-read the last one against a zero activation: no branch around a load */
    auto load = [&](int c) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int kt = c + u < ktiles ? c + u : ktiles - 1;
#pragma unroll
            for (int n = 0; n < NT; ++n) wq[u][n] = ldg16_stream(wp[n] + (size_t)kt * 1024);
#pragma unroll
            for (int m = 0; m < MT; ++m) aq[u][m] = ldg16(ap[m] + (size_t)kt * 1024);
        }
    };
    int c = wave * U;
    if (c < ktiles) load(c);
    while (c < ktiles) {
        tk_v4u w0[U][NT], a0[U][MT];
#pragma unroll
        for (int u = 0; u < U; ++u) {
#pragma unroll
            for (int n = 0; n < NT; ++n) w0[u][n] = wq[u][n];
#pragma unroll
            for (int m = 0; m < MT; ++m) a0[u][m] = c + u < ktiles ? aq[u][m] : zero;
        }
        const int next = c + WAVES * U;
        if (next < ktiles) load(next);
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int n = 0; n < NT; ++n)
#pragma unroll
                for (int m = 0; m < MT; ++m) acc[n][m] = TkImg<T>::mma(w0[u][n], a0[u][m], acc[n][m]);
        c = next;
    }
    /* partial sums of the waves, ascending */
    tk_v4f* red = (tk_v4f*)lds;
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < MT; ++m) red[((wave * NT + n) * MT + m) * 64 + lane] = acc[n][m];
    __syncthreads();
    auto total = [&](int n, int m) {
        tk_v4f s = red[(n * MT + m) * 64 + lane];
        for (int w = 1; w < WAVES; ++w) s += red[((w * NT + n) * MT + m) * 64 + lane];
        return s;
    };
    constexpr int UNITS = SWIGLU ? NT / 2 * MT : NT * MT;
    for (int i = wave; i < UNITS; i += WAVES) {
        const int n = i / MT, m = i % MT;
        const int64_t row = (int64_t)(m0 + m) * 16 + (lane & 15);
        if (m >= mlive || (!GROUPED && row >= a.nrows)) continue;
        if (SWIGLU) {
            if (n0 + 2 * n < ntot) store_act<T>(a, row, (n0 / 2 + n) * 16 + 4 * (lane >> 4), total(2 * n, m), total(2 * n + 1, m));
        } else if (n0 + n < ntot) {
            store_f32<T>(a, row, (n0 + n) * 16 + 4 * (lane >> 4), total(n, m));
        }
    }
}

/* s_waitcnt vmcnt(N): all but this wave's N youngest vector-memory requests are done */
template <int N> __device__ __forceinline__ void wait_vm() { __builtin_amdgcn_s_waitcnt(0x0F70 | (N & 15) | (N >> 4) << 14); }

/* ---- wide: 128 rows x 16 * NBT columns per workgroup, waves 2 x 2, two k tiles per stage, a ring of LDS stages filled by LDS-DMA ---- */
template <int NBT> constexpr int wide_ring() { return NBT == 8 ? 2 : NBT == 4 ? 3 : 4; } /* stages: as many as let two workgroups share a CU */
template <typename T, int NBT /* column tiles of the workgroup: 2, 4, 8 */, bool SWIGLU, bool GROUPED>
__global__ __launch_bounds__(256) void k_gemm_wide(TkImgGemm a, int nblk_n, int nblk_m, int ks) {
    constexpr int MBT = 8, NW = NBT / 2, MW = MBT / 2; /* tiles of one wave */
    constexpr int STAGE = (MBT + NBT) * 2 * 1024, RING = wide_ring<NBT>();
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    /* workgroups go to the eight XCDs in turn: give each XCD a contiguous range of blocks (row blocks fastest) so that it re-reads the same
     * columns of W from its own L2 */
    int id = blockIdx.x;
    const int total = nblk_n * nblk_m * ks;
    {
        const int per = total / 8, rem = total % 8, x = id % 8, i = id / 8;
        id = x * per + (x < rem ? x : rem) + i;
    }
    const int slab = id / (nblk_n * nblk_m), bn = id / nblk_m % nblk_n, bm = id % nblk_m;
    const int ktiles = a.K / TkImg<T>::KT, s0 = (int)((int64_t)(ktiles / 2) * slab / ks), stages = (int)((int64_t)(ktiles / 2) * (slab + 1) / ks) - s0;
    a.out += slab * a.slab_floats;
    int m0 = bm * MBT, mlive = (a.nrows + 15) / 16 - m0;
    const uint8_t* wbase = (const uint8_t*)a.w;
    if (GROUPED) {
        if (bm >= *a.n_blocks) return;
        const TkImgBlock b = a.blocks[bm];
        m0 = b.tile0; mlive = b.ntiles;
        wbase += (size_t)b.group * a.group_bytes;
    }
    if (mlive > MBT) mlive = MBT;
    const int ntot = a.N / 16, n0 = bn * NBT;
    constexpr int PIECES = (MBT + NBT) * 2, PPW = PIECES / 4;
    const uint8_t* src[PPW];
#pragma unroll
    for (int i = 0; i < PPW; ++i) { /* piece p: tile p / 2 (M-tiles first, then column tiles), k tile p % 2 of the stage */
        const int p = wave * PPW + i, t = p >> 1, k0 = 2 * s0 + (p & 1);
        if (t < MBT) src[i] = (const uint8_t*)a.a + ((size_t)(m0 + (t < mlive ? t : 0)) * ktiles + k0) * 1024 + lane * 16;
        else {
            const int nt = n0 + t - MBT < ntot ? n0 + t - MBT : ntot - 1;
            src[i] = wbase + ((size_t)nt * ktiles + k0) * 1024 + lane * 16;
        }
    }
    auto stage = [&](int buf) {
#pragma unroll
        for (int i = 0; i < PPW; ++i) {
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src[i],
                                             (__attribute__((address_space(3))) void*)(lds + buf * STAGE + (wave * PPW + i) * 1024), 16, 0, 0);
            src[i] += 2048;
        }
    };
    const int wm = (wave & 1) * MW, wn = (wave >> 1) * NW;
    tk_v4f acc[NW][MW];
#pragma unroll
    for (int n = 0; n < NW; ++n)
#pragma unroll
        for (int m = 0; m < MW; ++m) acc[n][m] = tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
    for (int s = 0; s < RING - 1 && s < stages; ++s) stage(s);
    int cur = 0, fill = RING - 1;
#pragma unroll 1
    for (int s = 0; s < stages; ++s) {
        /* stage s has landed when at most the RING - 2 younger ones are outstanding (at the end there are fewer: wait for all) */
        if (s + RING - 1 <= stages) wait_vm<(RING - 2) * PPW>();
        else wait_vm<0>();
        asm volatile("s_barrier" ::: "memory"); /* every wave's pieces of stage s have landed, and every wave has read stage s - 1, whose place is filled next */
        if (s + RING - 1 < stages) stage(fill);
        const uint8_t* b = lds + cur * STAGE + lane * 16;
        cur = cur + 1 < RING ? cur + 1 : 0;
        fill = fill + 1 < RING ? fill + 1 : 0;
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            tk_v4u av[MW], wv[NW];
#pragma unroll
            for (int m = 0; m < MW; ++m) av[m] = *(const tk_v4u*)(b + ((wm + m) * 2 + k) * 1024);
#pragma unroll
            for (int n = 0; n < NW; ++n) wv[n] = *(const tk_v4u*)(b + ((MBT + wn + n) * 2 + k) * 1024);
#pragma unroll
            for (int n = 0; n < NW; ++n)
#pragma unroll
                for (int m = 0; m < MW; ++m) acc[n][m] = TkImg<T>::mma(wv[n], av[m], acc[n][m]);
        }
    }
#pragma unroll
    for (int m = 0; m < MW; ++m) {
        const int64_t row = (int64_t)(m0 + wm + m) * 16 + (lane & 15);
        if (wm + m >= mlive || (!GROUPED && row >= a.nrows)) continue;
        if (SWIGLU) {
#pragma unroll
            for (int n = 0; n < NW / 2; ++n)
                if (n0 + wn + 2 * n < ntot) store_act<T>(a, row, ((n0 + wn) / 2 + n) * 16 + 4 * (lane >> 4), acc[2 * n][m], acc[2 * n + 1 < NW ? 2 * n + 1 : 0][m]);
        } else {
#pragma unroll
            for (int n = 0; n < NW; ++n)
                if (n0 + wn + n < ntot) store_f32<T>(a, row, (n0 + wn + n) * 16 + 4 * (lane >> 4), acc[n][m]);
        }
    }
}

template <typename T>
__global__ void k_put_image(const void* src, int src_f32, int64_t N, int64_t K, T* img, int ktiles, int64_t n0, int64_t k0, int interleave) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= N * K) return;
    const int64_t n = i / K;
    const int k = (int)(i % K);
    const float v = src_f32 ? ((const float*)src)[i] : tk_bf16_float(((const uint16_t*)src)[i]);
    const int64_t row = interleave < 0 ? n0 + n : (2 * (n / 16) + interleave) * 16 + n % 16;
    tk_img_put(img, row, (int)k0 + k, ktiles, v);
}

template <typename T, bool SWIGLU, bool GROUPED>
const char* launch(const TkImgGemm& g, hipStream_t s, int* slabs) {
    const int ntiles = g.N / 16;
    const int mtiles = GROUPED ? g.block_tiles : (g.nrows + 15) / 16;
    if (mtiles <= 4) {
        /* GROUPED: one block per table entry */
        const int gy = GROUPED ? g.max_blocks : 1;
#define TK_SK(MT, NT, WV) hipLaunchKernelGGL((k_gemm_skinny<T, MT, NT, WV, SWIGLU, GROUPED>), dim3((ntiles + NT - 1) / NT, gy), dim3(64 * WV), (size_t)WV * NT * MT * 1024, s, g)
#define TK_SKM(NT, WV) do { if (mtiles <= 1) TK_SK(1, NT, WV); else if (mtiles <= 2) TK_SK(2, NT, WV); else TK_SK(4, NT, WV); } while (0)
        if (SWIGLU || ntiles * gy >= 1024) {
            if (ntiles * gy >= 2048) TK_SKM(2, 4); else TK_SKM(2, 8);
        } else {
            TK_SKM((SWIGLU ? 2 : 1), 8);
        }
#undef TK_SKM
#undef TK_SK
        return nullptr;
    }
    const int nblk_m = GROUPED ? g.max_blocks : (g.nrows + 127) / 128;
    int nb = 8, ks = 1;
    const int64_t full = (int64_t)nblk_m * ((ntiles + 7) / 8);
    if (!SWIGLU && !GROUPED && g.max_slabs > 1 && full < 256) { /* large blocks of a part of K rather than small blocks of all of it: at least eight stages each */
        ks = (int)(512 / full);
        if (ks > g.max_slabs) ks = g.max_slabs;
        const int most = g.K / TkImg<T>::KT / 16;
        if (ks > most) ks = most;
        if (ks < 1) ks = 1;
    }
    while (nb > (SWIGLU ? 4 : 2) && (int64_t)nblk_m * ((ntiles + nb - 1) / nb) * ks < 200) nb /= 2;
    if (slabs) *slabs = ks;
#define TK_WD(NB) do { const int nbn = (ntiles + NB - 1) / NB; hipLaunchKernelGGL((k_gemm_wide<T, NB, SWIGLU, GROUPED>), dim3(nbn * nblk_m * ks), dim3(256), (size_t)wide_ring<NB>() * (8 + NB) * 2048, s, g, nbn, nblk_m, ks); } while (0)
    if (nb == 8) TK_WD(8);
    else if (nb == 4 || SWIGLU) TK_WD(4);
    else TK_WD((SWIGLU ? 4 : 2));
#undef TK_WD
    return nullptr;
}

} // namespace

const char* tk_launch_gemm_image(const TkImgGemm& g, hipStream_t s, int* slabs) {
    if (slabs) *slabs = 1;
    if (g.type != TK_IMG_BF16 && g.type != TK_IMG_F32) return "gemm_image: unknown element type";
    if (!g.w || !g.a || g.K <= 0 || g.K % (2 * tk_img_kt(g.type))) return "gemm_image: K is not a multiple of two tiles";
    if (g.N <= 0 || g.N % (g.swiglu ? 32 : 16)) return "gemm_image: N is not a multiple of its tile";
    if (g.swiglu ? (!g.act_img || g.act_ktiles * tk_img_kt(g.type) < g.N / 2) : (!g.out || g.n_valid > g.N || g.ldc < g.n_valid)) return "gemm_image: output does not fit";
    if (g.copy_img && g.copy_ktiles * tk_img_kt(g.type) < g.copy1 - g.copy0) return "gemm_image: copied columns do not fit their image";
    if (g.max_slabs > 1 && (!slabs || g.swiglu || g.copy_img || g.slab_floats % 4)) return "gemm_image: this product cannot be split over k";
    if (g.blocks ? (!g.n_blocks || g.max_blocks < 1 || g.block_tiles < 1 || g.block_tiles > 8) : g.nrows < 1) return "gemm_image: no rows";
#define TK_GI(T) (g.swiglu ? (g.blocks ? launch<T, true, true>(g, s, slabs) : launch<T, true, false>(g, s, slabs)) : (g.blocks ? launch<T, false, true>(g, s, slabs) : launch<T, false, false>(g, s, slabs)))
    return g.type == TK_IMG_F32 ? TK_GI(float) : TK_GI(TkBf16);
#undef TK_GI
}

template <typename T>
static hipError_t opt_in_wide() {
    hipError_t e = hipSuccess;
#define TK_OPT(NB, S, G) if (e == hipSuccess) e = hipFuncSetAttribute((const void*)k_gemm_wide<T, NB, S, G>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024)
    TK_OPT(2, false, false); TK_OPT(2, false, true);
    TK_OPT(4, false, false); TK_OPT(4, false, true); TK_OPT(4, true, false); TK_OPT(4, true, true);
#undef TK_OPT
    return e;
}

const char* tk_gemm_image_prepare_device() {
    static std::atomic<bool> done[64];
    static std::mutex mu;
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return "no current device";
    if (done[dev].load(std::memory_order_acquire)) return nullptr;
    std::lock_guard<std::mutex> lk(mu);
    hipError_t e = opt_in_wide<TkBf16>();
    if (e == hipSuccess) e = opt_in_wide<float>();
    if (e != hipSuccess) return hipGetErrorString(e);
    done[dev].store(true, std::memory_order_release);
    return nullptr;
}

void tk_launch_put_image(int type, const void* src, int src_f32, int64_t N, int64_t K, void* img, int ktiles, int64_t n0, int64_t k0, int interleave, hipStream_t s) {
    const unsigned blocks = (unsigned)((N * K + 255) / 256);
    if (type == TK_IMG_F32) hipLaunchKernelGGL((k_put_image<float>), dim3(blocks), dim3(256), 0, s, src, src_f32, N, K, (float*)img, ktiles, n0, k0, interleave);
    else hipLaunchKernelGGL((k_put_image<TkBf16>), dim3(blocks), dim3(256), 0, s, src, src_f32, N, K, (TkBf16*)img, ktiles, n0, k0, interleave);
}
