/* tk_image_device.h — device helpers for operand images (tk_gemm_image.h) */
#ifndef TK_IMAGE_DEVICE_H
#define TK_IMAGE_DEVICE_H

#include <hip/hip_runtime.h>
#include <stdint.h>

typedef float tk_v4f __attribute__((ext_vector_type(4)));
typedef __bf16 tk_v8bf __attribute__((ext_vector_type(8)));
typedef uint32_t tk_v4u __attribute__((ext_vector_type(4)));
typedef uint32_t tk_v2u __attribute__((ext_vector_type(2)));

struct TkBf16 { uint16_t bits; };

__device__ __forceinline__ uint16_t tk_bf16_bits(float x) { return __builtin_bit_cast(uint16_t, (__bf16)x); }
__device__ __forceinline__ float tk_bf16_float(uint16_t b) { return __uint_as_float((uint32_t)b << 16); }

template <typename T> struct TkImg;
template <> struct TkImg<TkBf16> {
    static constexpr int KT = 32, EP = 8; /* k per tile, elements per lane */
    __device__ static __forceinline__ TkBf16 from(float x) { return TkBf16{tk_bf16_bits(x)}; }
    __device__ static __forceinline__ float to(TkBf16 v) { return tk_bf16_float(v.bits); }
    /* c += a b over one tile; a's row = the accumulator's row index 4 g + r, b's row = the accumulator's column l % 16 */
    __device__ static __forceinline__ tk_v4f mma(tk_v4u a, tk_v4u b, tk_v4f c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(tk_v8bf, a), __builtin_bit_cast(tk_v8bf, b), c, 0, 0, 0);
    }
};
template <> struct TkImg<float> {
    static constexpr int KT = 16, EP = 4;
    __device__ static __forceinline__ float from(float x) { return x; }
    __device__ static __forceinline__ float to(float v) { return v; }
    __device__ static __forceinline__ tk_v4f mma(tk_v4u a, tk_v4u b, tk_v4f c) {
        const tk_v4f x = __builtin_bit_cast(tk_v4f, a), y = __builtin_bit_cast(tk_v4f, b);
        c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[0], y[0], c, 0, 0, 0);
        c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[1], y[1], c, 0, 0, 0);
        c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[2], y[2], c, 0, 0, 0);
        c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[3], y[3], c, 0, 0, 0);
        return c;
    }
};

/* element (row, k) of an image */
template <typename T>
__device__ __forceinline__ size_t tk_img_index(int64_t row, int k, int ktiles) {
    constexpr int KT = TkImg<T>::KT, EP = TkImg<T>::EP;
    return ((size_t)(row >> 4) * ktiles + k / KT) * (1024 / sizeof(T)) + (size_t)((row & 15) + 16 * ((k % KT) / EP)) * EP + k % EP;
}
template <typename T>
__device__ __forceinline__ void tk_img_put(T* img, int64_t row, int k, int ktiles, float v) { img[tk_img_index<T>(row, k, ktiles)] = TkImg<T>::from(v); }

/* four consecutive k, k % 4 == 0 */
__device__ __forceinline__ void tk_img_put4(float* img, int64_t row, int k, int ktiles, tk_v4f v) { *(tk_v4f*)(img + tk_img_index<float>(row, k, ktiles)) = v; }
__device__ __forceinline__ void tk_img_put4(TkBf16* img, int64_t row, int k, int ktiles, tk_v4f v) {
    tk_v2u p;
    p[0] = (uint32_t)tk_bf16_bits(v[0]) | (uint32_t)tk_bf16_bits(v[1]) << 16;
    p[1] = (uint32_t)tk_bf16_bits(v[2]) | (uint32_t)tk_bf16_bits(v[3]) << 16;
    *(tk_v2u*)(img + tk_img_index<TkBf16>(row, k, ktiles)) = p;
}

/* eight consecutive k, k % 8 == 0 */
__device__ __forceinline__ void tk_img_put8(float* img, int64_t row, int k, int ktiles, tk_v4f a, tk_v4f b) { tk_img_put4(img, row, k, ktiles, a); tk_img_put4(img, row, k + 4, ktiles, b); }
__device__ __forceinline__ void tk_img_put8(TkBf16* img, int64_t row, int k, int ktiles, tk_v4f a, tk_v4f b) {
    tk_v4u p;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        p[i] = (uint32_t)tk_bf16_bits(a[2 * i]) | (uint32_t)tk_bf16_bits(a[2 * i + 1]) << 16;
        p[2 + i] = (uint32_t)tk_bf16_bits(b[2 * i]) | (uint32_t)tk_bf16_bits(b[2 * i + 1]) << 16;
    }
    *(tk_v4u*)(img + tk_img_index<TkBf16>(row, k, ktiles)) = p;
}

/* lane exchanges on the vector pipe: DPP rotations inside a row of 16 lanes, row and half-wave swaps between rows */
template <int CTRL> __device__ __forceinline__ float tk_dpp(float v) { return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false)); }
/* sum over the 16 lanes of a row, in every lane of it (row_ror 8, 4, 2, 1) */
__device__ __forceinline__ float tk_row16_sum(float v) {
    v += tk_dpp<0x128>(v);
    v += tk_dpp<0x124>(v);
    v += tk_dpp<0x122>(v);
    v += tk_dpp<0x121>(v);
    return v;
}
/* the values of a pair of rows (lanes l, l ^ 16) or of the two halves (l, l ^ 32), in every lane */
struct TkPair { float a, b; };
__device__ __forceinline__ TkPair tk_rows(float v) {
    const auto p = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return TkPair{__uint_as_float(p[0]), __uint_as_float(p[1])};
}
__device__ __forceinline__ TkPair tk_halves(float v) {
    const auto p = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return TkPair{__uint_as_float(p[0]), __uint_as_float(p[1])};
}
__device__ __forceinline__ float tk_row32_sum(float v) { const TkPair p = tk_rows(tk_row16_sum(v)); return p.a + p.b; }
__device__ __forceinline__ float tk_wave_sum(float v) { const TkPair p = tk_halves(tk_row32_sum(v)); return p.a + p.b; }
/* over the four lanes l % 16 + 16 g */
__device__ __forceinline__ float tk_quad_sum(float v) { const TkPair p = tk_rows(v); const TkPair q = tk_halves(p.a + p.b); return q.a + q.b; }
__device__ __forceinline__ float tk_quad_max(float v) { const TkPair p = tk_rows(v); const TkPair q = tk_halves(fmaxf(p.a, p.b)); return fmaxf(q.a, q.b); }
__device__ __forceinline__ float tk_sigmoid32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float tk_silu32(float z) { return z / (1.0f + expf(-z)); }

#endif
