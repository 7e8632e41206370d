/* tk_mixer_kernels.hip — see tk_mixer_kernels.h */
#include "tk_mixer_kernels.h"

#include <math.h>

#include <atomic>
#include <mutex>

#include "../nn/tk_image_device.h"

namespace {

constexpr float LOG2E = 1.44269504088896340736f;

/* ------------------------------------------------------------------ embedding, norms ------- */

__device__ __forceinline__ float block_sum(float v, float* red /* [16] */) {
    v = tk_wave_sum(v);
    const int w = threadIdx.x >> 6, nw = blockDim.x >> 6;
    if ((threadIdx.x & 63) == 0) red[w] = v;
    __syncthreads();
    float t = 0.0f;
    for (int i = 0; i < nw; ++i) t += red[i];
    __syncthreads();
    return t;
}

/* A row of `width` elements over a workgroup, NV groups of eight a thread.  VEC (width a multiple of eight): a group is eight consecutive
 * elements; otherwise elements a workgroup apart. */
template <bool VEC, int NV>
struct Row {
    float v[NV][8];
    __device__ static __forceinline__ int at(int j, int e) { return VEC ? (int)(j * blockDim.x + threadIdx.x) * 8 + e : (int)((j * 8 + e) * blockDim.x + threadIdx.x); }
    /* f(group, element, k) of the thread's elements below width */
    template <typename F>
    __device__ static __forceinline__ void each(int width, F f) {
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            if (VEC && at(j, 0) >= width) break;
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (VEC || at(j, e) < width) f(j, e, at(j, e));
        }
    }
    __device__ __forceinline__ void load(const float* p, int width) {
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            if (VEC) {
                if (at(j, 0) >= width) break;
                const tk_v4f a = *(const tk_v4f*)(p + at(j, 0)), b = *(const tk_v4f*)(p + at(j, 0) + 4);
#pragma unroll
                for (int e = 0; e < 4; ++e) { v[j][e] = a[e]; v[j][4 + e] = b[e]; }
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e) v[j][e] = at(j, e) < width ? p[at(j, e)] : 0.0f;
            }
        }
    }
    __device__ __forceinline__ void store(float* p, int width) const {
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            if (VEC) {
                if (at(j, 0) >= width) break;
                *(tk_v4f*)(p + at(j, 0)) = tk_v4f{v[j][0], v[j][1], v[j][2], v[j][3]};
                *(tk_v4f*)(p + at(j, 0) + 4) = tk_v4f{v[j][4], v[j][5], v[j][6], v[j][7]};
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e)
                    if (at(j, e) < width) p[at(j, e)] = v[j][e];
            }
        }
    }
    template <typename T>
    __device__ __forceinline__ void image(T* img, int64_t row, int ktiles, int width) const {
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            if (VEC) {
                if (at(j, 0) >= width) break;
                tk_img_put8(img, row, at(j, 0), ktiles, tk_v4f{v[j][0], v[j][1], v[j][2], v[j][3]}, tk_v4f{v[j][4], v[j][5], v[j][6], v[j][7]});
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e)
                    if (at(j, e) < width) tk_img_put(img, row, at(j, e), ktiles, v[j][e]);
            }
        }
    }
    /* the row over its root mean square, or less its mean over its deviation; red: [24], of this call only.  The variance is merged from the waves'
     * own means and squared deviations. */
    __device__ __forceinline__ void normalise(const TkNorm& n, float eps, int width, float* red) {
        Row w, b;
        w.load(n.w, width);
        if (n.layer) b.load(n.b, width);
        const int wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
        float mean = 0.0f, r;
        if (n.layer) {
            float s = 0.0f, c = 0.0f, d = 0.0f;
            each(width, [&](int j, int e, int) { s += v[j][e]; c += 1.0f; });
            s = tk_wave_sum(s);
            c = tk_wave_sum(c);
            const float m = c > 0.0f ? s / c : 0.0f;
            each(width, [&](int j, int e, int) { d += (v[j][e] - m) * (v[j][e] - m); });
            d = tk_wave_sum(d);
            if ((threadIdx.x & 63) == 0) { red[wave] = s; red[8 + wave] = c; red[16 + wave] = d; }
            __syncthreads();
            for (int i = 0; i < nw; ++i) mean += red[i];
            mean /= (float)width;
            float var = 0.0f;
            for (int i = 0; i < nw; ++i) {
                const float ci = red[8 + i], off = ci > 0.0f ? red[i] / ci - mean : 0.0f;
                var += red[16 + i] + ci * off * off;
            }
            r = 1.0f / sqrtf(var / (float)width + eps);
        } else {
            float d = 0.0f;
            each(width, [&](int j, int e, int) { d += v[j][e] * v[j][e]; });
            d = tk_wave_sum(d);
            if ((threadIdx.x & 63) == 0) red[wave] = d;
            __syncthreads();
            float t = 0.0f;
            for (int i = 0; i < nw; ++i) t += red[i];
            r = 1.0f / sqrtf(t / (float)width + eps);
        }
        each(width, [&](int j, int e, int) { v[j][e] = (v[j][e] - mean) * r * w.v[j][e] + (n.layer ? b.v[j][e] : 0.0f); });
    }
};

template <typename T, bool VEC, int NV>
__global__ __launch_bounds__(512) void k_layer_embed(const uint16_t* table, int width, float scale, const int32_t* tok, float* x, TkNorm next, float eps, T* img, int ktiles) {
    __shared__ float red[24];
    const int row = blockIdx.x;
    const uint16_t* e = table + (size_t)tok[row] * width;
    Row<VEC, NV> v;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        if (VEC) {
            if (v.at(j, 0) >= width) break;
            const tk_v4u u = *(const tk_v4u*)(e + v.at(j, 0));
#pragma unroll
            for (int i = 0; i < 4; ++i) { v.v[j][2 * i] = __uint_as_float(u[i] << 16) * scale; v.v[j][2 * i + 1] = __uint_as_float(u[i] & 0xffff0000u) * scale; }
        } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) v.v[j][i] = v.at(j, i) < width ? tk_bf16_float(e[v.at(j, i)]) * scale : 0.0f;
        }
    }
    v.store(x + (size_t)row * width, width);
    if (next.w) v.normalise(next, eps, width, red);
    v.image(img, row, ktiles, width);
}

template <typename T, bool VEC, int NV>
__global__ __launch_bounds__(512) void k_post_norm(TkSubOut o, TkNorm norm, TkNorm next, float eps, int width, float* x, T* img, int ktiles) {
    __shared__ float red[2][24];
    const int row = blockIdx.x;
    float* xr = x + (size_t)row * width;
    Row<VEC, NV> y, z;
    if (o.top > 0) {
#pragma unroll
        for (int j = 0; j < NV; ++j)
#pragma unroll
            for (int e = 0; e < 8; ++e) y.v[j][e] = 0.0f;
        for (int j = 0; j < o.top; ++j) {
            z.load(o.y + (size_t)o.slot[row * o.top + j] * o.ld, width);
            const float c = o.weight[row * o.top + j];
            y.each(width, [&](int g, int e, int) { y.v[g][e] += z.v[g][e] * c; });
        }
    } else {
        y.load(o.y + (size_t)row * o.ld, width);
        for (int i = 1; i < o.slabs; ++i) {
            z.load(o.y + i * o.slab_floats + (size_t)row * o.ld, width);
            y.each(width, [&](int g, int e, int) { y.v[g][e] += z.v[g][e]; });
        }
        if (o.bias) {
            z.load(o.bias, width);
            y.each(width, [&](int g, int e, int) { y.v[g][e] += z.v[g][e] * o.bias_scale; });
        }
    }
    z.load(xr, width);
    y.normalise(norm, eps, width, red[0]);
    y.each(width, [&](int g, int e, int) { y.v[g][e] += z.v[g][e]; });
    y.store(xr, width);
    if (next.w) y.normalise(next, eps, width, red[1]);
    y.image(img, row, ktiles, width);
}

template <typename T, bool VEC, int NV>
__global__ __launch_bounds__(512) void k_rows_norm(const float* x, const int32_t* rows, TkNorm norm, float eps, int width, T* img, int ktiles) {
    __shared__ float red[24];
    const int i = blockIdx.x;
    Row<VEC, NV> v;
    v.load(x + (size_t)(rows ? rows[i] : i) * width, width);
    v.normalise(norm, eps, width, red);
    v.image(img, i, ktiles, width);
}

/* ------------------------------------------------------------------ short convolutions ----- */

/* V neighbouring elements of a row a lane, i = 0, V, 2 V ..: element(lane, i) + 0 .. V - 1 */
template <int V> struct TkVf;
template <> struct TkVf<1> { typedef float type __attribute__((ext_vector_type(1))); };
template <> struct TkVf<2> { typedef float type __attribute__((ext_vector_type(2))); };
template <int V> using tk_vf = typename TkVf<V>::type;
template <int V> __device__ __forceinline__ int element(int lane, int i) { return V * lane + 64 * i; }
template <int V> __device__ __forceinline__ tk_vf<V> load_v(const float* p) { return *(const tk_vf<V>*)p; } /* V = 2: eight-byte aligned */

/* a causal convolution over the rows of a sequence; what came before the pass is in the history (zeros before the sequence) */
struct Conv {
    const float* w; /* [channels][taps] */
    float* state;   /* [copies][channels][taps - 1] */
    int channels, taps, col;
    __device__ __forceinline__ float input(const TkPassTab& t, const float* proj, int ld, int seg, int s, int c) const {
        if (s >= 0) return proj[(size_t)(t.seg_row0[seg] + s) * ld + col + c]; /* s: time inside the segment */
        const int in = t.seg_in[seg], hist = taps - 1;
        return in < 0 ? 0.0f : state[((size_t)in * channels + c) * hist + hist + s];
    }
    /* channels c0 + element(lane, i) (< c0 + n) of RW rows from rowb on (rows past the pass repeat its last one) */
    template <int RW, int V>
    __device__ __forceinline__ void rows(const TkPassTab& t, const float* proj, int ld, int rowb, int nrows, int c0, int n, int lane, float (&y)[RW][4]) const {
        const int hist = taps - 1, seg0 = t.seg[rowb], first = rowb - t.seg_row0[seg0];
        const bool inside = first >= hist && first + RW <= t.seg_n[seg0]; /* every input is a row of this pass */
        const int in0 = t.seg_in[seg0];
#pragma unroll
        for (int i = 0; i < 4; i += V) {
#pragma unroll
            for (int r = 0; r < RW; ++r)
#pragma unroll
                for (int k = 0; k < V; ++k) y[r][i + k] = 0.0f;
            const int c = c0 + element<V>(lane, i);
            if (64 * i >= n || element<V>(lane, i) >= n) continue;
            if (inside && taps == 4) { /* every input once */
                tk_vf<V> x[RW + 3];
#pragma unroll
                for (int j = 0; j < RW + 3; ++j) x[j] = load_v<V>(proj + (size_t)(rowb - 3 + j) * ld + col + c);
#pragma unroll
                for (int k = 0; k < V; ++k) {
                    const tk_v4f f = *(const tk_v4f*)(w + (size_t)(c + k) * 4);
#pragma unroll
                    for (int r = 0; r < RW; ++r)
#pragma unroll
                        for (int j = 0; j < 4; ++j) y[r][i + k] = fmaf(f[j], x[r + j][k], y[r][i + k]);
                }
            } else if (RW == 1 && first == 0 && taps == 4) { /* decoding: the history and one row */
                const tk_vf<V> x = load_v<V>(proj + (size_t)rowb * ld + col + c);
#pragma unroll
                for (int k = 0; k < V; ++k) {
                    const tk_v4f f = *(const tk_v4f*)(w + (size_t)(c + k) * 4);
                    const float* old = state + ((size_t)(in0 < 0 ? 0 : in0) * channels + c + k) * 3;
                    float past = fmaf(f[2], old[2], fmaf(f[1], old[1], f[0] * old[0]));
                    if (in0 < 0) past = 0.0f;
                    y[0][i + k] = fmaf(f[3], x[k], past);
                }
            } else if (inside) {
                for (int j = 0; j < taps; ++j)
#pragma unroll
                    for (int k = 0; k < V; ++k) {
                        const float tap = w[(size_t)(c + k) * taps + j];
#pragma unroll
                        for (int r = 0; r < RW; ++r) y[r][i + k] = fmaf(tap, proj[(size_t)(rowb + r - hist + j) * ld + col + c + k], y[r][i + k]);
                    }
            } else {
#pragma unroll
                for (int r = 0; r < RW; ++r) {
                    const int row = rowb + r < nrows ? rowb + r : nrows - 1, seg = t.seg[row], at = row - t.seg_row0[seg];
                    for (int j = 0; j < taps; ++j)
#pragma unroll
                        for (int k = 0; k < V; ++k) y[r][i + k] = fmaf(w[(size_t)(c + k) * taps + j], input(t, proj, ld, seg, at - hist + j, c + k), y[r][i + k]);
                }
            }
        }
    }
    /* a segment's last row leaves the history behind */
    __device__ __forceinline__ void leave(const TkPassTab& t, const float* proj, int ld, int row, int c0, int n, int lane) const {
        const int seg = t.seg[row], at = row - t.seg_row0[seg], hist = taps - 1;
        if (at + 1 != t.seg_n[seg]) return;
        for (int e = lane; e < n; e += 64)
            for (int j = 0; j < hist; ++j) state[((size_t)t.seg_out[seg] * channels + c0 + e) * hist + j] = input(t, proj, ld, seg, at + 1 - hist + j, c0 + e);
    }
};

/* ------------------------------------------------------------------ between projections and mixers ---- */

/* one wave: one head of q, k or v of RW consecutive rows (rows past the pass repeat its last one and store nothing); all loads come first.
 * CONV: the elements are convolved ones; rotation partners meet in `ex`, [RW][TK_MAX_HEAD_DIM] of LDS of this wave's own.  V = 2: sizes, columns and
 * pitch are even, half the rotating dimensions too */
template <typename T, int RW, bool CONV, int V>
__device__ __forceinline__ void attn_unit(const TkAttnArgs& a, const TkPassTab& t, const float* proj, int ld, int row0, int nrows, int u, int lane, float* ex) {
    const bool is_q = u < a.heads, is_v = u >= a.heads + a.kv_heads;
    const int n = is_v ? a.vdim : a.dim;
    const int head = is_q ? u : is_v ? u - a.heads - a.kv_heads : u - a.heads;
    const int off = is_q ? head * a.dim : is_v ? (a.heads + a.kv_heads) * a.dim + head * a.vdim : (a.heads + head) * a.dim;
    const float* b = a.bias ? a.bias + off : nullptr;
    const float* w = is_v ? nullptr : is_q ? a.q_norm : a.k_norm;
    const int half = is_v ? 0 : a.rot_dims / 2;
    float v[RW][4], z[RW][4], c[RW][4], s[RW][4]; /* element, its rotation partner, cosine, signed sine */
    int pos[RW];
    size_t page[RW];
    const Conv conv{a.conv, a.conv_state, (a.heads + a.kv_heads) * a.dim + a.kv_heads * a.vdim, a.taps, a.col};
#pragma unroll
    for (int r = 0; r < RW; ++r) {
        const int row = row0 + r < nrows ? row0 + r : nrows - 1;
        pos[r] = t.pos[row];
        page[r] = is_q ? 0 : (size_t)t.page_of[(size_t)t.seq[row] * t.max_pages + pos[r] / TK_PAGE];
        const float* src = proj + (size_t)row * ld + a.col + off;
        const float *cosp = a.rope_cos + (size_t)pos[r] * half, *sinp = a.rope_sin + (size_t)pos[r] * half;
#pragma unroll
        for (int i = 0; i < 4; i += V) {
            const int e = element<V>(lane, i);
            tk_vf<V> x = {}, y = {}, cs, sn = {};
#pragma unroll
            for (int k = 0; k < V; ++k) cs[k] = 1.0f;
            if (64 * i < n && e < n) {
                const int f = e < half ? e + half : e - half, j = e < half ? e : f;
                if (!CONV) x = load_v<V>(src + e);
                if (e < 2 * half) {
                    if (!CONV) y = load_v<V>(src + f);
                    cs = load_v<V>(cosp + j);
                    sn = load_v<V>(sinp + j) * (e < half ? -1.0f : 1.0f);
                }
#pragma unroll
                for (int k = 0; k < V; ++k) {
                    if (b) x[k] += b[e + k];
                    if (e < 2 * half) y[k] = (y[k] + (b ? b[f + k] : 0.0f)) * (w ? w[f + k] : 1.0f);
                }
            }
#pragma unroll
            for (int k = 0; k < V; ++k) { v[r][i + k] = x[k]; z[r][i + k] = y[k]; c[r][i + k] = cs[k]; s[r][i + k] = sn[k]; }
        }
    }
    if (CONV) {
        conv.rows<RW, V>(t, proj, ld, row0, nrows, off, n, lane, v);
        if (half > 0) { /* partners change hands inside the wave */
#pragma unroll
            for (int r = 0; r < RW; ++r)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int e = element<V>(lane, i / V * V) + i % V;
                    if (e < 2 * half) ex[r * TK_MAX_HEAD_DIM + e] = v[r][i];
                }
            __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
            __builtin_amdgcn_wave_barrier();
            __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
            for (int r = 0; r < RW; ++r)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int e = element<V>(lane, i / V * V) + i % V;
                    if (e < 2 * half) z[r][i] = ex[r * TK_MAX_HEAD_DIM + (e < half ? e + half : e - half)];
                }
        }
    }
    float wv[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int e = element<V>(lane, i / V * V) + i % V;
        wv[i] = w && e < n ? w[e] : 1.0f;
    }
#pragma unroll
    for (int r = 0; r < RW; ++r) {
        if (row0 + r >= nrows) break;
        float f = 1.0f;
        if (w) {
            float ss = 0.0f;
#pragma unroll
            for (int i = 0; i < 4; ++i) ss += v[r][i] * v[r][i];
            f = 1.0f / sqrtf(tk_wave_sum(ss) / (float)n + a.eps);
        }
        T* dst = is_q ? (T*)a.q + ((size_t)(row0 + r) * a.heads + head) * a.kv.dim_pad
                      : is_v ? (T*)a.kv.v + (page[r] * a.kv_heads + head) * a.kv.vdim_pad * TK_PAGE + pos[r] % TK_PAGE
                             : (T*)a.kv.k + ((page[r] * a.kv_heads + head) * TK_PAGE + pos[r] % TK_PAGE) * a.kv.dim_pad;
#pragma unroll
        for (int i = 0; i < 4; i += V) {
            const int e = element<V>(lane, i);
            if (64 * i >= n || e >= n) break;
            T y[V];
#pragma unroll
            for (int k = 0; k < V; ++k) y[k] = TkImg<T>::from((v[r][i + k] * f * wv[i + k]) * c[r][i + k] + (z[r][i + k] * f) * s[r][i + k]);
            if (is_v) {
#pragma unroll
                for (int k = 0; k < V; ++k) dst[(e + k) * TK_PAGE] = y[k];
            } else if constexpr (V == 2) {
                struct __attribute__((aligned(2 * sizeof(T)))) Two { T a, b; };
                *(Two*)(dst + e) = Two{y[0], y[1]};
            } else {
                dst[e] = y[0];
            }
        }
        if (CONV) conv.leave(t, proj, ld, row0 + r, off, n, lane);
    }
}

/* one wave: one head of q, k or v after its convolution, or one head's decays and step size, of RW consecutive rows */
template <int RW>
__device__ __forceinline__ void delta_unit(const TkDeltaArgs& d, const TkPassTab& t, const float* proj, int ld, int rowb, int nrows, int u, int lane) {
    const int qk = d.kv_heads * d.dim, channels = 2 * qk + d.heads * d.vdim;
    if (u >= 2 * d.kv_heads + d.heads) {
        const int h = u - 2 * d.kv_heads - d.heads;
        const float rate = -expf(d.a_log[h]);
#pragma unroll
        for (int r = 0; r < RW; ++r) {
            const int row = rowb + r;
            if (row >= nrows) break;
            for (int e = lane; e < d.dim; e += 64) {
                const float z = d.low[(size_t)row * d.low_ld + d.low_a + h * d.dim + e] + d.dt_bias[h * d.dim + e];
                const float sp = fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); /* softplus */
                d.g[((size_t)row * d.heads + h) * d.dim + e] = expf(rate * sp);
            }
            if (lane == 0) d.beta[(size_t)row * d.heads + h] = tk_sigmoid32(proj[(size_t)row * ld + d.col + channels + h]);
        }
        return;
    }
    const int which = u < d.kv_heads ? 0 : u < 2 * d.kv_heads ? 1 : 2;
    const int head = which == 2 ? u - 2 * d.kv_heads : which == 1 ? u - d.kv_heads : u;
    const int n = which == 2 ? d.vdim : d.dim, c0 = which == 2 ? 2 * qk + head * d.vdim : which * qk + head * d.dim;
    float* dst = which == 0 ? d.q + head * d.dim : which == 1 ? d.k + head * d.dim : d.v + (size_t)head * d.vdim;
    const size_t pitch = which == 2 ? (size_t)d.heads * d.vdim : qk;
    const Conv conv{d.conv, d.conv_state, channels, d.taps, d.col};
    float y[RW][4];
    conv.rows<RW, 1>(t, proj, ld, rowb, nrows, c0, n, lane, y);
#pragma unroll
    for (int r = 0; r < RW; ++r) {
        const int row = rowb + r;
        if (row >= nrows) break;
        float ss = 0.0f;
#pragma unroll
        for (int i = 0; i < 4; ++i) { y[r][i] = tk_silu32(y[r][i]); ss += y[r][i] * y[r][i]; } /* silu(0) = 0 past the head */
        float f = 1.0f;
        if (which < 2) {
            f = 1.0f / sqrtf(tk_wave_sum(ss) + d.unit_eps);
            if (which == 0) f *= 1.0f / sqrtf((float)d.dim);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (lane + 64 * i < n) dst[row * pitch + lane + 64 * i] = y[r][i] * f;
        conv.leave(t, proj, ld, row, c0, n, lane);
    }
}

template <typename T, int RW, bool CONV, int V>
__global__ __launch_bounds__(256) void k_mixer_prep(const float* proj, int ld, TkAttnArgs a, TkDeltaArgs d, TkPassTab t, int na, int nd, int nrows) {
    __shared__ float ex[CONV ? 4 * RW * TK_MAX_HEAD_DIM : 1];
    const int row = blockIdx.y * RW, lane = threadIdx.x & 63;
    const int u = __builtin_amdgcn_readfirstlane(blockIdx.x * 4 + (threadIdx.x >> 6));
    if (u < na) attn_unit<T, RW, CONV, V>(a, t, proj, ld, row, nrows, u, lane, ex + (CONV ? (threadIdx.x >> 6) * RW * TK_MAX_HEAD_DIM : 0));
    else if (u < na + nd) delta_unit<RW>(d, t, proj, ld, row, nrows, u - na, lane);
}

/* ------------------------------------------------------------------ attention -------------- */

/* the lowest position (kept first ones aside) that a query at position p reads; never falls as p grows */
__device__ __forceinline__ int first_visible(const TkAttnArgs& a, int p) {
    int lo = 0;
    if (a.window > 0) lo = p - a.window + 1;
    if (a.chunk > 0) { const int c = p - (int)((unsigned)p % (unsigned)a.chunk); lo = c > lo ? c : lo; }
    return lo > 0 ? lo : 0;
}

/* the pages a range of query positions [p0, p1] reads: the kept first ones, then the window's or chunk's */
struct PageWalk {
    int nkeep, first, count;
    __device__ __forceinline__ PageWalk(const TkAttnArgs& a, int p0, int p1) {
        const int keep = a.keep_first;
        first = first_visible(a, p0) / TK_PAGE;
        const int k = keep < p1 + 1 ? keep : p1 + 1;
        const int kp = (k + TK_PAGE - 1) / TK_PAGE;
        nkeep = kp < first ? kp : first;
        count = nkeep + p1 / TK_PAGE - first + 1;
    }
    __device__ __forceinline__ int page(int i) const { return i < nkeep ? i : first + i - nkeep; }
};

/* cap * tanh(score / cap), in log2 units; EXACT: the library's function rather than a quotient of exponentials (absolute error 1e-7 of the cap) */
template <bool EXACT>
__device__ __forceinline__ float soft_cap(float x, float inv, float cap2) {
    if (EXACT) return cap2 * tanhf(x * inv);
    const float e = __builtin_amdgcn_exp2f(x * (inv * 2.0f * LOG2E));
    return cap2 - 2.0f * cap2 * __builtin_amdgcn_rcpf(1.0f + e);
}

/* scores of one page (raw products, keys k0 + 16 j + 4 g + r) -> log2 units, -inf where the query at position pq, which reads `first` on, may not
 * look.  lo, whole: the lowest query position of the wave, and the first position that all of the wave's queries read; a page that all of them see
 * whole is not masked. */
template <typename T>
__device__ __forceinline__ void mask_scores(tk_v4f (&s)[4], const TkAttnArgs& a, int k0, int g, int pq, int first, int lo, int whole) {
    if (a.softcap > 0.0f) {
        const float inv = a.scale / a.softcap, cap2 = a.softcap * LOG2E;
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) s[j][r] = soft_cap<sizeof(T) == 4>(s[j][r], inv, cap2);
    } else {
        const float c = a.scale * LOG2E;
#pragma unroll
        for (int j = 0; j < 4; ++j) s[j] *= c;
    }
    if (k0 + TK_PAGE - 1 <= lo && (whole <= k0 || k0 + TK_PAGE <= a.keep_first)) return;
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int key = k0 + 16 * j + 4 * g + r;
            const bool see = (key <= pq) & ((key >= first) | (key < a.keep_first));
            s[j][r] = see ? s[j][r] : -INFINITY;
        }
}

/* running softmax of one wave: 16 queries (lane % 16), VT 16-wide tiles of the output (rows 4 (lane / 16) + r) */
template <typename T, int VT>
struct Flash {
    float m, l;
    tk_v4f o[VT];
    __device__ __forceinline__ void init() {
        m = -INFINITY; l = 0.0f;
#pragma unroll
        for (int i = 0; i < VT; ++i) o[i] = tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
    }
    /* s[j]: scores (log2 units) of keys 16 j + 4 g + r of this page; vfrag(vt, j): four values (keys 16 j + 4 g ..) of output column
     * 16 vt + lane % 16.  The weights stay 32-bit: with bf16 values each weight enters as the sum of two bf16 numbers. */
    template <typename VF>
    __device__ __forceinline__ void update(const tk_v4f (&s)[4], int nv, VF vfrag) {
        float mx = -INFINITY;
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[j][r]);
        mx = tk_quad_max(mx);
        const float mn = fmaxf(m, mx), ms = mn == -INFINITY ? 0.0f : mn;
        const float al = __builtin_amdgcn_exp2f(m - ms);
        m = mn;
        tk_v4f p[4];
        float sum = 0.0f;
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) { p[j][r] = __builtin_amdgcn_exp2f(s[j][r] - ms); sum += p[j][r]; }
        l = l * al + tk_quad_sum(sum);
#pragma unroll
        for (int i = 0; i < VT; ++i) o[i] *= al;
        accumulate(p, nv, vfrag);
    }
    template <typename VF>
    __device__ __forceinline__ void accumulate(const tk_v4f (&p)[4], int nv, VF vfrag);
};

template <int VT, typename VF>
__device__ __forceinline__ void flash_acc(Flash<TkBf16, VT>& f, const tk_v4f (&p)[4], int nv, VF vfrag) {
#pragma unroll
    for (int h = 0; h < 2; ++h) {
        tk_v4u hi, lo;
#pragma unroll
        for (int q = 0; q < 4; ++q) { /* pair q: elements 2 q, 2 q + 1 of [p[2h], p[2h + 1]] */
            const float x = p[2 * h + (q >> 1)][2 * (q & 1)], y = p[2 * h + (q >> 1)][2 * (q & 1) + 1];
            const uint16_t xh = tk_bf16_bits(x), yh = tk_bf16_bits(y);
            hi[q] = (uint32_t)xh | (uint32_t)yh << 16;
            lo[q] = (uint32_t)tk_bf16_bits(x - tk_bf16_float(xh)) | (uint32_t)tk_bf16_bits(y - tk_bf16_float(yh)) << 16;
        }
#pragma unroll
        for (int i = 0; i < VT; ++i)
            if (i < nv) {
                const tk_v2u a = vfrag(i, 2 * h), b = vfrag(i, 2 * h + 1);
                const tk_v4u v = {a[0], a[1], b[0], b[1]};
                f.o[i] = TkImg<TkBf16>::mma(v, hi, f.o[i]);
                f.o[i] = TkImg<TkBf16>::mma(v, lo, f.o[i]);
            }
    }
}
template <int VT, typename VF>
__device__ __forceinline__ void flash_acc(Flash<float, VT>& f, const tk_v4f (&p)[4], int nv, VF vfrag) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < VT; ++i)
            if (i < nv) f.o[i] = TkImg<float>::mma(vfrag(i, j), __builtin_bit_cast(tk_v4u, p[j]), f.o[i]);
}
template <typename T, int VT>
template <typename VF>
__device__ __forceinline__ void Flash<T, VT>::accumulate(const tk_v4f (&p)[4], int nv, VF vfrag) { flash_acc(*this, p, nv, vfrag); }

/* four values of a transposed value row: 8 bytes (bf16) or 16 (f32) */
template <typename T> struct VFrag;
template <> struct VFrag<TkBf16> { typedef tk_v2u type; };
template <> struct VFrag<float> { typedef tk_v4u type; };

/* head h of `row`, columns 16 i + 4 g + r, times `f` */
template <typename T, int VT>
__device__ __forceinline__ void attn_store(const TkAttnArgs& a, const tk_v4f (&o)[VT], int64_t row, int h, int g, float f) {
    const int k0 = a.out_k0 + h * a.vdim;
#pragma unroll
    for (int i = 0; i < VT; ++i) {
        const int e = 16 * i + 4 * g;
        if (e >= a.vdim) break;
        const tk_v4f y = o[i] * f;
        if ((k0 & 3) == 0 && e + 3 < a.vdim) tk_img_put4((T*)a.out_img, row, k0 + e, a.out_ktiles, y);
        else
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (e + r < a.vdim) tk_img_put((T*)a.out_img, row, k0 + e + r, a.out_ktiles, y[r]);
    }
}

/* prompts: 64 consecutive positions of a sequence x one head per workgroup, 16 per wave.  Pages go through two LDS buffers (one where two do not
 * fit): while page i is used, page i + 1 is written to the other one and page i + 2 is on its way to registers. */
template <typename T, int B> constexpr bool attn_two_buffers() { return sizeof(T) == 2 || B < 256; }

template <typename T, int B, bool FULL /* head sizes fill the bucket */>
__global__ __launch_bounds__(256, B * sizeof(T) >= 512 ? 1 : 2) void k_attn_tiles(TkAttnArgs a, TkPassTab t, const int32_t* tiles) {
    constexpr int DT = B / TkImg<T>::KT, VT = B / 16, SZ = sizeof(T);
    typedef typename VFrag<T>::type VF;
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4;
    const int row0 = tiles[2 * blockIdx.x], n = tiles[2 * blockIdx.x + 1], h = blockIdx.y, kvh = h / (a.heads / a.kv_heads);
    const int nd = FULL ? DT : a.kv.dim_pad / TkImg<T>::KT, nv = FULL ? VT : a.kv.vdim_pad / 16;
    const int krow = a.kv.dim_pad * SZ + 16, vrow = TK_PAGE * SZ + 16; /* LDS pitches: rows start in different banks */
    const int buf = TK_PAGE * krow + a.kv.vdim_pad * vrow;
    constexpr bool TWO = attn_two_buffers<T, B>();
    const int p0 = t.pos[row0], seq = t.seq[row0];
    const int q = wave * 16 + (lane & 15), live = q < n ? q : 0;
    const int pq = q < n ? p0 + q : -1; /* rows past the tile see nothing and store nothing */
    const PageWalk walk(a, p0, p0 + n - 1);
    const int32_t* pages = t.page_of + (size_t)seq * t.max_pages;
    int ids = pages[walk.page(lane < walk.count ? lane : 0)], ids0 = 0; /* lane l: page id of step ids0 + l */
    const int kc = TK_PAGE * a.kv.dim_pad * SZ / 16, vc = a.kv.vdim_pad * TK_PAGE * SZ / 16; /* 16-byte pieces of a page */
    constexpr int KP = TK_PAGE * B * SZ / 16 / 256, VP = B * TK_PAGE * SZ / 16 / 256;
    tk_v4u kr[KP], vr[VP];
    auto fetch = [&](int i) {
        if (i - ids0 >= 64) {
            ids0 = i;
            ids = pages[walk.page(i + lane < walk.count ? i + lane : i)];
        }
        const size_t page = (size_t)__builtin_amdgcn_readlane(ids, i - ids0) * a.kv_heads + kvh;
        const uint8_t* kp = (const uint8_t*)a.kv.k + page * TK_PAGE * a.kv.dim_pad * SZ;
        const uint8_t* vp = (const uint8_t*)a.kv.v + page * a.kv.vdim_pad * TK_PAGE * SZ;
#pragma unroll
        for (int c = 0; c < KP; ++c) { const int p = threadIdx.x + 256 * c; if (FULL || p < kc) kr[c] = *(const tk_v4u*)(kp + (size_t)p * 16); }
#pragma unroll
        for (int c = 0; c < VP; ++c) { const int p = threadIdx.x + 256 * c; if (FULL || p < vc) vr[c] = *(const tk_v4u*)(vp + (size_t)p * 16); }
    };
    const int kpr = FULL ? B * SZ / 16 : a.kv.dim_pad * SZ / 16, vpr = TK_PAGE * SZ / 16; /* pieces of a row */
    auto put = [&](int i) {
        uint8_t *lk = lds + (TWO ? (i & 1) * buf : 0), *lv = lk + TK_PAGE * krow;
#pragma unroll
        for (int c = 0; c < KP; ++c) { const int p = threadIdx.x + 256 * c; if (FULL || p < kc) *(tk_v4u*)(lk + (p / kpr) * krow + (p % kpr) * 16) = kr[c]; }
#pragma unroll
        for (int c = 0; c < VP; ++c) { const int p = threadIdx.x + 256 * c; if (FULL || p < vc) *(tk_v4u*)(lv + (p / vpr) * vrow + (p % vpr) * 16) = vr[c]; }
    };
    fetch(0);
    tk_v4u qf[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d)
        if (d < nd) qf[d] = *(const tk_v4u*)((const uint8_t*)a.q + (((size_t)(row0 + live) * a.heads + h) * a.kv.dim_pad) * SZ + d * 64 + g * 16);
    Flash<T, VT> f;
    f.init();
    const int wave_lo = p0 + wave * 16, wave_hi = p0 + (wave * 16 + 15 < n ? wave * 16 + 15 : n - 1);
    /* what this lane's query reads from on, what any and what all of the wave's queries do (a wave with rows past the tile always masks) */
    const int first = pq >= 0 ? first_visible(a, pq) : 0, any = first_visible(a, wave_lo);
    const int whole = wave * 16 + 15 < n || (a.window <= 0 && a.chunk <= 0) ? first_visible(a, wave_hi) : 0x7fffffff;
    put(0);
    if (walk.count > 1) fetch(1);
    __syncthreads();
    for (int i = 0; i < walk.count; ++i) {
        if (i > 0) { /* page i is in its buffer; every wave is done with page i - 1 */
            if (!TWO) put(i);
            __syncthreads();
        }
        if (TWO) {
            if (i + 1 < walk.count) put(i + 1);
            if (i + 2 < walk.count) fetch(i + 2);
        } else if (i > 0 && i + 1 < walk.count) {
            fetch(i + 1);
        }
        const uint8_t *lk = lds + (TWO ? (i & 1) * buf : 0), *lv = lk + TK_PAGE * krow;
        const int k0 = walk.page(i) * TK_PAGE;
        /* not a page that none of this wave's rows reads */
        if (wave * 16 < n && k0 <= wave_hi && (any < k0 + TK_PAGE || k0 < a.keep_first)) {
            tk_v4f s[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                s[j] = tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
                const uint8_t* kp = lk + (16 * j + (lane & 15)) * krow + g * 16;
#pragma unroll
                for (int d = 0; d < DT; ++d)
                    if (d < nd) s[j] = TkImg<T>::mma(*(const tk_v4u*)(kp + d * 64), qf[d], s[j]);
            }
            mask_scores<T>(s, a, k0, g, pq, first, wave_lo, whole);
            f.update(s, nv, [&](int vt, int j) { return *(const VF*)(lv + (16 * vt + (lane & 15)) * vrow + (16 * j + 4 * g) * SZ); });
        }
        if (!TWO) __syncthreads(); /* the only buffer is free again */
    }
    if (q < n) attn_store<T, VT>(a, f.o, row0 + q, h, g, a.out_scale / f.l);
}

/* decoding: one row x up to 16 query heads of one kv head per workgroup, pages dealt to the waves (and to `splits` workgroups), merged in LDS */
template <typename T, int B, int WAVES, bool FULL>
__device__ __forceinline__ void attn_row(const TkAttnArgs& a, const TkPassTab& t, int block, int row, int split, int splits, float* scratch, uint8_t* lds) {
    constexpr int DT = B / TkImg<T>::KT, VT = B / 16, SZ = sizeof(T);
    constexpr bool AHEAD = SZ == 2 && B <= 128; /* a page's values are requested together with its keys */
    typedef typename VFrag<T>::type VF;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4;
    const int gq = a.heads / a.kv_heads, per = (gq + 15) / 16;
    const int kvh = block / per, q = (block % per) * 16 + (lane & 15);
    const int h = kvh * gq + (q < gq ? q : 0);
    const int nd = FULL ? DT : a.kv.dim_pad / TkImg<T>::KT, nv = FULL ? VT : a.kv.vdim_pad / 16;
    const int pos = t.pos[row], seq = t.seq[row];
    tk_v4u qf[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d)
        if (d < nd) qf[d] = *(const tk_v4u*)((const uint8_t*)a.q + (((size_t)row * a.heads + h) * a.kv.dim_pad) * SZ + d * 64 + g * 16);
    Flash<T, VT> f;
    f.init();
    const PageWalk walk(a, pos, pos);
    const int low = first_visible(a, pos);
    for (int i = split * WAVES + wave; i < walk.count; i += WAVES * splits) {
        const size_t page = (size_t)t.page_of[(size_t)seq * t.max_pages + walk.page(i)] * a.kv_heads + kvh;
        const uint8_t* kp = (const uint8_t*)a.kv.k + (page * TK_PAGE + (lane & 15)) * a.kv.dim_pad * SZ + g * 16;
        const uint8_t* vp = (const uint8_t*)a.kv.v + (page * a.kv.vdim_pad + (lane & 15)) * TK_PAGE * SZ + 4 * g * SZ;
        const int k0 = walk.page(i) * TK_PAGE;
        auto vload = [&](int vt, int j) { return *(const VF*)(vp + ((size_t)16 * vt * TK_PAGE + 16 * j) * SZ); };
        tk_v4u kf[AHEAD ? 4 : 1][AHEAD ? DT : 1];
        VF vf[AHEAD ? VT : 1][4];
        if (AHEAD) {
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int d = 0; d < DT; ++d)
                    if (d < nd) kf[j][d] = *(const tk_v4u*)(kp + (size_t)16 * j * a.kv.dim_pad * SZ + d * 64);
#pragma unroll
            for (int i2 = 0; i2 < VT; ++i2)
                if (i2 < nv)
#pragma unroll
                    for (int j = 0; j < 4; ++j) vf[i2][j] = vload(i2, j);
        }
        tk_v4f s[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            s[j] = tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int d = 0; d < DT; ++d)
                if (d < nd) s[j] = TkImg<T>::mma(AHEAD ? kf[AHEAD ? j : 0][AHEAD ? d : 0] : *(const tk_v4u*)(kp + (size_t)16 * j * a.kv.dim_pad * SZ + d * 64), qf[d], s[j]);
        }
        mask_scores<T>(s, a, k0, g, pos, low, pos, low);
        f.update(s, nv, [&](int vt, int j) { return AHEAD ? vf[AHEAD ? vt : 0][j] : vload(vt, j); });
    }
    /* the upper half of the waves into the lower half, and again */
    tk_v4f* so = (tk_v4f*)lds; /* [WAVES / 2][VT][64] */
    float *sm = (float*)(so + WAVES / 2 * VT * 64), *sl = sm + WAVES / 2 * 64;
#pragma unroll
    for (int half = WAVES / 2; half >= 1; half >>= 1) {
        if (wave >= half && wave < 2 * half) {
#pragma unroll
            for (int i = 0; i < VT; ++i) so[((wave - half) * VT + i) * 64 + lane] = f.o[i];
            sm[(wave - half) * 64 + lane] = f.m; sl[(wave - half) * 64 + lane] = f.l;
        }
        __syncthreads();
        if (wave < half) {
            const float m2 = sm[wave * 64 + lane], mn = fmaxf(f.m, m2), ms = mn == -INFINITY ? 0.0f : mn;
            const float c1 = __builtin_amdgcn_exp2f(f.m - ms), c2 = __builtin_amdgcn_exp2f(m2 - ms);
            f.l = f.l * c1 + sl[wave * 64 + lane] * c2;
            f.m = mn;
#pragma unroll
            for (int i = 0; i < VT; ++i) f.o[i] = f.o[i] * c1 + so[(wave * VT + i) * 64 + lane] * c2;
        }
        __syncthreads();
    }
    if (wave != 0 || q >= gq) return;
    if (splits == 1) { attn_store<T, VT>(a, f.o, row, h, g, a.out_scale / f.l); return; }
    float* out = scratch + (((size_t)row * a.heads + h) * splits + split) * (a.kv.vdim_pad + 2);
    if (g == 0) { out[0] = f.m; out[1] = f.l; }
#pragma unroll
    for (int i = 0; i < VT; ++i)
        if (i < nv)
#pragma unroll
            for (int r = 0; r < 4; ++r) out[2 + 16 * i + 4 * g + r] = f.o[i][r];
}
template <int B, int WAVES> constexpr size_t attn_row_lds() { return (size_t)WAVES / 2 * (B / 16 * 1024 + 512); }

template <typename T, int B, int WAVES, bool FULL>
__global__ __launch_bounds__(64 * WAVES, B == 256 ? 1 : 2) void k_attn_rows(TkAttnArgs a, TkPassTab t, int splits, float* scratch) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    attn_row<T, B, WAVES, FULL>(a, t, blockIdx.x, blockIdx.y, blockIdx.z, splits, scratch, lds);
}

template <typename T>
__global__ __launch_bounds__(64) void k_attn_merge(TkAttnArgs a, int splits, const float* scratch) {
    const int h = blockIdx.x, row = blockIdx.y, pitch = a.kv.vdim_pad + 2;
    const float* p = scratch + ((size_t)row * a.heads + h) * splits * pitch;
    float m = -INFINITY;
    for (int s = 0; s < splits; ++s) m = fmaxf(m, p[s * pitch]);
    float l = 0.0f;
    for (int s = 0; s < splits; ++s) l += p[s * pitch + 1] * __builtin_amdgcn_exp2f(p[s * pitch] - m);
    const float f = a.out_scale / l;
    for (int e = threadIdx.x; e < a.vdim; e += 64) {
        float y = 0.0f;
        for (int s = 0; s < splits; ++s) y += p[s * pitch + 2 + e] * __builtin_amdgcn_exp2f(p[s * pitch] - m);
        tk_img_put((T*)a.out_img, row, a.out_k0 + h * a.vdim + e, a.out_ktiles, y * f);
    }
}

/* ------------------------------------------------------------------ gated delta rule ------- */

/* A workgroup walks 4 * 64 / LN columns of one head's state through a segment; a column is LN lanes x RPL key rows, so its recurrence never
 * leaves the wave.  q, k, decays, v and step sizes of TC tokens at a time go through LDS, the next TC in flight in registers.  32 lanes a column
 * where columns are few (the shorter chain), 16 where they are many (fewer operand reads per column). */
template <int LN, int RPL>
__global__ __launch_bounds__(256) void k_delta_scan(TkDeltaArgs d, TkPassTab t) {
    constexpr int DP = LN * RPL, TC = DP > 128 ? 8 : 16, NL = TC * DP / 256, CW = 64 / LN, NC = 4 * CW;
    __shared__ __attribute__((aligned(16))) float lq[2][TC][DP], lk[2][TC][DP], lg[2][TC][DP];
    __shared__ float lv[2][TC][NC], lb[2][TC];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int h = blockIdx.y, seg = blockIdx.z, kvh = h / (d.heads / d.kv_heads), vp = (d.vdim + 3) & ~3;
    const int row0 = t.seg_row0[seg], n = t.seg_n[seg], in = t.seg_in[seg], out = t.seg_out[seg];
    const int cl = wave * CW + lane / LN, col = blockIdx.x * NC + cl, r0 = (lane % LN) * RPL;
    const bool live = col < d.vdim;
    float S[RPL];
#pragma unroll
    for (int i = 0; i < RPL; ++i)
        S[i] = in >= 0 && live && r0 + i < d.dim ? d.state[(((size_t)in * d.heads + h) * d.dim + r0 + i) * vp + col] : 0.0f;
    float rq[NL], rk[NL], rg[NL], rv = 0.0f, rb = 0.0f;
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NL; ++i) {
            const int idx = tid + 256 * i, tt = t0 + idx / DP, e = idx % DP;
            const bool ok = tt < n && e < d.dim;
            const size_t row = row0 + (ok ? tt : 0);
            rq[i] = ok ? d.q[(row * d.kv_heads + kvh) * d.dim + e] : 0.0f;
            rk[i] = ok ? d.k[(row * d.kv_heads + kvh) * d.dim + e] : 0.0f;
            rg[i] = ok ? d.g[(row * d.heads + h) * d.dim + e] : 1.0f;
        }
        if (tid < TC * NC) {
            const int tt = t0 + tid / NC, c = blockIdx.x * NC + tid % NC;
            rv = tt < n && c < d.vdim ? d.v[((size_t)(row0 + tt) * d.heads + h) * d.vdim + c] : 0.0f;
        }
        if (tid < TC) rb = t0 + tid < n ? d.beta[(size_t)(row0 + t0 + tid) * d.heads + h] : 0.0f;
    };
    auto put = [&](int b) {
#pragma unroll
        for (int i = 0; i < NL; ++i) {
            const int idx = tid + 256 * i;
            (&lq[b][0][0])[idx] = rq[i]; (&lk[b][0][0])[idx] = rk[i]; (&lg[b][0][0])[idx] = rg[i];
        }
        if (tid < TC * NC) lv[b][tid / NC][tid % NC] = rv;
        if (tid < TC) lb[b][tid] = rb;
    };
    fetch(0);
    put(0);
    __syncthreads();
    for (int t0 = 0, b = 0; t0 < n; t0 += TC, b ^= 1) {
        if (t0 + TC < n) fetch(t0 + TC);
        const int m = n - t0 < TC ? n - t0 : TC;
        for (int i = 0; i < m; ++i) {
            float sk = 0.0f, so = 0.0f;
#pragma unroll
            for (int e = 0; e < RPL; ++e) { S[e] *= lg[b][i][r0 + e]; sk = fmaf(S[e], lk[b][i][r0 + e], sk); }
            sk = LN == 16 ? tk_row16_sum(sk) : tk_row32_sum(sk);
            const float u = lb[b][i] * (lv[b][i][cl] - sk);
#pragma unroll
            for (int e = 0; e < RPL; ++e) { S[e] = fmaf(lk[b][i][r0 + e], u, S[e]); so = fmaf(S[e], lq[b][i][r0 + e], so); }
            so = LN == 16 ? tk_row16_sum(so) : tk_row32_sum(so);
            if (lane % LN == 0 && live) d.o[((size_t)(row0 + t0 + i) * d.heads + h) * d.vdim + col] = so;
        }
        if (t0 + TC < n) put(b ^ 1); /* the other buffer was last read one iteration ago, before the barrier below */
        __syncthreads();
    }
    if (live)
#pragma unroll
        for (int i = 0; i < RPL; ++i)
            if (r0 + i < d.dim) d.state[(((size_t)out * d.heads + h) * d.dim + r0 + i) * vp + col] = S[i];
}

/* o over its root mean square, times the norm's weight, times the gate: one wave per (row, head) */
template <typename T>
__global__ __launch_bounds__(256) void k_delta_out(TkDeltaArgs d) {
    const int lane = threadIdx.x & 63, h = blockIdx.x * 4 + (threadIdx.x >> 6), row = blockIdx.y;
    if (h >= d.heads) return;
    const float* o = d.o + ((size_t)row * d.heads + h) * d.vdim;
    float v[4], ss = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; ++i) { const int e = lane + 64 * i; v[i] = e < d.vdim ? o[e] : 0.0f; ss += v[i] * v[i]; }
    const float r = 1.0f / sqrtf(tk_wave_sum(ss) / (float)d.vdim + d.eps);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int e = lane + 64 * i;
        if (e >= d.vdim) break;
        const float gate = tk_sigmoid32(d.low[(size_t)row * d.low_ld + d.low_g + h * d.vdim + e]);
        tk_img_put((T*)d.out_img, row, d.out_k0 + h * d.vdim + e, d.out_ktiles, v[i] * r * d.norm[e] * gate * d.out_scale);
    }
}

/* one token of one head: the state is read once and written once, a thread holds RPT rows x 4 columns of it.
 * o = S_new^T q = (g S)^T q + (k . q) u, so both reductions over the key rows run on the decayed old state at once. */
template <typename T, int THREADS, int RPT>
__device__ __forceinline__ void delta_row(const TkDeltaArgs& d, const TkPassTab& t, int h, int row, int ct_log2, float* step_lds) {
    const int tid = threadIdx.x, kvh = h / (d.heads / d.kv_heads), vp = (d.vdim + 3) & ~3;
    const int ct = tid & ((1 << ct_log2) - 1), rg = tid >> ct_log2, RG = THREADS >> ct_log2;
    const bool live = 4 * ct < vp;
    const int seg = t.seg[row], in = t.seg_in[seg], out = t.seg_out[seg];
    float *red = step_lds, *lq = red + 16, *lk = lq + d.dim, *lg = lk + d.dim, *lu = red + 16 + (3 * d.dim + 3) / 4 * 4, *pk = lu + vp, *pq = pk + RG * vp;
    tk_v4f S[RPT];
    const float* sin = d.state + ((size_t)(in < 0 ? 0 : in) * d.heads + h) * d.dim * vp + 4 * ct;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int e = rg + RG * i;
        S[i] = in >= 0 && live && e < d.dim ? *(const tk_v4f*)(sin + (size_t)e * vp) : tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
    }
    float kq = 0.0f;
    for (int e = tid; e < d.dim; e += THREADS) {
        const float q = d.q[((size_t)row * d.kv_heads + kvh) * d.dim + e], k = d.k[((size_t)row * d.kv_heads + kvh) * d.dim + e];
        lq[e] = q; lk[e] = k; lg[e] = d.g[((size_t)row * d.heads + h) * d.dim + e];
        kq += q * k;
    }
    kq = block_sum(kq, red); /* also orders the LDS writes above before the reads below */
    tk_v4f ak = {0.0f, 0.0f, 0.0f, 0.0f}, aq = ak;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int e = rg + RG * i;
        if (e < d.dim) { S[i] *= lg[e]; ak += S[i] * lk[e]; aq += S[i] * lq[e]; }
    }
    if (live) { *(tk_v4f*)(pk + rg * vp + 4 * ct) = ak; *(tk_v4f*)(pq + rg * vp + 4 * ct) = aq; }
    __syncthreads();
    const float beta = d.beta[(size_t)row * d.heads + h];
    float o = 0.0f, ss = 0.0f;
    if (tid < vp) { /* vdim <= 256 <= THREADS: one column per thread */
        float sk = 0.0f, sq = 0.0f;
        for (int i = 0; i < RG; ++i) { sk += pk[i * vp + tid]; sq += pq[i * vp + tid]; }
        const float v = tid < d.vdim ? d.v[((size_t)row * d.heads + h) * d.vdim + tid] : 0.0f;
        const float u = tid < d.vdim ? beta * (v - sk) : 0.0f;
        lu[tid] = u;
        o = tid < d.vdim ? sq + kq * u : 0.0f;
        ss = o * o;
    }
    ss = block_sum(ss, red);
    if (live) {
        const tk_v4f u = *(const tk_v4f*)(lu + 4 * ct);
        float* so = d.state + ((size_t)out * d.heads + h) * d.dim * vp + 4 * ct;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const int e = rg + RG * i;
            if (e < d.dim) *(tk_v4f*)(so + (size_t)e * vp) = S[i] + u * lk[e];
        }
    }
    if (tid < d.vdim) {
        const float r = 1.0f / sqrtf(ss / (float)d.vdim + d.eps);
        const float gate = tk_sigmoid32(d.low[(size_t)row * d.low_ld + d.low_g + h * d.vdim + tid]);
        tk_img_put((T*)d.out_img, row, d.out_k0 + h * d.vdim + tid, d.out_ktiles, o * r * d.norm[tid] * gate * d.out_scale);
    }
}

static size_t delta_row_lds(const TkDeltaArgs& d, int threads, int ct_log2) {
    const size_t vp = (d.vdim + 3) & ~3;
    return (16 + (size_t)(3 * d.dim + 3) / 4 * 4 + vp + 2 * (size_t)(threads >> ct_log2) * vp) * sizeof(float);
}

template <typename T, int THREADS, int RPT>
__global__ __launch_bounds__(THREADS) void k_delta_step(TkDeltaArgs d, TkPassTab t, int ct_log2) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    delta_row<T, THREADS, RPT>(d, t, blockIdx.x, blockIdx.y, ct_log2, (float*)lds);
}

/* a decode step's attention and delta rule side by side: the first na workgroups of a row are attention's, the others one delta head each */
template <typename T, int B, int WAVES, int RPT, bool FULL>
__global__ __launch_bounds__(64 * WAVES, 2) void k_mixers_step(TkAttnArgs a, TkDeltaArgs d, TkPassTab t, int na, int ct_log2) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    if ((int)blockIdx.x < na) attn_row<T, B, WAVES, FULL>(a, t, blockIdx.x, blockIdx.y, 0, 1, nullptr, lds);
    else delta_row<T, 64 * WAVES, RPT>(d, t, blockIdx.x - na, blockIdx.y, ct_log2, (float*)lds);
}

__global__ void k_swap_state(TkPassTab t, int n) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) { const int o = t.seg_out[i]; t.seg_in[i] = o; t.seg_out[i] = o ^ 1; }
}

/* ------------------------------------------------------------------ retention -------------- */

/* Prompts.  With pw(n) = decay^n, a chunk of up to C tokens that starts from the state S0 gives
 *     o_i = pw(i + 1) S0^T q_i + sum over j <= i of pw(i - j) (q_i . k_j) v_j,      S = pw(n) S0 + sum over j of pw(n - 1 - j) k_j v_j^T:
 * four matrix products.  A workgroup walks one head's block of rows; every wave owns NT 16-column tiles of the state, in the registers that the
 * products leave it in: an accumulator tile [key dimension][value column] is at once the operand of S^T q, because the key dimensions of q (and k)
 * lie in LDS in the order in which a lane's accumulators hold them.  Scores go through LDS.  bf16 sessions: v is bf16; what is 32-bit (rotated q and
 * k, the state, decayed scores and values) enters a product as the sum of two bf16 numbers, without the product of the two small parts.
 * SUMS: only what the block adds to the state, into args.sums; k_retention_prefix turns these into the states that the segment's next blocks start
 * from, so that all blocks run side by side. */
template <typename T> struct RetChunk { static constexpr int C = 32; };

/* where element e of a key row lies: see above (f32 accumulators are in order already) */
template <typename T> __device__ __forceinline__ int ret_place(int e) { return sizeof(T) == 2 ? (e & ~31) | (e & 12) << 1 | (e & 16) >> 2 | (e & 3) : e; }

/* x as operand words: one bf16 pair per word, hi and the rest lo; f32 as it is (lo unused) */
template <typename T> struct Split;
template <> struct Split<TkBf16> {
    tk_v4u hi, lo;
    __device__ __forceinline__ Split(tk_v4f a, tk_v4f b) {
        const float x[8] = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const uint16_t p = tk_bf16_bits(x[2 * i]), q = tk_bf16_bits(x[2 * i + 1]);
            hi[i] = (uint32_t)p | (uint32_t)q << 16;
            lo[i] = (uint32_t)tk_bf16_bits(x[2 * i] - tk_bf16_float(p)) | (uint32_t)tk_bf16_bits(x[2 * i + 1] - tk_bf16_float(q)) << 16;
        }
    }
};

/* a gate on its way into a bf16 image needs no more than the hardware's exponential and reciprocal (1e-7) */
template <typename T> __device__ __forceinline__ float silu_out(float z) { return sizeof(T) == 4 ? tk_silu32(z) : z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-LOG2E * z)); }

template <typename T, int DIM, int VB>
struct RetLds { /* byte offsets */
    static constexpr int C = RetChunk<T>::C, SZ = sizeof(T), RP = DIM * SZ + 16, TP = C * SZ + 16;
    /* the small parts (bf16) lie behind the large ones */
    static constexpr int PARTS = SZ == 2 ? 2 : 1, q_lo = C * RP, k_lo = C * RP, kt_lo = DIM * TP, p_lo = C * TP;
    static constexpr int q = 0, k = q + PARTS * q_lo, kt = k + PARTS * k_lo, vt = kt + PARTS * kt_lo, p = vt + VB * TP, pw = p + PARTS * p_lo,
                         red = pw + (TK_RETENTION_BLOCK + 4) * 4, bytes = red + 8 * C * 4; /* eight waves at most */
};

/* four tokens' elements side by side, and their small parts */
__device__ __forceinline__ void ret_put4(TkBf16* p, const float (&x)[4]) {
    *(tk_v2u*)p = tk_v2u{(uint32_t)tk_bf16_bits(x[0]) | (uint32_t)tk_bf16_bits(x[1]) << 16, (uint32_t)tk_bf16_bits(x[2]) | (uint32_t)tk_bf16_bits(x[3]) << 16};
}
__device__ __forceinline__ void ret_put4(float* p, const float (&x)[4]) { *(tk_v4f*)p = tk_v4f{x[0], x[1], x[2], x[3]}; }
__device__ __forceinline__ float ret_rest(float x) { return x - tk_bf16_float(tk_bf16_bits(x)); }
__device__ __forceinline__ void ret_put4_split(uint8_t* p, int lo, TkBf16, const float (&x)[4]) {
    const float y[4] = {ret_rest(x[0]), ret_rest(x[1]), ret_rest(x[2]), ret_rest(x[3])};
    ret_put4((TkBf16*)p, x);
    ret_put4((TkBf16*)(p + lo), y);
}
__device__ __forceinline__ void ret_put4_split(uint8_t* p, int, float, const float (&x)[4]) { ret_put4((float*)p, x); }
__device__ __forceinline__ void ret_put_split(uint8_t* p, int lo, TkBf16, float x) { *(uint16_t*)p = tk_bf16_bits(x); *(uint16_t*)(p + lo) = tk_bf16_bits(ret_rest(x)); }
__device__ __forceinline__ void ret_put_split(uint8_t* p, int, float, float x) { *(float*)p = x; }

template <typename T, int DIM, int WAVES, int NT, bool SUMS>
__global__ __launch_bounds__(64 * WAVES, SUMS && DIM <= 128 && NT == 1 ? 4 : 2) void k_retention_scan(TkRetentionArgs a, const float* proj, int ld, TkPassTab t, const TkRetentionBlock* blocks) {
    constexpr int C = RetChunk<T>::C, KT = TkImg<T>::KT, EP = TkImg<T>::EP, SZ = sizeof(T), THREADS = 64 * WAVES, VB = 16 * WAVES * NT;
    constexpr int DT = DIM / KT, DS = DIM / 16, CT = C / 16, CK = C / KT;
    typedef RetLds<T, DIM, VB> L;
    static_assert(WAVES <= 8 && L::bytes <= 160 * 1024, "a chunk fits the LDS");
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, r16 = lane & 15;
    /* workgroups go to the eight XCDs in turn, and the L2 slices of one repeat every 4 KiB of a row: an XCD's heads lie side by side, other ones in the next block */
    const int per = a.heads / 8, h = a.heads % 8 ? blockIdx.x : (blockIdx.x % 8 * per + blockIdx.x / 8 + blockIdx.y * per) % a.heads;
    const TkRetentionBlock b = blocks[blockIdx.y];
    if (SUMS && b.last) return;
    const int vp = (a.vdim + 3) & ~3, in = t.seg_in[b.seg], pos0 = t.pos[b.row0];
    const size_t head_floats = (size_t)a.dim * vp;
    for (int i = tid; i < L::bytes / 16; i += THREADS) *(tk_v4u*)(lds + i * 16) = tk_v4u{0, 0, 0, 0}; /* paddings stay zero */
    __syncthreads();
    float *pw = (float*)(lds + L::pw), *red = (float*)(lds + L::red);
    if (tid <= TK_RETENTION_BLOCK) pw[tid] = a.decay[(size_t)h * (TK_RETENTION_BLOCK + 1) + tid];
    int col[NT]; /* this lane's value columns */
#pragma unroll
    for (int n = 0; n < NT; ++n) col[n] = (wave * NT + n) * 16 + r16;
    tk_v4f S[NT][DS]; /* [key dimension 16 d + 4 g + r][column col[n]] */
    auto state_at = [&](float* base, auto f) {
#pragma unroll
        for (int n = 0; n < NT; ++n)
#pragma unroll
            for (int d = 0; d < DS; ++d)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int e = 16 * d + 4 * g + r;
                    if (e < a.dim && col[n] < a.vdim) S[n][d][r] = f(S[n][d][r], base[(size_t)e * vp + col[n]]);
                }
    };
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int d = 0; d < DS; ++d) S[n][d] = tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
    if (!SUMS) {
        if (b.index > 0) state_at(a.sums + ((size_t)(b.slot0 + b.index - 1) * a.heads + h) * head_floats, [](float, float& m) { return m; });
        else if (in >= 0) state_at(a.state + ((size_t)in * a.heads + h) * head_floats, [](float, float& m) { return m; });
    }
    const int half = a.rot_dims / 2, units = (a.dim + 1) / 2, qk = a.heads * a.dim;
    const float kscale = 1.0f / sqrtf((float)a.dim);
    const float *qp = proj + a.col + h * a.dim, *kp = qp + qk, *vsrc = proj + a.col + 2 * qk + h * a.vdim, *gsrc = vsrc + a.heads * a.vdim;
    /* a thread's share of a chunk, four tokens at a time: pairs of key dimensions (rotation partners, or neighbours among those that do not turn) and
     * value columns.  Small heads: the next chunk's is on its way to registers while one is used. */
    constexpr int QI = (DIM / 2 * (C / 4) + THREADS - 1) / THREADS, VI = VB * (C / 4) / THREADS;
    float q0[QI][4], q1[QI][4], k0[QI][4], k1[QI][4], cs[QI][4], sn[QI][4], vv[VI][4];
    auto fetch = [&](int c0) {
        const int n = b.n - c0 < C ? b.n - c0 : C, base = b.row0 + c0;
#pragma unroll
        for (int i = 0; i < QI; ++i) {
            const int it = tid + i * THREADS, u = it % (DIM / 2) < units ? it % (DIM / 2) : units - 1, t0 = it / (DIM / 2) * 4;
            const int e0 = u < half ? u : 2 * u, e1 = u < half ? u + half : 2 * u + 1 < a.dim ? 2 * u + 1 : 2 * u;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const size_t row = (size_t)(base + (t0 + r < n ? t0 + r : n - 1)) * ld;
                if (!SUMS) { q0[i][r] = qp[row + e0]; q1[i][r] = qp[row + e1]; }
                k0[i][r] = kp[row + e0];
                k1[i][r] = kp[row + e1];
            }
            if (half > 0)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const size_t at = (size_t)(pos0 + c0 + (t0 + r < n ? t0 + r : n - 1)) * half + (u < half ? u : 0);
                    cs[i][r] = a.rope_cos[at];
                    sn[i][r] = a.rope_sin[at];
                }
        }
#pragma unroll
        for (int i = 0; i < VI; ++i) {
            const int it = tid + i * THREADS, e = it % VB < a.vdim ? it % VB : a.vdim - 1, t0 = it / VB * 4;
#pragma unroll
            for (int r = 0; r < 4; ++r) vv[i][r] = vsrc[(size_t)(base + (t0 + r < n ? t0 + r : n - 1)) * ld + e];
        }
    };
    auto put = [&](int n) {
#pragma unroll
        for (int i = 0; i < QI; ++i) {
            const int it = tid + i * THREADS, u = it % (DIM / 2), t0 = it / (DIM / 2) * 4;
            if (u >= units || t0 >= C) break;
            const bool turns = u < half, two = turns || 2 * u + 1 < a.dim;
            const int e0 = turns ? u : 2 * u, e1 = turns ? u + half : two ? 2 * u + 1 : 2 * u;
            float ka[4], kb[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const bool ok = t0 + r < n;
                const float c = turns ? cs[i][r] : 1.0f, z = turns ? sn[i][r] : 0.0f;
                ka[r] = ok ? (k0[i][r] * c - k1[i][r] * z) * kscale : 0.0f;
                kb[r] = ok ? (k1[i][r] * c + k0[i][r] * z) * kscale : 0.0f;
                if (!SUMS) {
                    uint8_t *at0 = lds + (t0 + r) * L::RP + ret_place<T>(e0) * SZ, *at1 = lds + (t0 + r) * L::RP + ret_place<T>(e1) * SZ;
                    ret_put_split(at0 + L::q, L::q_lo, T(), q0[i][r] * c - q1[i][r] * z);
                    ret_put_split(at0 + L::k, L::k_lo, T(), ka[r]);
                    if (two) {
                        ret_put_split(at1 + L::q, L::q_lo, T(), q1[i][r] * c + q0[i][r] * z);
                        ret_put_split(at1 + L::k, L::k_lo, T(), kb[r]);
                    }
                }
            }
            ret_put4_split(lds + L::kt + e0 * L::TP + t0 * SZ, L::kt_lo, T(), ka);
            if (two) ret_put4_split(lds + L::kt + e1 * L::TP + t0 * SZ, L::kt_lo, T(), kb);
        }
#pragma unroll
        for (int i = 0; i < VI; ++i) {
            const int it = tid + i * THREADS, e = it % VB, t0 = it / VB * 4;
            float v[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = t0 + r < n ? vv[i][r] : 0.0f;
            if (e < a.vdim) ret_put4((T*)(lds + L::vt + e * L::TP) + t0, v);
        }
    };
    constexpr bool AHEAD = NT * DIM <= 128; /* as many registers as that takes are free */
    if (AHEAD) fetch(0);
    for (int c0 = 0; c0 < b.n; c0 += C) {
        const int n = b.n - c0 < C ? b.n - c0 : C, base = b.row0 + c0;
        const bool more = c0 + C < b.n;
        if (!AHEAD) fetch(c0);
        put(n);
        __syncthreads();
        if (AHEAD && more) fetch(c0 + C);
        tk_v4f gate[SUMS ? 1 : NT][SUMS ? 1 : CT];
        if constexpr (!SUMS) {
            const bool vec = ((uintptr_t)gsrc & 15) == 0 && (ld & 3) == 0 && (a.vdim & 3) == 0;
#pragma unroll
            for (int m = 0; m < CT; ++m)
#pragma unroll
                for (int nt = 0; nt < NT; ++nt) {
                    const int e = (wave * NT + nt) * 16 + 4 * g;
                    const float* gp = gsrc + (size_t)(base + (16 * m + r16 < n ? 16 * m + r16 : n - 1)) * ld;
                    if (vec) gate[nt][m] = *(const tk_v4f*)(gp + (e < a.vdim ? e : 0));
                    else
#pragma unroll
                        for (int r = 0; r < 4; ++r) gate[nt][m][r] = gp[e + r < a.vdim ? e + r : 0];
                }
        }
        tk_v4f o[SUMS ? 1 : NT][SUMS ? 1 : CT]; /* [column 4 g + r of tile n][query 16 m + lane % 16] */
        if constexpr (!SUMS) {
            /* ---- decayed scores, tiles of 16 queries x 16 keys dealt to the waves ---- */
            for (int i = wave; i < CT * (CT + 1) / 2; i += WAVES) {
                const int m = i < 1 ? 0 : i < 3 ? 1 : i < 6 ? 2 : 3, j = i - m * (m + 1) / 2;
                if (16 * m >= n) continue;
                tk_v4f s = {0.0f, 0.0f, 0.0f, 0.0f};
                const uint8_t *lk = lds + L::k + (16 * j + r16) * L::RP + g * 16, *lq = lds + L::q + (16 * m + r16) * L::RP + g * 16;
#pragma unroll
                for (int d = 0; d < DT; ++d) {
                    const tk_v4u kf = *(const tk_v4u*)(lk + d * 64), qf = *(const tk_v4u*)(lq + d * 64);
                    s = TkImg<T>::mma(kf, qf, s);
                    if constexpr (SZ == 2) {
                        s = TkImg<T>::mma(*(const tk_v4u*)(lk + L::k_lo + d * 64), qf, s);
                        s = TkImg<T>::mma(kf, *(const tk_v4u*)(lq + L::q_lo + d * 64), s);
                    }
                }
                const int age = 16 * (m - j) + r16 - 4 * g;
#pragma unroll
                for (int r = 0; r < 4; ++r) s[r] = age - r >= 0 ? s[r] * pw[age - r >= 0 ? age - r : 0] : 0.0f;
                const int at = (16 * m + r16) * L::TP + (16 * j + 4 * g) * SZ;
                if constexpr (SZ == 2) {
                    const Split<TkBf16> w(s, s);
                    *(tk_v2u*)(lds + L::p + at) = tk_v2u{w.hi[0], w.hi[1]};
                    *(tk_v2u*)(lds + L::p + L::p_lo + at) = tk_v2u{w.lo[0], w.lo[1]};
                } else {
                    *(tk_v4f*)(lds + L::p + at) = s;
                }
            }
            /* ---- what the state gives ---- */
#pragma unroll
            for (int nt = 0; nt < NT; ++nt)
#pragma unroll
                for (int m = 0; m < CT; ++m) o[nt][m] = tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
            if (in >= 0 || b.index > 0 || c0 > 0) {
#pragma unroll
                for (int d = 0; d < DT; ++d) {
                    tk_v4u qf[CT];
#pragma unroll
                    for (int m = 0; m < CT; ++m) qf[m] = *(const tk_v4u*)(lds + L::q + (16 * m + r16) * L::RP + d * 64 + g * 16);
#pragma unroll
                    for (int nt = 0; nt < NT; ++nt) {
                        if constexpr (SZ == 2) {
                            const Split<TkBf16> w(S[nt][2 * d], S[nt][2 * d + 1]);
#pragma unroll
                            for (int m = 0; m < CT; ++m) {
                                o[nt][m] = TkImg<T>::mma(w.hi, qf[m], o[nt][m]);
                                o[nt][m] = TkImg<T>::mma(w.lo, qf[m], o[nt][m]);
                                o[nt][m] = TkImg<T>::mma(w.hi, *(const tk_v4u*)(lds + L::q + L::q_lo + (16 * m + r16) * L::RP + d * 64 + g * 16), o[nt][m]);
                            }
                        } else {
#pragma unroll
                            for (int m = 0; m < CT; ++m) o[nt][m] = TkImg<T>::mma(__builtin_bit_cast(tk_v4u, S[nt][d]), qf[m], o[nt][m]);
                        }
                    }
                }
#pragma unroll
                for (int m = 0; m < CT; ++m) {
                    const float f = pw[16 * m + r16 + 1];
#pragma unroll
                    for (int nt = 0; nt < NT; ++nt) o[nt][m] *= f;
                }
            }
            __syncthreads();
        }
        /* ---- what the chunk's own tokens give, and the state after them ---- */
        tk_v4u vf[NT][CK];
#pragma unroll
        for (int nt = 0; nt < NT; ++nt)
#pragma unroll
            for (int k = 0; k < CK; ++k) vf[nt][k] = *(const tk_v4u*)(lds + L::vt + col[nt] * L::TP + k * 64 + g * 16);
        if constexpr (!SUMS) {
#pragma unroll
            for (int k = 0; k < CK; ++k)
#pragma unroll
                for (int m = 0; m < CT; ++m)
                    if (k * KT < 16 * m + 16) {
                        const int at = (16 * m + r16) * L::TP + k * 64 + g * 16;
                        const tk_v4u hi = *(const tk_v4u*)(lds + L::p + at), lo = SZ == 2 ? *(const tk_v4u*)(lds + L::p + L::p_lo + at) : hi;
#pragma unroll
                        for (int nt = 0; nt < NT; ++nt) {
                            o[nt][m] = TkImg<T>::mma(vf[nt][k], hi, o[nt][m]);
                            if (SZ == 2) o[nt][m] = TkImg<T>::mma(vf[nt][k], lo, o[nt][m]);
                        }
                    }
        }
        if (SUMS || more || b.last) {
            const float fade = pw[n];
#pragma unroll
            for (int nt = 0; nt < NT; ++nt)
#pragma unroll
                for (int d = 0; d < DS; ++d) S[nt][d] *= fade;
#pragma unroll
            for (int k = 0; k < CK; ++k) {
                float w[EP];
#pragma unroll
                for (int e = 0; e < EP; ++e) { const int left = n - 1 - (k * KT + g * EP + e); w[e] = pw[left >= 0 ? left : 0]; } /* past n: v is zero */
                if constexpr (SZ == 2) {
                    tk_v4u hi[NT], lo[NT];
#pragma unroll
                    for (int nt = 0; nt < NT; ++nt) {
                        tk_v4f x, y;
#pragma unroll
                        for (int e = 0; e < 4; ++e) {
                            x[e] = tk_bf16_float((uint16_t)(vf[nt][k][e >> 1] >> 16 * (e & 1))) * w[e];
                            y[e] = tk_bf16_float((uint16_t)(vf[nt][k][2 + (e >> 1)] >> 16 * (e & 1))) * w[EP - 4 + e];
                        }
                        const Split<TkBf16> z(x, y);
                        hi[nt] = z.hi; lo[nt] = z.lo;
                    }
#pragma unroll
                    for (int d = 0; d < DS; ++d) {
                        const uint8_t* kat = lds + L::kt + (16 * d + r16) * L::TP + k * 64 + g * 16;
                        const tk_v4u kf = *(const tk_v4u*)kat, kl = *(const tk_v4u*)(kat + L::kt_lo);
#pragma unroll
                        for (int nt = 0; nt < NT; ++nt) {
                            S[nt][d] = TkImg<T>::mma(kf, hi[nt], S[nt][d]);
                            S[nt][d] = TkImg<T>::mma(kf, lo[nt], S[nt][d]);
                            S[nt][d] = TkImg<T>::mma(kl, hi[nt], S[nt][d]);
                        }
                    }
                } else {
                    tk_v4f x[NT];
#pragma unroll
                    for (int nt = 0; nt < NT; ++nt) {
                        x[nt] = __builtin_bit_cast(tk_v4f, vf[nt][k]);
#pragma unroll
                        for (int e = 0; e < 4; ++e) x[nt][e] *= w[e];
                    }
#pragma unroll
                    for (int d = 0; d < DS; ++d) {
                        const tk_v4u kf = *(const tk_v4u*)(lds + L::kt + (16 * d + r16) * L::TP + k * 64 + g * 16);
#pragma unroll
                        for (int nt = 0; nt < NT; ++nt) S[nt][d] = TkImg<T>::mma(kf, __builtin_bit_cast(tk_v4u, x[nt]), S[nt][d]);
                    }
                }
            }
        }
        if constexpr (!SUMS) {
            /* ---- each head's output over its root mean square, times the gate ---- */
#pragma unroll
            for (int m = 0; m < CT; ++m) {
                float ss = 0.0f;
#pragma unroll
                for (int nt = 0; nt < NT; ++nt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) ss += o[nt][m][r] * o[nt][m][r];
                ss = tk_quad_sum(ss);
                if (g == 0) red[wave * C + 16 * m + r16] = ss;
            }
            __syncthreads();
#pragma unroll
            for (int m = 0; m < CT; ++m) {
                const int i = 16 * m + r16;
                float ss = 0.0f;
#pragma unroll
                for (int w = 0; w < WAVES; ++w) ss += red[w * C + i];
                if (i >= n) continue;
                const float f = a.out_scale / sqrtf(ss / (float)a.vdim + a.eps);
                const int64_t row = base + i;
#pragma unroll
                for (int nt = 0; nt < NT; ++nt) {
                    const int e = (wave * NT + nt) * 16 + 4 * g, at = a.out_k0 + h * a.vdim + e;
                    if (e >= a.vdim) continue;
                    tk_v4f y;
#pragma unroll
                    for (int r = 0; r < 4; ++r) y[r] = o[nt][m][r] * f * silu_out<T>(gate[nt][m][r]);
                    if ((at & 3) == 0 && e + 3 < a.vdim) tk_img_put4((T*)a.out_img, row, at, a.out_ktiles, y);
                    else
#pragma unroll
                        for (int r = 0; r < 4; ++r)
                            if (e + r < a.vdim) tk_img_put((T*)a.out_img, row, at + r, a.out_ktiles, y[r]);
                }
            }
        } else {
            __syncthreads(); /* the next chunk takes the operands' place (outputs: every wave is past them at the barrier above) */
        }
    }
    if (SUMS) state_at(a.sums + ((size_t)(b.slot0 + b.index) * a.heads + h) * head_floats, [](float s, float& m) { return m = s; });
    else if (b.last) state_at(a.state + ((size_t)t.seg_out[b.seg] * a.heads + h) * head_floats, [](float s, float& m) { return m = s; });
}

/* sums of a segment's blocks -> the state behind each of them; one thread per element of a head's state */
__global__ __launch_bounds__(256) void k_retention_prefix(TkRetentionArgs a, TkPassTab t, const TkRetentionBlock* blocks) {
    const TkRetentionBlock b = blocks[blockIdx.z];
    if (b.index > 0 || b.last) return;
    const int vp = (a.vdim + 3) & ~3, h = blockIdx.y, i = (blockIdx.x * 256 + threadIdx.x) * 4, in = t.seg_in[b.seg], nb = (t.seg_n[b.seg] + b.n - 1) / b.n;
    const size_t head_floats = (size_t)a.dim * vp;
    if (i >= (int)head_floats) return;
    const float step = a.decay[(size_t)h * (TK_RETENTION_BLOCK + 1) + TK_RETENTION_BLOCK];
    float fade = 1.0f; /* over a block */
    for (int n = 0; n < b.n; n += TK_RETENTION_BLOCK) fade *= step;
    tk_v4f S = in >= 0 ? *(const tk_v4f*)(a.state + ((size_t)in * a.heads + h) * head_floats + i) : tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
    float* p = a.sums + ((size_t)b.slot0 * a.heads + h) * head_floats + i;
    const size_t pitch = a.heads * head_floats;
    for (int k = 0; k + 1 < nb; k += 8) {
        tk_v4f m[8]; /* loads ahead of the chain */
#pragma unroll
        for (int j = 0; j < 8; ++j)
            if (k + j + 1 < nb) m[j] = *(const tk_v4f*)(p + (k + j) * pitch);
#pragma unroll
        for (int j = 0; j < 8; ++j)
            if (k + j + 1 < nb) { S = S * fade + m[j]; *(tk_v4f*)(p + (k + j) * pitch) = S; }
    }
}

/* One token of one head: the state is read once and written once, a thread holds RPT rows x 4 columns of it.  Rotation, output norm and gate with it. */
template <typename T, int THREADS, int RPT>
__global__ __launch_bounds__(THREADS) void k_retention_step(TkRetentionArgs a, const float* proj, int ld, TkPassTab t, int ct_log2) {
    extern __shared__ __attribute__((aligned(16))) float ret_lds[];
    const int h = blockIdx.x, seg = blockIdx.y, tid = threadIdx.x, vp = (a.vdim + 3) & ~3;
    if (t.seg_n[seg] != 1) return;
    const int row = t.seg_row0[seg], in = t.seg_in[seg], out = t.seg_out[seg], pos = t.pos[row];
    const int ct = tid & ((1 << ct_log2) - 1), rg = tid >> ct_log2, RG = THREADS >> ct_log2;
    const bool live = 4 * ct < vp;
    float *red = ret_lds, *lv = red + 16, *po = lv + vp, *lq = po + RG * vp, *lk = lq + a.dim;
    tk_v4f S[RPT];
    const float* sin = a.state + ((size_t)(in < 0 ? 0 : in) * a.heads + h) * a.dim * vp + 4 * ct;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int e = rg + RG * i;
        S[i] = in >= 0 && live && e < a.dim ? *(const tk_v4f*)(sin + (size_t)e * vp) : tk_v4f{0.0f, 0.0f, 0.0f, 0.0f};
    }
    const int half = a.rot_dims / 2, qk = a.heads * a.dim;
    const float *qp = proj + (size_t)row * ld + a.col + h * a.dim, *kp = qp + qk, *vsrc = proj + (size_t)row * ld + a.col + 2 * qk + h * a.vdim;
    const float gate = tid < a.vdim ? vsrc[a.heads * a.vdim + tid] : 0.0f; /* vdim <= 256 <= THREADS: one column per thread */
    const float kscale = 1.0f / sqrtf((float)a.dim), decay = a.decay[(size_t)h * (TK_RETENTION_BLOCK + 1) + 1];
    for (int e = tid; e < a.dim; e += THREADS) {
        float q = qp[e], k = kp[e];
        if (e < 2 * half) {
            const int f = e < half ? e + half : e - half, j = e < half ? e : f;
            const float c = a.rope_cos[(size_t)pos * half + j], s = a.rope_sin[(size_t)pos * half + j] * (e < half ? -1.0f : 1.0f);
            q = q * c + qp[f] * s;
            k = k * c + kp[f] * s;
        }
        lq[e] = q;
        lk[e] = k * kscale;
    }
    if (tid < vp) lv[tid] = tid < a.vdim ? vsrc[tid] : 0.0f;
    __syncthreads();
    tk_v4f ao = {0.0f, 0.0f, 0.0f, 0.0f};
    if (live) {
        const tk_v4f v = *(const tk_v4f*)(lv + 4 * ct);
        float* so = a.state + ((size_t)out * a.heads + h) * a.dim * vp + 4 * ct;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const int e = rg + RG * i;
            if (e < a.dim) {
                S[i] = S[i] * decay + v * lk[e];
                *(tk_v4f*)(so + (size_t)e * vp) = S[i];
                ao += S[i] * lq[e];
            }
        }
        *(tk_v4f*)(po + rg * vp + 4 * ct) = ao;
    }
    __syncthreads();
    float o = 0.0f;
    if (tid < a.vdim)
        for (int i = 0; i < RG; ++i) o += po[i * vp + tid];
    const float ss = block_sum(o * o, red);
    if (tid < a.vdim)
        tk_img_put((T*)a.out_img, row, a.out_k0 + h * a.vdim + tid, a.out_ktiles, o * (a.out_scale / sqrtf(ss / (float)a.vdim + a.eps)) * tk_silu32(gate));
}

/* ------------------------------------------------------------------ mixture of experts ----- */

/* experts' tile counts (threads 0 .. 255, one expert each) -> first tiles and row blocks.  Every thread of the workgroup calls it. */
__device__ __forceinline__ void moe_plan(int experts, int block_tiles, int count, const TkMoeTab& t, int* st /* [512] LDS */) {
    const int e = threadIdx.x;
    const int tiles = e < experts ? (count + 15) / 16 : 0, nb = (tiles + block_tiles - 1) / block_tiles;
    int* sb = st + 256;
    if (e < 256) { st[e] = tiles; sb[e] = nb; }
    __syncthreads();
    for (int s = 1; s < 256; s <<= 1) { /* inclusive sums */
        const int a = e < 256 && e >= s ? st[e - s] : 0, b = e < 256 && e >= s ? sb[e - s] : 0;
        __syncthreads();
        if (e < 256) { st[e] += a; sb[e] += b; }
        __syncthreads();
    }
    if (e < experts) {
        const int tile0 = st[e] - tiles, b0 = sb[e] - nb;
        t.tile0[e] = tile0;
        for (int i = 0; i < nb; ++i) {
            const int left = tiles - i * block_tiles;
            t.blocks[b0 + i] = TkImgBlock{e, tile0 + i * block_tiles, left < block_tiles ? left : block_tiles, 0};
        }
    }
    if (e == 255) *t.n_blocks = sb[255];
}

/* one wave per row, 16 rows per workgroup; an expert's rows are counted in LDS first, one global addition per workgroup and expert.  A launch of
 * one workgroup goes on to the plan itself. */
__global__ __launch_bounds__(1024) void k_moe_select(const float* logits, int ld, int experts, int top, int groups, int keep, int nrows, int block_tiles, TkMoeTab t) {
    __shared__ float sc_[16][TK_MAX_EXPERTS], gs_[16][64];
    __shared__ uint8_t on_[16][64];
    __shared__ int cnt[TK_MAX_EXPERTS], base[TK_MAX_EXPERTS], st[512];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, row = blockIdx.x * 16 + wave, per = experts / groups;
    const bool live = row < nrows;
    float *sc = sc_[wave], *gs = gs_[wave];
    uint8_t* on = on_[wave];
    if (threadIdx.x < TK_MAX_EXPERTS) cnt[threadIdx.x] = 0;
    if (live)
        for (int e = lane; e < experts; e += 64) sc[e] = tk_sigmoid32(logits[(size_t)row * ld + e]);
    __syncthreads();
    if (live && lane < groups) { /* a group's score: the sum of its two best */
        float a = -INFINITY, b = -INFINITY;
        for (int e = lane * per; e < (lane + 1) * per; ++e) {
            const float v = sc[e];
            if (v > a) { b = a; a = v; } else if (v > b) b = v;
        }
        gs[lane] = per > 1 ? a + b : a;
    }
    __syncthreads();
    if (live && lane < groups) {
        int better = 0;
        for (int j = 0; j < groups; ++j) better += gs[j] > gs[lane] || (gs[j] == gs[lane] && j < lane);
        on[lane] = better < keep;
    }
    __syncthreads();
    int mine = 0, rank = 0; /* lane j keeps the row's j-th choice */
    if (live) {
        float c[TK_MAX_EXPERTS / 64]; /* this lane's candidates */
#pragma unroll
        for (int i = 0; i < TK_MAX_EXPERTS / 64; ++i) {
            const int e = lane + 64 * i;
            c[i] = e < experts && on[e / per] ? sc[e] : -INFINITY;
        }
        for (int j = 0; j < top; ++j) {
            float best = -INFINITY;
            int id = 0x7fffffff;
#pragma unroll
            for (int i = 0; i < TK_MAX_EXPERTS / 64; ++i)
                if (c[i] > best) { best = c[i]; id = lane + 64 * i; }
            for (int s = 32; s >= 1; s >>= 1) {
                const float ov = __shfl_xor(best, s, 64);
                const int oi = __shfl_xor(id, s, 64);
                if (ov > best || (ov == best && oi < id)) { best = ov; id = oi; }
            }
            if (id >= experts) id = 0; /* no finite score is left: a defined expert all the same */
#pragma unroll
            for (int i = 0; i < TK_MAX_EXPERTS / 64; ++i)
                if (lane + 64 * i == id) c[i] = -INFINITY;
            if (lane == j) mine = id;
        }
        if (lane < top) rank = atomicAdd(&cnt[mine], 1);
    }
    __syncthreads();
    if ((int)threadIdx.x < experts) {
        const int n = cnt[threadIdx.x];
        base[threadIdx.x] = gridDim.x > 1 && n > 0 ? atomicAdd(t.count + threadIdx.x, n) : 0;
    }
    __syncthreads();
    if (live && lane < top) {
        const int i = row * top + lane;
        t.expert[i] = mine;
        t.weight[i] = sc[mine];
        t.rank[i] = base[mine] + rank;
    }
    if (gridDim.x == 1) moe_plan(experts, block_tiles, (int)threadIdx.x < experts ? cnt[threadIdx.x] : 0, t, st);
}

/* the plan of a launch of several workgroups; the counts are cleared for the next layer */
__global__ __launch_bounds__(256) void k_moe_plan(int experts, int block_tiles, TkMoeTab t) {
    __shared__ int st[512];
    const int e = threadIdx.x, n = e < experts ? t.count[e] : 0;
    if (e < experts) t.count[e] = 0;
    moe_plan(experts, block_tiles, n, t, st);
}

/* 16-byte pieces of a row of the image to its places among the experts' rows */
__global__ __launch_bounds__(256) void k_moe_gather(const tk_v4u* img, tk_v4u* out, int ktiles, int top, TkMoeTab t) {
    const int i = blockIdx.x, row = i / top;
    const int slot = t.tile0[t.expert[i]] * 16 + t.rank[i];
    if (blockIdx.y == 0 && threadIdx.x == 0) t.slot[i] = slot;
    const int p = blockIdx.y * 256 + threadIdx.x; /* piece: k tile p / 4, lane group p % 4 */
    if (p >= ktiles * 4) return;
    out[((size_t)(slot >> 4) * ktiles + p / 4) * 64 + (slot & 15) + 16 * (p % 4)] = img[((size_t)(row >> 4) * ktiles + p / 4) * 64 + (row & 15) + 16 * (p % 4)];
}

} // namespace

/* ------------------------------------------------------------------ launchers -------------- */

#define TK_TYPED(type, ...) do { if ((type) == TK_IMG_F32) { typedef float T; __VA_ARGS__; } else { typedef TkBf16 T; __VA_ARGS__; } } while (0)

/* threads and register groups that hold a row */
static int norm_threads(int width) { return width > 2048 ? 512 : 256; }
#define TK_ROW(vec, width, ...) do { \
        if (vec) { constexpr bool VEC = true; if ((width) <= 8 * norm_threads(width)) { constexpr int NV = 1; __VA_ARGS__; } else { constexpr int NV = 4; __VA_ARGS__; } } \
        else { constexpr bool VEC = false; if ((width) <= 8 * norm_threads(width)) { constexpr int NV = 1; __VA_ARGS__; } else { constexpr int NV = 4; __VA_ARGS__; } } } while (0)

void tk_launch_layer_embed(int type, const uint16_t* table, int width, float scale, const int32_t* tok, int nrows, float* x, const TkNorm& next, float eps, void* img, int ktiles, hipStream_t s) {
    TK_TYPED(type, TK_ROW(width % 8 == 0, width, hipLaunchKernelGGL((k_layer_embed<T, VEC, NV>), dim3(nrows), dim3(norm_threads(width)), 0, s, table, width, scale, tok, x, next, eps, (T*)img, ktiles)));
}

void tk_launch_mixer_prep(int type, const float* proj, int ld, const TkAttnArgs* attn, const TkDeltaArgs* delta, const TkPassTab& t, int nrows, hipStream_t s) {
    const TkAttnArgs a = attn ? *attn : TkAttnArgs{};
    const TkDeltaArgs d = delta ? *delta : TkDeltaArgs{};
    const int na = attn ? a.heads + 2 * a.kv_heads : 0, nd = delta ? 2 * d.kv_heads + 2 * d.heads : 0;
    const int gx = (na + nd + 3) / 4;
    const bool even = a.dim % 2 == 0 && a.vdim % 2 == 0 && a.rot_dims % 4 == 0 && a.col % 2 == 0 && ld % 2 == 0;
#define TK_PREP(RW, CV, V) TK_TYPED(type, hipLaunchKernelGGL((k_mixer_prep<T, RW, CV, V>), dim3(gx, (nrows + RW - 1) / RW), dim3(256), 0, s, proj, ld, a, d, t, na, nd, nrows))
#define TK_PREP_V(RW, CV) do { if (even) TK_PREP(RW, CV, 2); else TK_PREP(RW, CV, 1); } while (0)
    if (nrows >= 512) { if (a.taps > 0) TK_PREP_V(4, true); else TK_PREP_V(4, false); }
    else { if (a.taps > 0) TK_PREP_V(1, true); else TK_PREP_V(1, false); }
#undef TK_PREP_V
#undef TK_PREP
}

static int attn_bucket(const TkAttnArgs& a) {
    const int m = a.kv.dim_pad > a.kv.vdim_pad ? a.kv.dim_pad : a.kv.vdim_pad;
    return m <= 64 ? 64 : m <= 128 ? 128 : 256;
}

static bool attn_full(const TkAttnArgs& a) { return a.kv.dim_pad == attn_bucket(a) && a.kv.vdim_pad == attn_bucket(a); }

void tk_launch_attn_tiles(int type, const TkAttnArgs& a, const TkPassTab& t, const int32_t* tiles, int n_tiles, hipStream_t s) {
    const int b = attn_bucket(a);
    const dim3 grid(n_tiles, a.heads);
    const size_t sz = type == TK_IMG_F32 ? 4 : 2, lds = (TK_PAGE * (a.kv.dim_pad * sz + 16) + a.kv.vdim_pad * (TK_PAGE * sz + 16)) * (type == TK_IMG_F32 && b == 256 ? 1 : 2);
#define TK_TILES(T, B, F) hipLaunchKernelGGL((k_attn_tiles<T, B, F>), grid, dim3(256), lds, s, a, t, tiles)
#define TK_TILES_B(T, F) do { if (b == 64) TK_TILES(T, 64, F); else if (b == 128) TK_TILES(T, 128, F); else TK_TILES(T, 256, F); } while (0)
    if (type == TK_IMG_F32) TK_TILES_B(float, false);
    else if (attn_full(a)) TK_TILES_B(TkBf16, true);
    else TK_TILES_B(TkBf16, false);
#undef TK_TILES_B
#undef TK_TILES
}

size_t tk_attn_rows_scratch_floats(const TkAttnArgs& a, int nrows, int splits) { return splits > 1 ? (size_t)nrows * a.heads * splits * (a.kv.vdim_pad + 2) : 0; }

static int attn_row_blocks(const TkAttnArgs& a) { return a.kv_heads * ((a.heads / a.kv_heads + 15) / 16); }
/* waves of a row's workgroup: eight where the pass has few workgroups (a latency chain of pages), four where it has many */
static int attn_row_waves(const TkAttnArgs& a, int nrows) { return nrows * attn_row_blocks(a) < 512 && attn_bucket(a) < 256 ? 8 : 4; }

int tk_attn_rows_splits(const TkAttnArgs& a, int pages, int nrows) {
    const int wgs = nrows * attn_row_blocks(a), want = (512 + wgs - 1) / wgs, most = pages / (2 * attn_row_waves(a, nrows));
    const int s = want < most ? want : most;
    return s < 1 ? 1 : s > 32 ? 32 : s;
}

void tk_launch_attn_rows(int type, const TkAttnArgs& a, const TkPassTab& t, int nrows, int splits, float* scratch, hipStream_t s) {
    const int b = attn_bucket(a);
    const bool eight = attn_row_waves(a, nrows) == 8;
    const dim3 grid(attn_row_blocks(a), nrows, splits);
#define TK_ROWS(T, B, W, F) hipLaunchKernelGGL((k_attn_rows<T, B, W, F>), grid, dim3(64 * W), (attn_row_lds<B, W>()), s, a, t, splits, scratch)
#define TK_ROWS_B(T, F) do { \
        if (b == 64) { if (eight) TK_ROWS(T, 64, 8, F); else TK_ROWS(T, 64, 4, F); } \
        else if (b == 128) { if (eight) TK_ROWS(T, 128, 8, F); else TK_ROWS(T, 128, 4, F); } \
        else TK_ROWS(T, 256, 4, F); } while (0)
    if (type == TK_IMG_F32) TK_ROWS_B(float, false);
    else if (attn_full(a)) TK_ROWS_B(TkBf16, true);
    else TK_ROWS_B(TkBf16, false);
#undef TK_ROWS_B
#undef TK_ROWS
    if (splits > 1) TK_TYPED(type, hipLaunchKernelGGL((k_attn_merge<T>), dim3(a.heads, nrows), dim3(64), 0, s, a, splits, scratch));
}

/* column threads of a delta row: the power of two that covers vdim in fours */
static int delta_ct_log2(const TkDeltaArgs& d) {
    int l = 0;
    while ((4 << l) < d.vdim) ++l;
    return l;
}

bool tk_launch_mixers_step(int type, const TkAttnArgs& a, const TkDeltaArgs& d, const TkPassTab& t, int nrows, hipStream_t s) {
    const int b = attn_bucket(a), ctl = delta_ct_log2(d), waves = attn_row_waves(a, nrows), threads = 64 * waves;
    const int rg = threads >> ctl, rpt = rg ? (d.dim + rg - 1) / rg : 1 << 20;
    if (type != TK_IMG_BF16 || b > 128 || rpt > (waves == 8 ? 8 : 16) || d.vdim > threads) return false;
    const dim3 grid(attn_row_blocks(a) + d.heads, nrows);
    const size_t dl = delta_row_lds(d, threads, ctl);
#define TK_STEP(B, W, R) do { const size_t al = attn_row_lds<B, W>(); \
        if (attn_full(a)) hipLaunchKernelGGL((k_mixers_step<TkBf16, B, W, R, true>), grid, dim3(threads), al > dl ? al : dl, s, a, d, t, attn_row_blocks(a), ctl); \
        else hipLaunchKernelGGL((k_mixers_step<TkBf16, B, W, R, false>), grid, dim3(threads), al > dl ? al : dl, s, a, d, t, attn_row_blocks(a), ctl); } while (0)
    if (b == 64) { if (waves == 8) TK_STEP(64, 8, 8); else TK_STEP(64, 4, 16); }
    else { if (waves == 8) TK_STEP(128, 8, 8); else TK_STEP(128, 4, 16); }
#undef TK_STEP
    return true;
}

void tk_launch_delta_scan(int type, const TkDeltaArgs& d, const TkPassTab& t, int n_segments, int nrows, hipStream_t s) {
    const bool many = (int64_t)((d.vdim + 15) / 16) * d.heads * n_segments >= 512;
    const dim3 grid(many ? (d.vdim + 15) / 16 : (d.vdim + 7) / 8, d.heads, n_segments);
#define TK_SCAN(RPL) do { if (many) hipLaunchKernelGGL((k_delta_scan<16, 2 * RPL>), grid, dim3(256), 0, s, d, t); else hipLaunchKernelGGL((k_delta_scan<32, RPL>), grid, dim3(256), 0, s, d, t); } while (0)
    if (d.dim <= 32) TK_SCAN(1);
    else if (d.dim <= 64) TK_SCAN(2);
    else if (d.dim <= 128) TK_SCAN(4);
    else TK_SCAN(8);
#undef TK_SCAN
    TK_TYPED(type, hipLaunchKernelGGL((k_delta_out<T>), dim3((d.heads + 3) / 4, nrows), dim3(256), 0, s, d));
}

void tk_launch_delta_step(int type, const TkDeltaArgs& d, const TkPassTab& t, int nrows, hipStream_t s) {
    const int ctl = delta_ct_log2(d);
    const dim3 grid(d.heads, nrows);
    auto rpt = [&](int threads) { const int rg = threads >> ctl; return (d.dim + rg - 1) / rg; };
    TK_TYPED(type, {
        if (rpt(256) <= 4) hipLaunchKernelGGL((k_delta_step<T, 256, 4>), grid, dim3(256), delta_row_lds(d, 256, ctl), s, d, t, ctl);
        else if (rpt(256) <= 8) hipLaunchKernelGGL((k_delta_step<T, 256, 8>), grid, dim3(256), delta_row_lds(d, 256, ctl), s, d, t, ctl);
        else if (rpt(256) <= 16) hipLaunchKernelGGL((k_delta_step<T, 256, 16>), grid, dim3(256), delta_row_lds(d, 256, ctl), s, d, t, ctl);
        else if (rpt(256) <= 32) hipLaunchKernelGGL((k_delta_step<T, 256, 32>), grid, dim3(256), delta_row_lds(d, 256, ctl), s, d, t, ctl);
        else hipLaunchKernelGGL((k_delta_step<T, 1024, 16>), grid, dim3(1024), delta_row_lds(d, 1024, ctl), s, d, t, ctl);
    });
}

void tk_launch_post_norm(int type, const TkSubOut& o, const TkNorm& norm, const TkNorm& next, float eps, int width, int nrows, float* x, void* img, int ktiles, hipStream_t s) {
    TK_TYPED(type, TK_ROW(width % 8 == 0 && o.ld % 4 == 0, width, hipLaunchKernelGGL((k_post_norm<T, VEC, NV>), dim3(nrows), dim3(norm_threads(width)), 0, s, o, norm, next, eps, width, x, (T*)img, ktiles)));
}

void tk_launch_rows_norm(int type, const float* x, const int32_t* rows, int n, const TkNorm& norm, float eps, int width, void* img, int ktiles, hipStream_t s) {
    TK_TYPED(type, TK_ROW(width % 8 == 0, width, hipLaunchKernelGGL((k_rows_norm<T, VEC, NV>), dim3(n), dim3(norm_threads(width)), 0, s, x, rows, norm, eps, width, (T*)img, ktiles)));
}

/* the forms of the scan: key dimensions 64, 128, 256 x value columns 64, 128, 256 */
#define TK_RET_FORMS(X, T) X(T, 64, 4, 1) X(T, 64, 8, 1) X(T, 64, 8, 2) X(T, 128, 4, 1) X(T, 128, 8, 1) X(T, 128, 8, 2) X(T, 256, 4, 1) X(T, 256, 8, 1) X(T, 256, 8, 2)

void tk_launch_retention_scan(int type, const TkRetentionArgs& a, const float* proj, int ld, const TkPassTab& t, const TkRetentionBlock* blocks, int n_blocks, int n_sums, hipStream_t s) {
    const int dim = a.dim <= 64 ? 64 : a.dim <= 128 ? 128 : 256, vb = a.vdim <= 64 ? 64 : a.vdim <= 128 ? 128 : 256;
    const dim3 grid(a.heads, n_blocks);
#define TK_RET(T, D, W, N) \
    if (dim == D && vb == 16 * W * N) { \
        constexpr size_t lds = RetLds<T, D, 16 * W * N>::bytes; \
        if (n_sums) { \
            hipLaunchKernelGGL((k_retention_scan<T, D, W, N, true>), grid, dim3(64 * W), lds, s, a, proj, ld, t, blocks); \
            hipLaunchKernelGGL(k_retention_prefix, dim3((a.dim * ((a.vdim + 3) / 4) + 255) / 256, a.heads, n_blocks), dim3(256), 0, s, a, t, blocks); \
        } \
        hipLaunchKernelGGL((k_retention_scan<T, D, W, N, false>), grid, dim3(64 * W), lds, s, a, proj, ld, t, blocks); \
    }
    if (type == TK_IMG_F32) { TK_RET_FORMS(TK_RET, float) } else { TK_RET_FORMS(TK_RET, TkBf16) }
#undef TK_RET
}

void tk_launch_retention_step(int type, const TkRetentionArgs& a, const float* proj, int ld, const TkPassTab& t, int n_segments, hipStream_t s) {
    int ctl = 0;
    while ((4 << ctl) < a.vdim) ++ctl;
    const dim3 grid(a.heads, n_segments);
    const size_t vp = (a.vdim + 3) & ~3;
    auto lds = [&](int threads) { return (16 + vp + (size_t)(threads >> ctl) * vp + 2 * (size_t)a.dim) * sizeof(float); };
    auto rpt = [&](int threads) { const int rg = threads >> ctl; return (a.dim + rg - 1) / rg; };
    TK_TYPED(type, {
        if (rpt(256) <= 4) hipLaunchKernelGGL((k_retention_step<T, 256, 4>), grid, dim3(256), lds(256), s, a, proj, ld, t, ctl);
        else if (rpt(256) <= 8) hipLaunchKernelGGL((k_retention_step<T, 256, 8>), grid, dim3(256), lds(256), s, a, proj, ld, t, ctl);
        else if (rpt(256) <= 16) hipLaunchKernelGGL((k_retention_step<T, 256, 16>), grid, dim3(256), lds(256), s, a, proj, ld, t, ctl);
        else if (rpt(256) <= 32) hipLaunchKernelGGL((k_retention_step<T, 256, 32>), grid, dim3(256), lds(256), s, a, proj, ld, t, ctl);
        else hipLaunchKernelGGL((k_retention_step<T, 1024, 16>), grid, dim3(1024), lds(1024), s, a, proj, ld, t, ctl);
    });
}

void tk_launch_moe_select(const float* logits, int ld, int experts, int top, int groups, int keep, int nrows, int block_tiles, const TkMoeTab& t, hipStream_t s) {
    const int wgs = (nrows + 15) / 16;
    hipLaunchKernelGGL(k_moe_select, dim3(wgs), dim3(1024), 0, s, logits, ld, experts, top, groups, keep, nrows, block_tiles, t);
    if (wgs > 1) hipLaunchKernelGGL(k_moe_plan, dim3(1), dim3(256), 0, s, experts, block_tiles, t);
}
void tk_launch_moe_gather(const void* img, void* gathered, int ktiles, int top, int nrows, const TkMoeTab& t, hipStream_t s) {
    hipLaunchKernelGGL(k_moe_gather, dim3(nrows * top, (ktiles * 4 + 255) / 256), dim3(256), 0, s, (const tk_v4u*)img, (tk_v4u*)gathered, ktiles, top, t);
}
void tk_launch_swap_state(const TkPassTab& t, int n, hipStream_t s) { hipLaunchKernelGGL(k_swap_state, dim3((n + 255) / 256), dim3(256), 0, s, t, n); }

const char* tk_mixer_prepare_device() {
    static std::atomic<bool> done[64];
    static std::mutex mu;
    int dev = 0;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return "no current device";
    if (done[dev].load(std::memory_order_acquire)) return nullptr;
    std::lock_guard<std::mutex> lk(mu);
    hipError_t e = hipSuccess;
    auto opt = [&](const void* f) { if (e == hipSuccess) e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); };
    opt((const void*)k_attn_tiles<float, 64, false>); opt((const void*)k_attn_tiles<float, 128, false>); opt((const void*)k_attn_tiles<float, 256, false>);
    opt((const void*)k_attn_tiles<TkBf16, 64, false>); opt((const void*)k_attn_tiles<TkBf16, 128, false>); opt((const void*)k_attn_tiles<TkBf16, 256, false>);
    opt((const void*)k_attn_tiles<TkBf16, 64, true>); opt((const void*)k_attn_tiles<TkBf16, 128, true>); opt((const void*)k_attn_tiles<TkBf16, 256, true>);
#define TK_RET_OPT(T, D, W, N) opt((const void*)k_retention_scan<T, D, W, N, true>); opt((const void*)k_retention_scan<T, D, W, N, false>);
    TK_RET_FORMS(TK_RET_OPT, float) TK_RET_FORMS(TK_RET_OPT, TkBf16)
#undef TK_RET_OPT
    if (e != hipSuccess) return hipGetErrorString(e);
    done[dev].store(true, std::memory_order_release);
    return nullptr;
}
