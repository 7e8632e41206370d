/* tk_layered_model.hip — weights of the layer-list decoders (tk_layered.h) */
#include <math.h>
#include <stdio.h>
#include <string.h>

#include "../nn/tk_image_device.h"
#include "tk_layered.h"
#include "tk_safetensors.h"

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

namespace {
/* bf16 values uniform in [-a, a] by a counter hash */
__global__ void k_random_bf16(uint64_t seed, int64_t n, float a, uint16_t* out) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    uint64_t z = seed + 0x9E3779B97F4A7C15ull * (uint64_t)(i + 1);
    z = (z ^ (z >> 30)) * 0xBF58476D1CE4E5B9ull;
    z = (z ^ (z >> 27)) * 0x94D049BB133111EBull;
    z ^= z >> 31;
    out[i] = tk_bf16_bits(a * ((float)(z >> 40) * (2.0f / 16777216.0f) - 1.0f));
}
} // namespace

/* where tensors come from: matrices as row-major device data, vectors as host floats */
struct TkLayeredModel::Source {
    TkLayeredModel* m;
    TkSafetensorsFile* file = nullptr; /* null: synthetic */
    uint64_t seed = 0, count = 0;
    int rank = 0;
    void* dev = nullptr;
    size_t dev_bytes = 0;
    ~Source() { if (dev) (void)hipFree(dev); }
    bool room(size_t b) {
        if (b <= dev_bytes) return true;
        if (dev) { (void)hipDeviceSynchronize(); (void)hipFree(dev); }
        dev = nullptr; dev_bytes = 0;
        if (hipMalloc(&dev, b) != hipSuccess) { m->error = "out of device memory (weight staging)"; return false; }
        dev_bytes = b;
        return true;
    }
    const TkSafeTensor* check(const std::string& name, std::vector<int64_t> shape) {
        const TkSafeTensor* t = file->find(name);
        if (!t) { m->error = "tensor missing: " + name; return nullptr; }
        if (t->shape != shape) { m->error = "tensor " + name + " does not have the shape that config.json implies"; return nullptr; }
        if (t->dtype != "BF16" && t->dtype != "F32") { m->error = "tensor " + name + " has type " + t->dtype + " (want BF16 or F32)"; return nullptr; }
        return t;
    }
    /* rows of a matrix whose height only the file gives */
    int rows_of(const std::string& name) {
        if (!file) return rank;
        const TkSafeTensor* t = file->find(name);
        if (!t || t->shape.size() != 2 || t->shape[0] < 1 || t->shape[0] > 1 << 20) { m->error = "tensor missing or not a matrix: " + name; return 0; }
        return (int)t->shape[0];
    }
    /* [rows][cols] into dst at (n0, k0) */
    bool put(const std::string& name, int rows, int cols, void* img, int K, int n0, int k0, int interleave = -1) {
        const int kt = tk_img_kt(m->type);
        if (!file) {
            if (!room((size_t)rows * cols * 2)) return false;
            const int64_t n = (int64_t)rows * cols;
            hipLaunchKernelGGL(k_random_bf16, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, nullptr, seed + 0x1000003ull * ++count, n, sqrtf(3.0f / (float)cols), (uint16_t*)dev);
            tk_launch_put_image(m->type, dev, 0, rows, cols, img, K / kt, n0, k0, interleave, nullptr);
        } else {
            const TkSafeTensor* t = check(name, {rows, cols});
            if (!t || !room(t->nbytes)) return false;
            if (hipMemcpy(dev, t->data, t->nbytes, hipMemcpyHostToDevice) != hipSuccess) { m->error = "upload of " + name + " failed"; return false; }
            tk_launch_put_image(m->type, dev, t->dtype == "F32", rows, cols, img, K / kt, n0, k0, interleave, nullptr);
        }
        if (hipGetLastError() != hipSuccess || hipStreamSynchronize(nullptr) != hipSuccess) { m->error = "tiling of " + name + " failed"; return false; }
        return true;
    }
    /* any tensor as floats; synthetic: uniform in [lo, hi] */
    bool values(const std::string& name, std::vector<int64_t> shape, std::vector<float>* out, float lo, float hi) {
        size_t n = 1;
        for (int64_t d : shape) n *= (size_t)d;
        const size_t at = out->size();
        out->resize(at + n);
        if (!file) {
            uint64_t z = seed + 0x1000003ull * ++count;
            for (size_t i = 0; i < n; ++i) {
                z = z * 6364136223846793005ull + 1442695040888963407ull;
                (*out)[at + i] = lo + (hi - lo) * (float)(z >> 40) / 16777216.0f;
            }
            return true;
        }
        const TkSafeTensor* t = check(name, shape);
        if (!t) return false;
        for (size_t i = 0; i < n; ++i) {
            if (t->dtype == "F32") memcpy(&(*out)[at + i], t->data + 4 * i, 4);
            else {
                const uint32_t b = ((uint32_t)t->data[2 * i] | (uint32_t)t->data[2 * i + 1] << 8) << 16;
                memcpy(&(*out)[at + i], &b, 4);
            }
        }
        return true;
    }
    bool upload(const std::vector<float>& v, float** dst) {
        if (!m->alloc((void**)dst, v.size() * 4)) return false;
        if (hipMemcpy(*dst, v.data(), v.size() * 4, hipMemcpyHostToDevice) != hipSuccess) { m->error = "upload failed"; return false; }
        return true;
    }
    bool vec(const std::string& name, std::vector<int64_t> shape, float** dst, float lo, float hi) {
        std::vector<float> v;
        return values(name, shape, &v, lo, hi) && upload(v, dst);
    }
    bool norm(const std::string& name, TkNorm* n) {
        if (name.empty()) return true;
        n->layer = m->cfg.norm == TkLayeredConfig::LAYER;
        return vec(name, {m->cfg.width}, (float**)&n->w, 0.8f, 1.2f) && (!n->layer || vec(name + ".b", {m->cfg.width}, (float**)&n->b, -0.1f, 0.1f));
    }
};

TkLayeredModel::~TkLayeredModel() {
    (void)hipSetDevice(device);
    for (void* p : owned_) (void)hipFree(p);
}

bool TkLayeredModel::alloc(void** p, size_t bytes) {
    HIPQ(hipMalloc(p, bytes ? bytes : 16));
    owned_.push_back(*p);
    return true;
}

/* zeroed: the padding of an image is never written again */
bool TkLayeredModel::mat(TkMat* t, int rows, int cols, int copies) {
    t->rows = rows; t->cols = cols;
    t->N = (rows + 15) / 16 * 16;
    t->K = tk_img_pad_k(type, cols);
    t->bytes = tk_img_bytes(type, t->N, cols);
    if (!alloc(&t->img, t->bytes * copies)) return false;
    HIPQ(hipMemset(t->img, 0, t->bytes * copies));
    matrix_bytes_ += t->bytes * copies;
    return true;
}

bool TkLayeredModel::begin(const std::string& text, const std::string& dtype, int dev) {
    device = dev;
    if (dtype == "bfloat16") type = TK_IMG_BF16;
    else if (dtype == "float32") type = TK_IMG_F32;
    else { error = "unknown dtype '" + dtype + "' (want bfloat16 or float32)"; return false; }
    if (!tk_layered_parse(text, &cfg, &error)) return false;
    if (cfg.width > 16384) { error = "width above 16384 is not supported"; return false; }
    HIPQ(hipSetDevice(device));
    return true;
}

bool TkLayeredModel::build(Source& src) {
    const int D = cfg.width;
    /* the embedding stays a table of bf16 rows */
    if (!alloc((void**)&embed, (size_t)cfg.vocab * D * 2)) return false;
    {
        std::vector<float> e;
        if (!src.values("embed", {cfg.vocab, D}, &e, -1.7f, 1.7f)) return false;
        std::vector<uint16_t> b(e.size());
        for (size_t i = 0; i < e.size(); ++i) {
            uint32_t u;
            memcpy(&u, &e[i], 4);
            b[i] = (uint16_t)((u + 0x7FFF + ((u >> 16) & 1)) >> 16); /* exact for bf16 files */
        }
        HIPQ(hipMemcpy(embed, b.data(), b.size() * 2, hipMemcpyHostToDevice));
    }
    layers.resize(cfg.layers.size());
    for (size_t i = 0; i < layers.size(); ++i) {
        const TkLayerSpec& s = cfg.layers[i];
        TkLayeredLayer& L = layers[i];
        if (s.weights_of >= 0) continue;
        const uint64_t before = matrix_bytes_;
        L.branches.resize(s.branches.size());
        /* columns: every branch's own projections, then the inner sides of the low-rank gates */
        int col = 0, out_k = 0, low_k = 0, low_n = 0;
        for (size_t b = 0; b < s.branches.size(); ++b) {
            const TkBranchSpec& bs = s.branches[b];
            TkLayeredBranch& B = L.branches[b];
            B.col = col; B.out_k0 = out_k;
            if (bs.kind == TkBranchSpec::ATTENTION) {
                const TkAttnSpec& a = bs.attn;
                col += a.heads * a.dim + a.kv_heads * (a.dim + a.vdim);
                out_k += a.heads * a.vdim;
            } else if (bs.kind == TkBranchSpec::RETENTION) {
                const TkRetentionSpec& t = bs.retention;
                col += 2 * t.heads * (t.dim + t.vdim);
                out_k += t.heads * t.vdim;
            } else {
                const TkDeltaSpec& d = bs.delta;
                if (!(B.rank_a = src.rows_of(bs.prefix + "a1")) || !(B.rank_g = src.rows_of(bs.prefix + "g1"))) return false;
                col += 2 * d.kv_heads * d.dim + d.heads * d.vdim + d.heads;
                out_k += d.heads * d.vdim;
                B.low_a = low_n; low_n += d.heads * d.dim;
                B.low_g = low_n; low_n += d.heads * d.vdim;
                low_k += B.rank_a + B.rank_g;
            }
        }
        L.low_col = col; L.low_cols = low_k;
        if (!mat(&L.in, col + low_k, D) || !mat(&L.out, D, out_k) || (low_k && !mat(&L.low, low_n, low_k))) return false;
        std::vector<float> out_bias;
        int lk = 0;
        for (size_t b = 0; b < s.branches.size(); ++b) {
            const TkBranchSpec& bs = s.branches[b];
            TkLayeredBranch& B = L.branches[b];
            const std::string& p = bs.prefix;
            if (bs.kind == TkBranchSpec::ATTENTION) {
                const TkAttnSpec& a = bs.attn;
                const int nq = a.heads * a.dim, nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim, no = a.heads * a.vdim;
                if (!src.put(p + "q", nq, D, L.in.img, L.in.K, B.col, 0) || !src.put(p + "k", nk, D, L.in.img, L.in.K, B.col + nq, 0) ||
                    !src.put(p + "v", nv, D, L.in.img, L.in.K, B.col + nq + nk, 0) || !src.put(p + "o", D, no, L.out.img, L.out.K, 0, B.out_k0))
                    return false;
                if (a.bias) {
                    std::vector<float> v, o;
                    if (!src.values(p + "q.b", {nq}, &v, -0.1f, 0.1f) || !src.values(p + "k.b", {nk}, &v, -0.1f, 0.1f) || !src.values(p + "v.b", {nv}, &v, -0.1f, 0.1f) ||
                        !src.upload(v, &B.bias) || !src.values(p + "o.b", {D}, &o, -0.1f, 0.1f))
                        return false;
                    out_bias.resize((size_t)D, 0.0f);
                    for (int k = 0; k < D; ++k) out_bias[(size_t)k] += bs.scale * o[(size_t)k];
                }
                if (a.taps > 0) {
                    std::vector<float> conv;
                    if (!src.values(p + "q.conv", {nq, a.taps}, &conv, -0.9f, 0.9f) || !src.values(p + "k.conv", {nk, a.taps}, &conv, -0.9f, 0.9f) ||
                        !src.values(p + "v.conv", {nv, a.taps}, &conv, -0.9f, 0.9f) || !src.upload(conv, &B.conv))
                        return false;
                }
                if (a.qk_norm && (!src.vec(p + "q.norm", {a.dim}, &B.q_norm, 0.8f, 1.2f) || !src.vec(p + "k.norm", {a.dim}, &B.k_norm, 0.8f, 1.2f))) return false;
            } else if (bs.kind == TkBranchSpec::RETENTION) {
                const TkRetentionSpec& t = bs.retention;
                const int nk = t.heads * t.dim, nv = t.heads * t.vdim, c0 = B.col;
                if (!src.put(p + "q", nk, D, L.in.img, L.in.K, c0, 0) || !src.put(p + "k", nk, D, L.in.img, L.in.K, c0 + nk, 0) ||
                    !src.put(p + "v", nv, D, L.in.img, L.in.K, c0 + 2 * nk, 0) || !src.put(p + "g", nv, D, L.in.img, L.in.K, c0 + 2 * nk + nv, 0) ||
                    !src.put(p + "o", D, nv, L.out.img, L.out.K, 0, B.out_k0))
                    return false;
            } else {
                const TkDeltaSpec& d = bs.delta;
                const int nk = d.kv_heads * d.dim, nv = d.heads * d.vdim, c0 = B.col;
                if (!src.put(p + "q", nk, D, L.in.img, L.in.K, c0, 0) || !src.put(p + "k", nk, D, L.in.img, L.in.K, c0 + nk, 0) ||
                    !src.put(p + "v", nv, D, L.in.img, L.in.K, c0 + 2 * nk, 0) || !src.put(p + "b", d.heads, D, L.in.img, L.in.K, c0 + 2 * nk + nv, 0) ||
                    !src.put(p + "a1", B.rank_a, D, L.in.img, L.in.K, L.low_col + lk, 0) || !src.put(p + "g1", B.rank_g, D, L.in.img, L.in.K, L.low_col + lk + B.rank_a, 0) ||
                    !src.put(p + "a2", d.heads * d.dim, B.rank_a, L.low.img, L.low.K, B.low_a, lk) ||
                    !src.put(p + "g2", nv, B.rank_g, L.low.img, L.low.K, B.low_g, lk + B.rank_a) || !src.put(p + "o", D, nv, L.out.img, L.out.K, 0, B.out_k0))
                    return false;
                lk += B.rank_a + B.rank_g;
                std::vector<float> conv;
                if (!src.values(p + "q.conv", {nk, d.taps}, &conv, -0.9f, 0.9f) || !src.values(p + "k.conv", {nk, d.taps}, &conv, -0.9f, 0.9f) ||
                    !src.values(p + "v.conv", {nv, d.taps}, &conv, -0.9f, 0.9f) || !src.upload(conv, &B.conv) || !src.vec(p + "A_log", {d.heads}, &B.a_log, 0.0f, 2.7f) ||
                    !src.vec(p + "dt_bias", {d.heads * d.dim}, &B.dt_bias, -6.0f, -2.0f) || !src.vec(p + "norm", {d.vdim}, &B.norm, 0.8f, 1.2f))
                    return false;
            }
        }
        if (!out_bias.empty() && !src.upload(out_bias, &L.out_bias)) return false;
        if (!src.norm(s.pre1, &L.pre1) || !src.norm(s.norm1, &L.norm1)) return false;
        const TkMlpSpec& f = s.mlp;
        L.bytes = matrix_bytes_ - before;
        if (f.kind == TkMlpSpec::NONE) continue;
        if (!src.norm(s.pre2, &L.pre2) || !src.norm(s.norm2, &L.norm2)) return false;
        const int E = f.kind == TkMlpSpec::MOE ? f.experts : 1, ffp = (f.ff + 15) / 16 * 16;
        if (!mat(&L.gate_up, 2 * ffp, D, E) || !mat(&L.down, D, f.ff, E)) return false;
        for (int e = 0; e < E; ++e) {
            const std::string p = f.prefix + (f.kind == TkMlpSpec::MOE ? "e" + std::to_string(e) + "." : "");
            uint8_t *gu = (uint8_t*)L.gate_up.img + e * L.gate_up.bytes, *dn = (uint8_t*)L.down.img + e * L.down.bytes;
            if (!src.put(p + "gate", f.ff, D, gu, L.gate_up.K, 0, 0, 0) || !src.put(p + "up", f.ff, D, gu, L.gate_up.K, 0, 0, 1) || !src.put(p + "down", D, f.ff, dn, L.down.K, 0, 0))
                return false;
        }
        if (f.kind == TkMlpSpec::MOE && (!mat(&L.router, f.experts, D) || !src.put(f.prefix + "router", f.experts, D, L.router.img, L.router.K, 0, 0))) return false;
        L.bytes = matrix_bytes_ - before;
    }
    for (size_t i = 0; i < layers.size(); ++i)
        if (cfg.layers[i].weights_of >= 0) {
            layers[i] = layers[(size_t)cfg.layers[i].weights_of]; /* the model owns the memory, layers only point to it */
            matrix_bytes_ += layers[i].bytes;                     /* streamed once more */
        }
    return src.norm("final.norm", &final_norm) && mat(&head, cfg.vocab, D) && src.put("head", cfg.vocab, D, head.img, head.K, 0, 0);
}

bool TkLayeredModel::load(const std::string& dir, const std::string& dtype, int dev) {
    const std::string path = dir + "/config.json";
    FILE* f = fopen(path.c_str(), "rb");
    if (!f) { error = "cannot open " + path; return false; }
    std::string text;
    char buf[65536];
    for (size_t n; (n = fread(buf, 1, sizeof buf, f)) > 0;) text.append(buf, n);
    fclose(f);
    if (!begin(text, dtype, dev)) return false;
    TkSafetensorsFile w;
    if (!w.open(dir + "/model.safetensors")) { error = w.error; return false; }
    Source src{this, &w};
    return build(src);
}

bool TkLayeredModel::fill_synthetic(const std::string& config_json, const std::string& dtype, int dev, uint64_t seed, int rank) {
    if (rank < 1 || rank > 1 << 16) { error = "rank of the low-rank gates is out of range"; return false; }
    if (!begin(config_json, dtype, dev)) return false;
    Source src{this, nullptr, seed};
    src.rank = rank;
    return build(src);
}

std::unique_ptr<TkDecodeSession> TkLayeredModel::open_session(int max_seq, int max_ctx, int pool_tokens, std::string* err) {
    std::unique_ptr<TkLayeredSession> s(new TkLayeredSession());
    if (!s->init(this, max_seq, max_ctx, pool_tokens)) { *err = s->error; return nullptr; }
    return s;
}
