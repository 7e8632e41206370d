/* tk_layered_session.hip — passes, paged cache and recurrent state of the layer-list decoders (tk_layered.h) */
#include <math.h>
#include <stdio.h>
#include <string.h>

#include <algorithm>

#include "tk_layered.h"
#include "tk_llm_kernels.h"

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

static constexpr int PASS_ROWS = 2048; /* rows of one pass at most */

/* floats between two rows of the projections: an odd number of 256-byte lines, so that a head's columns of many rows spread over the memory channels */
static int proj_pitch(int n) { return ((n + 63) / 64 | 1) * 64; }

bool TkLayeredSession::alloc(void** p, size_t bytes, bool zero) {
    HIPQ(hipMalloc(p, bytes ? bytes : 16));
    owned_.push_back(*p);
    if (zero) HIPQ(hipMemset(*p, 0, bytes ? bytes : 16));
    return true;
}

/* cosines and sines of the positions, double precision on the host; one table per (dims, base) */
bool TkLayeredSession::rotation(int dims, double base, Rope* out) {
    if (dims <= 0) return true;
    Rope& r = rope_[{dims, base}];
    if (!r.c) {
        const int half = dims / 2;
        std::vector<float> cs((size_t)max_ctx * half), sn(cs.size());
        for (int t = 0; t < max_ctx; ++t)
            for (int i = 0; i < half; ++i) {
                const double ang = (double)t * pow(base, -2.0 * i / (double)dims);
                cs[(size_t)t * half + i] = (float)cos(ang);
                sn[(size_t)t * half + i] = (float)sin(ang);
            }
        if (!alloc((void**)&r.c, cs.size() * 4) || !alloc((void**)&r.s, sn.size() * 4)) return false;
        HIPQ(hipMemcpy(r.c, cs.data(), cs.size() * 4, hipMemcpyHostToDevice));
        HIPQ(hipMemcpy(r.s, sn.data(), sn.size() * 4, hipMemcpyHostToDevice));
    }
    *out = r;
    return true;
}

/* rows of a retention scan's blocks: a workgroup (a head's block) for every compute unit */
int TkLayeredSession::retention_rows(int nrows) const {
    int n = TK_RETENTION_BLOCK;
    while ((int64_t)(nrows / n) * ret_heads_ > 256) n *= 2;
    return n;
}

bool TkLayeredSession::init(TkLayeredModel* m, int mseq, int mctx, int pool_tokens) {
    m_ = m;
    max_seq = mseq;
    max_ctx = mctx;
    if (mseq < 1 || mseq > TK_MAX_ROWS || mctx < 1) { error = "max_seq must be in [1, 256] and max_ctx positive"; return false; }
    const TkLayeredConfig& c = m->cfg;
    const int type = m->type;
    const size_t esz = type == TK_IMG_F32 ? 4 : 2;
    max_pages_ = (mctx + TK_PAGE - 1) / TK_PAGE;
    n_pages_ = pool_tokens > 0 ? (pool_tokens + TK_PAGE - 1) / TK_PAGE : mseq * max_pages_;
    const int64_t want = ((int64_t)mseq * mctx + 63) / 64 * 64;
    const int R = (int)std::max<int64_t>(TK_MAX_ROWS, std::min<int64_t>(PASS_ROWS, want));
    const int max_tiles = R / 64 + mseq;
    /* tables behind the base's rows: segment of a row, segments, wanted rows, attention tiles, retention blocks */
    int32_t* ext = nullptr;
    const size_t block_ints = sizeof(TkRetentionBlock) / 4, extra = (size_t)R + 4 * (size_t)mseq + R + (2 + block_ints) * (size_t)max_tiles;
    if (!init_tables(m->device, c.vocab, R, extra, &ext)) return false;
    tab_ints_ = 3 * (size_t)R + extra;
    d_tab_ = d_seq;
    int32_t* p = ext;
    tab_.seq = d_seq; tab_.pos = d_pos; tab_.tok = d_tok;
    tab_.seg = p; p += R;
    tab_.seg_row0 = p; p += mseq;
    tab_.seg_n = p; p += mseq;
    tab_.seg_in = p; p += mseq;
    tab_.seg_out = p; p += mseq;
    d_out_rows_ = p; p += R;
    d_tiles_ = p; p += 2 * (size_t)max_tiles;
    d_blocks_ = p;
    HIPQ(hipHostMalloc((void**)&h_tab_, tab_ints_ * 4, hipHostMallocDefault));
    memset(h_tab_, 0, tab_ints_ * 4);
    if (!alloc((void**)&d_pages_, (size_t)mseq * max_pages_ * 4, true) || !alloc((void**)&d_otok_, TK_MAX_ROWS * 4, true)) return false;
    tab_.page_of = d_pages_;
    tab_.max_pages = max_pages_;
    seqs_.resize((size_t)mseq);
    h_pages_.assign((size_t)mseq * max_pages_, 0);
    for (int i = n_pages_ - 1; i >= 0; --i) free_pages_.push_back(i);

    size_t proj = 16, low = 16, mix = 0, lowk = 0, q = 0, dq = 0, dv = 0, dg = 0, dh = 0, ff = 0, scratch = 0, E = 0, gather = 0, moe_ff = 0, assign = 0, moe_rows = 0, sums = 0;
    for (const TkLayerSpec& s : c.layers)
        for (const TkBranchSpec& b : s.branches)
            if (b.kind == TkBranchSpec::RETENTION) ret_heads_ = std::max(ret_heads_, b.retention.heads);
    int ret_slots = 0;
    for (int n = 1; ret_heads_ && n <= R; ++n) ret_slots = std::max(ret_slots, n / retention_rows(n));
    st_.resize(c.layers.size());
    for (size_t l = 0; l < c.layers.size(); ++l) {
        const TkLayeredLayer& L = m->layers[l];
        const TkLayerSpec& s = c.layers[l];
        proj = std::max(proj, (size_t)proj_pitch(L.in.N));
        low = std::max(low, (size_t)L.low.N);
        mix = std::max(mix, tk_img_bytes(type, R, L.out.cols));
        if (L.low_cols) lowk = std::max(lowk, tk_img_bytes(type, R, L.low_cols));
        st_[l].resize(s.branches.size());
        for (size_t b = 0; b < s.branches.size(); ++b) {
            BranchState& bs = st_[l][b];
            if (s.branches[b].kind == TkBranchSpec::ATTENTION) {
                const TkAttnSpec& a = s.branches[b].attn;
                bs.kv.dim_pad = (a.dim + tk_img_kt(type) - 1) / tk_img_kt(type) * tk_img_kt(type);
                bs.kv.vdim_pad = (a.vdim + 15) / 16 * 16;
                if (!alloc(&bs.kv.k, (size_t)n_pages_ * a.kv_heads * TK_PAGE * bs.kv.dim_pad * esz, true) || !alloc(&bs.kv.v, (size_t)n_pages_ * a.kv_heads * TK_PAGE * bs.kv.vdim_pad * esz, true))
                    return false;
                q = std::max(q, (size_t)a.heads * bs.kv.dim_pad);
                int64_t seen = a.window > 0 ? (int64_t)a.window / TK_PAGE + 2 + (a.keep_first + TK_PAGE - 1) / TK_PAGE : max_pages_;
                if (a.chunk > 0) seen = std::min<int64_t>(seen, (int64_t)a.chunk / TK_PAGE + 2);
                bs.splits_pages = (int)std::min<int64_t>(seen, max_pages_);
                TkAttnArgs aa{};
                aa.heads = a.heads; aa.kv_heads = a.kv_heads; aa.kv = bs.kv;
                for (int n = 1; n <= TK_MAX_ROWS; ++n) scratch = std::max(scratch, tk_attn_rows_scratch_floats(aa, n, tk_attn_rows_splits(aa, bs.splits_pages, n)));
                if (!rotation(a.rot_dims, a.rot_base, &bs.rope)) return false;
                if (a.taps > 0 && !alloc((void**)&bs.conv, 2 * (size_t)mseq * ((size_t)a.heads * a.dim + (size_t)a.kv_heads * (a.dim + a.vdim)) * (a.taps - 1) * 4, true)) return false;
            } else if (s.branches[b].kind == TkBranchSpec::RETENTION) {
                const TkRetentionSpec& t = s.branches[b].retention;
                const size_t state = (size_t)t.heads * t.dim * ((t.vdim + 3) / 4 * 4);
                std::vector<float> powers;
                for (double x : t.decay)
                    for (int n = 0; n <= TK_RETENTION_BLOCK; ++n) powers.push_back((float)pow(x, n));
                if (!rotation(t.rot_dims, t.rot_base, &bs.rope) || !alloc((void**)&bs.state, 2 * (size_t)mseq * state * 4, true) || !alloc((void**)&bs.decay, powers.size() * 4)) return false;
                HIPQ(hipMemcpy(bs.decay, powers.data(), powers.size() * 4, hipMemcpyHostToDevice));
                sums = std::max(sums, (size_t)ret_slots * state);
            } else {
                const TkDeltaSpec& d = s.branches[b].delta;
                const size_t ch = 2 * (size_t)d.kv_heads * d.dim + (size_t)d.heads * d.vdim;
                if (!alloc((void**)&bs.conv, 2 * (size_t)mseq * ch * (d.taps - 1) * 4, true) ||
                    !alloc((void**)&bs.state, 2 * (size_t)mseq * d.heads * d.dim * ((d.vdim + 3) / 4 * 4) * 4, true))
                    return false;
                dq = std::max(dq, (size_t)d.kv_heads * d.dim);
                dg = std::max(dg, (size_t)d.heads * d.dim);
                dv = std::max(dv, (size_t)d.heads * d.vdim);
                dh = std::max(dh, (size_t)d.heads);
            }
        }
        const TkMlpSpec& f = s.mlp;
        if (f.kind == TkMlpSpec::DENSE) ff = std::max(ff, tk_img_bytes(type, R, f.ff));
        if (f.kind == TkMlpSpec::MOE) {
            const size_t rows = (size_t)R * f.top + 16 * (size_t)std::min<int64_t>(f.experts, (int64_t)R * f.top);
            E = std::max(E, (size_t)f.experts);
            assign = std::max(assign, (size_t)R * f.top);
            moe_rows = std::max(moe_rows, rows);
            gather = std::max(gather, tk_img_bytes(type, (int64_t)rows, c.width));
            moe_ff = std::max(moe_ff, tk_img_bytes(type, (int64_t)rows, f.ff));
        }
    }
    const size_t yrows = std::max<size_t>({(size_t)R, moe_rows, 8 * TK_MAX_ROWS}); /* a product of up to 256 rows may be split over k into eight slabs */
    y_floats_ = yrows * c.width;
    if (!alloc((void**)&x_, (size_t)R * c.width * 4) || !alloc((void**)&proj_, (size_t)R * proj * 4, true) || !alloc((void**)&low_, (size_t)R * low * 4, true) ||
        !alloc((void**)&y_, yrows * c.width * 4, true) || !alloc(&img_x_, tk_img_bytes(type, R, c.width), true) || !alloc(&img_low_, lowk, true) ||
        !alloc(&img_mix_, mix, true) || !alloc(&img_ff_, std::max(ff, moe_ff), true) || !alloc(&img_head_, tk_img_bytes(type, TK_MAX_ROWS, c.width), true) ||
        !alloc(&q_, (size_t)R * q * esz, true) || !alloc((void**)&dq_, (size_t)R * dq * 4) || !alloc((void**)&dk_, (size_t)R * dq * 4) || !alloc((void**)&dv_, (size_t)R * dv * 4) ||
        !alloc((void**)&sums_, sums * 4) || !alloc((void**)&dg_, (size_t)R * dg * 4) || !alloc((void**)&db_, (size_t)R * dh * 4) || !alloc((void**)&do_, (size_t)R * dv * 4) || !alloc((void**)&scratch_, scratch * 4))
        return false;
    if (E && (!alloc((void**)&router_, (size_t)R * ((E + 15) / 16 * 16) * 4) || !alloc(&img_gather_, gather, true) || !alloc((void**)&moe_.count, E * 4, true) ||
              !alloc((void**)&moe_.expert, assign * 4) || !alloc((void**)&moe_.rank, assign * 4) || !alloc((void**)&moe_.weight, assign * 4) || !alloc((void**)&moe_.tile0, E * 4) ||
              !alloc((void**)&moe_.slot, assign * 4) || !alloc((void**)&moe_.blocks, (E + assign / 16 + 1) * sizeof(TkImgBlock), true) || !alloc((void**)&moe_.n_blocks, 4, true)))
        return false;
    if (const char* e = tk_gemm_image_prepare_device()) { error = std::string("LDS opt-in failed: ") + e; return false; }
    if (const char* e = tk_mixer_prepare_device()) { error = std::string("LDS opt-in failed: ") + e; return false; }
    HIPQ(hipDeviceSynchronize());
    return true;
}

TkLayeredSession::~TkLayeredSession() {
    (void)hipSetDevice(device_); /* the model may be gone already */
    if (stream) (void)hipStreamSynchronize(stream);
    for (auto& g : graphs_) if (g) (void)hipGraphExecDestroy(g);
    for (void* p : owned_) (void)hipFree(p);
    if (h_tab_) (void)hipHostFree(h_tab_);
}

/* ------------------------------------------------------------------ pages and state -------- */

void TkLayeredSession::release_sequence(int seq) {
    std::lock_guard<std::mutex> lk(mu_);
    if (seq < 0 || seq >= max_seq) return;
    give_back(seqs_[(size_t)seq]);
}

void TkLayeredSession::give_back(Seq& s) {
    for (auto it = s.pages.rbegin(); it != s.pages.rend(); ++it) free_pages_.push_back(*it);
    s.pages.clear();
    s.len = 0;
    s.prev = -1;
}

void TkLayeredSession::cache_usage(int* used, int* total) {
    std::lock_guard<std::mutex> lk(mu_);
    *total = n_pages_;
    *used = n_pages_ - (int)free_pages_.size();
}

/* the caller has made sure that the pool has them */
void TkLayeredSession::need_pages(Seq& s, int seq, int last_pos) {
    const size_t want = (size_t)last_pos / TK_PAGE + 1;
    while (s.pages.size() < want) {
        h_pages_[(size_t)seq * max_pages_ + s.pages.size()] = free_pages_.back();
        s.pages.push_back(free_pages_.back());
        free_pages_.pop_back();
        pages_dirty_ = true;
    }
}

bool TkLayeredSession::upload_pages() {
    if (!pages_dirty_) return true;
    HIPQ(hipMemcpyAsync(d_pages_, h_pages_.data(), h_pages_.size() * 4, hipMemcpyHostToDevice, stream)); /* pageable: staged before the call returns */
    pages_dirty_ = false;
    return true;
}

/* rows -> segments, tiles, pages and state copies; nothing of a sequence changes but its pages until commit().  mu_ held. */
bool TkLayeredSession::describe(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, Pass* p) {
    const int R = row_cap_;
    int32_t *h_seq = h_tab_, *h_pos = h_seq + R, *h_tok = h_pos + R, *h_seg = h_tok + R, *row0 = h_seg + R, *sn = row0 + max_seq, *sin = sn + max_seq, *sout = sin + max_seq,
            *tiles = sout + max_seq + R;
    TkRetentionBlock* blocks = (TkRetentionBlock*)(h_tab_ + (d_blocks_ - d_tab_));
    *p = Pass();
    p->nrows = nrows; p->singles = false;
    const int per = retention_rows(nrows);
    /* first whether the rows are allowed at all, with nothing changed */
    struct Run { int r, n, side; };
    std::vector<Run> runs;
    std::vector<char> seen((size_t)max_seq, 0);
    for (int r = 0; r < nrows;) {
        int n = 1;
        while (r + n < nrows && seq[r + n] == seq[r] && pos[r + n] == pos[r] + n) ++n;
        const int id = seq[r];
        const Seq& s = seqs_[(size_t)id];
        if (seen[(size_t)id]) { error = "the rows of a sequence must be one run of consecutive positions"; return false; }
        seen[(size_t)id] = 1;
        if (pos[r] != 0 && pos[r] != s.prev && pos[r] != s.len) {
            error = "sequence " + std::to_string(id) + " stands at position " + std::to_string(s.len) + ": its rows must continue there or start at 0";
            return false;
        }
        /* a run at the position where the sequence's last pass began takes that pass back */
        runs.push_back(Run{r, n, pos[r] != 0 && pos[r] == s.prev ? s.side ^ 1 : s.side});
        r += n;
    }
    for (const Run& u : runs)
        if (pos[u.r] == 0) give_back(seqs_[(size_t)seq[u.r]]); /* a new sequence in this slot */
    size_t need = 0;
    for (const Run& u : runs) {
        const size_t want = (size_t)(pos[u.r] + u.n - 1) / TK_PAGE + 1, have = seqs_[(size_t)seq[u.r]].pages.size();
        need += want > have ? want - have : 0;
    }
    if (need > free_pages_.size()) { error = "cache pool exhausted: " + std::to_string(need) + " more pages wanted, " + std::to_string(free_pages_.size()) + " of " + std::to_string(n_pages_) + " are free"; return false; }
    for (const Run& u : runs) {
        const int r = u.r, n = u.n, id = seq[r], side = u.side;
        need_pages(seqs_[(size_t)id], id, pos[r] + n - 1);
        row0[p->nseg] = r; sn[p->nseg] = n;
        sin[p->nseg] = pos[r] == 0 ? -1 : 2 * id + side;
        sout[p->nseg] = 2 * id + (side ^ 1);
        for (int t = 0; t < n; t += 64, ++p->ntiles) { tiles[2 * p->ntiles] = r + t; tiles[2 * p->ntiles + 1] = std::min(64, n - t); }
        for (int i = 0; i < n; ++i) { h_seq[r + i] = id; h_pos[r + i] = pos[r + i]; h_tok[r + i] = tok[r + i]; h_seg[r + i] = p->nseg; }
        if (n > 1) {
            p->single = false;
            const int nb = (n + per - 1) / per;
            if (ret_heads_)
                for (int b = 0; b < nb; ++b) blocks[p->nblocks++] = TkRetentionBlock{r + b * per, std::min(per, n - b * per), p->nseg, p->nsums, b, b + 1 == nb};
            p->nsums += nb - 1;
        } else {
            p->singles = true;
        }
        ++p->nseg;
    }
    return upload_pages();
}

void TkLayeredSession::commit(int nrows, const int32_t* seq, const int32_t* pos) {
    for (int r = 0; r < nrows;) {
        int n = 1;
        while (r + n < nrows && seq[r + n] == seq[r]) ++n;
        Seq& s = seqs_[(size_t)seq[r]];
        if (pos[r] != s.prev || pos[r] == 0) s.side ^= 1; /* a pass that replaced the one it took back wrote the same copy again */
        s.prev = pos[r] == 0 ? -1 : pos[r];
        s.len = pos[r] + n;
        r += n;
    }
}

/* ------------------------------------------------------------------ the layers ------------- */

void TkLayeredSession::gemm(const TkImgGemm& g, int* slabs) {
    if (const char* e = tk_launch_gemm_image(g, stream, slabs))
        if (launch_error.empty()) launch_error = e;
}

void TkLayeredSession::enqueue_moe(const TkLayerSpec& s, const TkLayeredLayer& L, int nrows) {
    const TkMlpSpec& f = s.mlp;
    const int type = m_->type, D = m_->cfg.width, kt = tk_img_kt(type), xkt = tk_img_pad_k(type, D) / kt, fkt = L.down.K / kt;
    TkImgGemm g{};
    g.type = type; g.w = L.router.img; g.a = img_x_; g.K = L.router.K; g.N = L.router.N; g.nrows = nrows;
    g.out = router_; g.ldc = L.router.N; g.n_valid = f.experts;
    gemm(g);
    const int64_t assign = (int64_t)nrows * f.top;
    const int64_t per = assign / f.experts;
    const int bt = per <= 16 ? 1 : per <= 32 ? 2 : per <= 64 ? 4 : 8;
    tk_launch_moe_select(router_, L.router.N, f.experts, f.top, f.groups, f.keep, nrows, bt, moe_, stream);
    tk_launch_moe_gather(img_x_, img_gather_, xkt, f.top, nrows, moe_, stream);
    TkImgGemm u{};
    u.type = type; u.w = L.gate_up.img; u.a = img_gather_; u.K = L.gate_up.K; u.N = L.gate_up.N;
    u.swiglu = 1; u.act_img = img_ff_; u.act_ktiles = fkt; u.act_valid = f.ff;
    u.blocks = moe_.blocks; u.n_blocks = moe_.n_blocks; u.block_tiles = bt; u.group_bytes = L.gate_up.bytes;
    u.max_blocks = (int)(std::min<int64_t>(f.experts, assign) + assign / (16 * bt));
    gemm(u);
    TkImgGemm d = u;
    d.w = L.down.img; d.a = img_ff_; d.K = L.down.K; d.N = L.down.N; d.swiglu = 0; d.act_img = nullptr; d.group_bytes = L.down.bytes;
    d.out = y_; d.ldc = D; d.n_valid = D;
    gemm(d);
}

void TkLayeredSession::enqueue_layers(const Pass& p) {
    const TkLayeredConfig& c = m_->cfg;
    const int type = m_->type, D = c.width, kt = tk_img_kt(type), xkt = tk_img_pad_k(type, D) / kt, n = p.nrows;
    hipStream_t s = stream;
    tk_launch_layer_embed(type, m_->embed, D, c.embed_scale, d_tok, n, x_, m_->layers[0].pre1, c.eps, img_x_, xkt, s);
    for (size_t l = 0; l < c.layers.size(); ++l) {
        const TkLayerSpec& spec = c.layers[l];
        const TkLayeredLayer& L = m_->layers[l];
        const TkNorm after = l + 1 < c.layers.size() ? m_->layers[l + 1].pre1 : TkNorm{}; /* on the next layer's input: fused into this layer's last kernel */
        const int pitch = proj_pitch(L.in.N);
        TkImgGemm g{};
        g.type = type; g.w = L.in.img; g.a = img_x_; g.K = L.in.K; g.N = L.in.N; g.nrows = n;
        g.out = proj_; g.ldc = pitch; g.n_valid = L.in.rows;
        if (L.low_cols) { g.copy_img = img_low_; g.copy0 = L.low_col; g.copy1 = L.low_col + L.low_cols; g.copy_ktiles = L.low.K / kt; }
        gemm(g);
        if (L.low_cols) { /* outer sides of all low-rank gates: one block-diagonal product */
            TkImgGemm w{};
            w.type = type; w.w = L.low.img; w.a = img_low_; w.K = L.low.K; w.N = L.low.N; w.nrows = n; w.out = low_; w.ldc = L.low.N; w.n_valid = L.low.rows;
            gemm(w);
        }
        /* attention and delta branches are prepared in pairs: one launch when a layer has one of each */
        std::vector<TkAttnArgs> as;
        std::vector<TkDeltaArgs> ds;
        std::vector<int> visible; /* pages an attention branch may see at most */
        for (size_t b = 0; b < spec.branches.size(); ++b) {
            const TkBranchSpec& bs = spec.branches[b];
            const TkLayeredBranch& B = L.branches[b];
            const BranchState& st = st_[l][b];
            if (bs.kind == TkBranchSpec::ATTENTION) {
                const TkAttnSpec& sp = bs.attn;
                TkAttnArgs a{};
                a.heads = sp.heads; a.kv_heads = sp.kv_heads; a.dim = sp.dim; a.vdim = sp.vdim; a.rot_dims = sp.rot_dims; a.window = sp.window; a.keep_first = sp.keep_first;
                a.chunk = sp.chunk; a.softcap = sp.softcap; a.taps = sp.taps; a.conv = B.conv; a.conv_state = st.conv;
                a.scale = sp.scale; a.out_scale = bs.scale; a.eps = c.eps; a.col = B.col; a.bias = B.bias; a.q_norm = B.q_norm; a.k_norm = B.k_norm;
                a.rope_cos = st.rope.c; a.rope_sin = st.rope.s; a.q = q_; a.kv = st.kv; a.out_img = img_mix_; a.out_k0 = B.out_k0; a.out_ktiles = L.out.K / kt;
                as.push_back(a);
                visible.push_back(st.splits_pages);
            } else if (bs.kind == TkBranchSpec::RETENTION) { /* reads the projections itself */
                const TkRetentionSpec& sp = bs.retention;
                TkRetentionArgs a{};
                a.heads = sp.heads; a.dim = sp.dim; a.vdim = sp.vdim; a.rot_dims = sp.rot_dims; a.out_scale = bs.scale; a.eps = c.eps; a.col = B.col;
                a.rope_cos = st.rope.c; a.rope_sin = st.rope.s; a.decay = st.decay; a.state = st.state; a.sums = sums_;
                a.out_img = img_mix_; a.out_k0 = B.out_k0; a.out_ktiles = L.out.K / kt;
                if (p.nblocks) tk_launch_retention_scan(type, a, proj_, pitch, tab_, (const TkRetentionBlock*)d_blocks_, p.nblocks, p.nsums, s);
                if (p.singles) tk_launch_retention_step(type, a, proj_, pitch, tab_, p.nseg, s);
            } else {
                const TkDeltaSpec& sp = bs.delta;
                TkDeltaArgs d{};
                d.heads = sp.heads; d.kv_heads = sp.kv_heads; d.dim = sp.dim; d.vdim = sp.vdim; d.taps = sp.taps; d.out_scale = bs.scale; d.eps = c.eps; d.unit_eps = sp.unit_eps;
                d.col = B.col; d.conv = B.conv; d.a_log = B.a_log; d.dt_bias = B.dt_bias; d.norm = B.norm; d.low = low_; d.low_ld = L.low.N; d.low_a = B.low_a; d.low_g = B.low_g;
                d.q = dq_; d.k = dk_; d.v = dv_; d.g = dg_; d.beta = db_; d.o = do_; d.conv_state = st.conv; d.state = st.state;
                d.out_img = img_mix_; d.out_k0 = B.out_k0; d.out_ktiles = L.out.K / kt;
                ds.push_back(d);
            }
        }
        /* q_ and the delta buffers are shared: a branch is finished before the next of its kind is prepared */
        for (size_t i = 0, ai = 0, di = 0; i < std::max(as.size(), ds.size()); ++i, ++ai, ++di) {
            const TkAttnArgs* a = ai < as.size() ? &as[ai] : nullptr;
            const TkDeltaArgs* d = di < ds.size() ? &ds[di] : nullptr;
            tk_launch_mixer_prep(type, proj_, pitch, a, d, tab_, n, s);
            if (!p.single) {
                if (a) tk_launch_attn_tiles(type, *a, tab_, d_tiles_, p.ntiles, s);
                if (d) tk_launch_delta_scan(type, *d, tab_, p.nseg, n, s);
                continue;
            }
            const int splits = a ? tk_attn_rows_splits(*a, visible[ai], n) : 1;
            if (a && d && splits == 1 && tk_launch_mixers_step(type, *a, *d, tab_, n, s)) continue;
            if (a) tk_launch_attn_rows(type, *a, tab_, n, splits, scratch_, s);
            if (d) tk_launch_delta_step(type, *d, tab_, n, s);
        }
        TkImgGemm o{};
        o.type = type; o.w = L.out.img; o.a = img_mix_; o.K = L.out.K; o.N = L.out.N; o.nrows = n; o.out = y_; o.ldc = D; o.n_valid = D;
        /* products whose result goes to a norm may come in slabs, as many as y_ holds */
        const size_t slab = (size_t)n * D;
        const int most = slab % 4 == 0 ? (int)std::min<size_t>(8, y_floats_ / slab) : 1;
        int slabs = 1;
        o.max_slabs = most; o.slab_floats = slab;
        gemm(o, &slabs);
        tk_launch_post_norm(type, TkSubOut{y_, D, slabs, slab, L.out_bias, 1.0f, nullptr, nullptr, 0}, L.norm1, spec.mlp.kind == TkMlpSpec::NONE ? after : L.pre2, c.eps, D, n, x_, img_x_, xkt, s);
        if (spec.mlp.kind == TkMlpSpec::DENSE) {
            TkImgGemm u{};
            u.type = type; u.w = L.gate_up.img; u.a = img_x_; u.K = L.gate_up.K; u.N = L.gate_up.N; u.nrows = n;
            u.swiglu = 1; u.act_img = img_ff_; u.act_ktiles = L.down.K / kt; u.act_valid = spec.mlp.ff;
            if (spec.mlp.act == TkMlpSpec::CLAMPED) { u.act_clamped = 1; u.act_limit = spec.mlp.limit; u.act_slope = spec.mlp.slope; u.act_shift = spec.mlp.shift; }
            gemm(u);
            TkImgGemm w{};
            w.type = type; w.w = L.down.img; w.a = img_ff_; w.K = L.down.K; w.N = L.down.N; w.nrows = n; w.out = y_; w.ldc = D; w.n_valid = D;
            w.max_slabs = most; w.slab_floats = slab;
            gemm(w, &slabs);
            tk_launch_post_norm(type, TkSubOut{y_, D, slabs, slab, nullptr, 0.0f, nullptr, nullptr, 0}, L.norm2, after, c.eps, D, n, x_, img_x_, xkt, s);
        } else if (spec.mlp.kind == TkMlpSpec::MOE) {
            enqueue_moe(spec, L, n);
            tk_launch_post_norm(type, TkSubOut{y_, D, 1, 0, nullptr, 0.0f, moe_.slot, moe_.weight, spec.mlp.top}, L.norm2, after, c.eps, D, n, x_, img_x_, xkt, s);
        }
        if (streams_) (void)hipMemcpyAsync(streams_ + l * (size_t)n * D, x_, (size_t)n * D * 4, hipMemcpyDeviceToHost, s);
    }
}

void TkLayeredSession::enqueue_head(int n, const int32_t* d_rows, int32_t* tok, int32_t* pos) {
    const TkLayeredConfig& c = m_->cfg;
    const int type = m_->type;
    tk_launch_rows_norm(type, x_, d_rows, n, m_->final_norm, c.eps, c.width, img_head_, m_->head.K / tk_img_kt(type), stream);
    TkImgGemm g{};
    g.type = type; g.w = m_->head.img; g.a = img_head_; g.K = m_->head.K; g.N = m_->head.N; g.nrows = n; g.out = logits; g.ldc = c.vocab; g.n_valid = c.vocab;
    gemm(g);
    tk_launch_argmax(logits, c.vocab, n, d_mask, d_mask_row, d_samp, tok, pos, pos ? d_nsteps : nullptr, pos ? d_hist : nullptr, TK_MAX_ROWS, stream);
}

hipGraphExec_t* TkLayeredSession::decode_slot(int nrows, int) { return &graphs_[nrows]; }

/* every row is a sequence of its own and every row is sampled */
void TkLayeredSession::enqueue_decode(int nrows) {
    Pass p;
    p.nrows = p.nseg = nrows;
    enqueue_layers(p);
    enqueue_head(nrows, nullptr, d_tok, d_pos);
    tk_launch_swap_state(tab_, nrows, stream);
}

/* ------------------------------------------------------------------ passes ----------------- */

bool TkLayeredSession::run(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, float* logits_host, int32_t* argmax_host, bool head,
                           const uint32_t* const* row_masks, const TkSampleRow* row_samp, int n_out, const int32_t* out_rows) {
    HIPQ(hipStreamSynchronize(stream)); /* the tables' staging buffer may still be read by the previous pass */
    Pass p;
    {
        std::lock_guard<std::mutex> lk(mu_);
        live_.clear();
        if (!describe(nrows, seq, pos, tok, &p)) return false;
    }
    bool all = head && n_out == nrows && nrows <= TK_MAX_ROWS;
    for (int i = 0; i < n_out && out_rows; ++i) {
        h_tab_[(size_t)(d_out_rows_ - d_tab_) + i] = out_rows[i];
        all = all && out_rows[i] == i;
    }
    if (!out_rows)
        for (int i = 0; i < n_out; ++i) h_tab_[(size_t)(d_out_rows_ - d_tab_) + i] = i;
    HIPQ(hipMemcpyAsync(d_tab_, h_tab_, tab_ints_ * 4, hipMemcpyHostToDevice, stream));
    HIPQ(hipMemsetAsync(d_nsteps, 0, TK_MAX_ROWS * 4, stream));
    launch_error.clear();
    if (all && p.single) { /* a decode step: the same launches every time, replayed */
        if (!stage_sampling(nrows, nullptr, row_masks, row_samp)) return false;
        if (graphs_enabled() && !streams_) {
            if (!capture(&graphs_[nrows], [&] { enqueue_decode(nrows); })) return false;
            HIPQ(hipGraphLaunch(graphs_[nrows], stream));
        } else {
            enqueue_decode(nrows);
        }
        if (logits_host) HIPQ(hipMemcpyAsync(logits_host, logits, (size_t)nrows * vocab_ * 4, hipMemcpyDeviceToHost, stream));
        if (argmax_host) HIPQ(hipMemcpyAsync(argmax_host, d_tok, nrows * 4, hipMemcpyDeviceToHost, stream));
    } else {
        enqueue_layers(p);
        for (int o = 0; head && o < n_out; o += TK_MAX_ROWS) {
            const int k = std::min(TK_MAX_ROWS, n_out - o);
            if (!stage_sampling(k, h_tab_ + (d_out_rows_ - d_tab_) + o, row_masks, row_samp)) return false;
            enqueue_head(k, d_out_rows_ + o, d_otok_, nullptr);
            if (logits_host) HIPQ(hipMemcpyAsync(logits_host + (size_t)o * vocab_, logits, (size_t)k * vocab_ * 4, hipMemcpyDeviceToHost, stream));
            if (argmax_host) HIPQ(hipMemcpyAsync(argmax_host + o, d_otok_, k * 4, hipMemcpyDeviceToHost, stream));
        }
    }
    if (!launch_error.empty()) { error = launch_error; (void)hipStreamSynchronize(stream); return false; }
    HIPQ(hipGetLastError());
    HIPQ(hipStreamSynchronize(stream));
    std::lock_guard<std::mutex> lk(mu_);
    commit(nrows, seq, pos);
    if (all && p.single) live_.assign(seq, seq + nrows);
    return true;
}

bool TkLayeredSession::forward(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, float* logits_host, int32_t* argmax_host, bool lm_head,
                               const uint32_t* const* row_masks, const TkSampleRow* row_samp, int n_out, const int32_t* out_rows) {
    if (nrows <= 0) { error = "nrows must be positive"; return false; }
    if (!rows_in_range(nrows, seq, pos, tok)) return false;
    for (int i = 0; i < n_out && out_rows; ++i)
        if (out_rows[i] < 0 || out_rows[i] >= nrows || (i && out_rows[i] <= out_rows[i - 1])) { error = "wanted rows must be ascending rows of the pass"; return false; }
    if (!out_rows) n_out = nrows;
    HIPQ(hipSetDevice(device_));
    /* more rows than a pass holds: passes in order; a run that is cut continues in the next one */
    int done_out = 0;
    std::vector<int32_t> local;
    for (int r = 0; r < nrows; r += row_cap_) {
        const int n = std::min(row_cap_, nrows - r);
        local.clear();
        if (lm_head)
            for (int i = done_out; i < n_out && (out_rows ? out_rows[i] : i) < r + n; ++i) local.push_back((out_rows ? out_rows[i] : i) - r);
        const int k = (int)local.size();
        if (!run(n, seq + r, pos + r, tok + r, logits_host ? logits_host + (size_t)done_out * vocab_ : nullptr, argmax_host ? argmax_host + done_out : nullptr, lm_head && k > 0,
                 row_masks ? row_masks + r : nullptr, row_samp ? row_samp + r : nullptr, k, local.data()))
            return false;
        done_out += k;
    }
    return true;
}

bool TkLayeredSession::forward_streams(int nrows, const int32_t* seq, const int32_t* pos, const int32_t* tok, float* streams_host) {
    if (nrows <= 0 || nrows > row_cap_) { error = "nrows must be in [1, rows of a pass]"; return false; }
    if (!rows_in_range(nrows, seq, pos, tok)) return false;
    HIPQ(hipSetDevice(device_));
    streams_ = streams_host;
    const bool ok = run(nrows, seq, pos, tok, nullptr, nullptr, false, nullptr, nullptr, 0, nullptr);
    streams_ = nullptr;
    return ok;
}

bool TkLayeredSession::prefill(int nseq, int n_prompt, const int32_t* tokens, int32_t* first_tokens_host) {
    if (nseq <= 0 || nseq > max_seq) { error = "nseq must be in [1, max_seq]"; return false; }
    if (n_prompt <= 0 || n_prompt >= max_ctx) { error = "prompt does not fit the context"; return false; }
    /* all but the last token of every prompt, nobody reads their logits; then one decode step whose rows decode() continues from */
    std::vector<int32_t> sq, ps, tk;
    for (int s = 0; s < nseq; ++s)
        for (int i = 0; i + 1 < n_prompt; ++i) { sq.push_back(s); ps.push_back(i); tk.push_back(tokens[(size_t)s * n_prompt + i]); }
    if (!sq.empty() && !forward((int)sq.size(), sq.data(), ps.data(), tk.data(), nullptr, nullptr, false)) return false;
    sq.clear(); ps.clear(); tk.clear();
    for (int s = 0; s < nseq; ++s) { sq.push_back(s); ps.push_back(n_prompt - 1); tk.push_back(tokens[(size_t)s * n_prompt + n_prompt - 1]); }
    return forward(nseq, sq.data(), ps.data(), tk.data(), nullptr, first_tokens_host, true);
}

bool TkLayeredSession::begin_decode(int nrows, const int32_t* pos, int n_steps) {
    std::lock_guard<std::mutex> lk(mu_);
    if (nrows > (int)live_.size()) { error = "decode() continues the rows of the previous decode step or forward() that sampled every row"; return false; }
    size_t need = 0;
    for (int r = 0; r < nrows; ++r) {
        const Seq& s = seqs_[(size_t)live_[(size_t)r]];
        if (s.len != pos[r]) { error = "a sequence has been released or moved since its row was sampled"; return false; }
        const size_t want = (size_t)(pos[r] + n_steps - 1) / TK_PAGE + 1;
        need += want > s.pages.size() ? want - s.pages.size() : 0;
    }
    if (need > free_pages_.size()) { error = "cache pool exhausted: the decode loop wants " + std::to_string(need) + " more pages"; return false; }
    for (int r = 0; r < nrows; ++r) need_pages(seqs_[(size_t)live_[(size_t)r]], live_[(size_t)r], pos[r] + n_steps - 1);
    return upload_pages();
}

void TkLayeredSession::end_decode(int nrows, int steps) {
    std::lock_guard<std::mutex> lk(mu_);
    live_.resize((size_t)nrows);
    if (steps < 1) return;
    for (int r = 0; r < nrows; ++r) {
        Seq& s = seqs_[(size_t)live_[(size_t)r]];
        s.len += steps;
        s.prev = s.len - 1;
        s.side ^= steps & 1;
    }
}
