#include "tk_layer_spec.h"

#include <math.h>
#include <string.h>

#include "../common/tk_json.h"

using namespace tk_json;

namespace {

/* typed access with the path of what is missing in the message */
struct Reader {
    std::string* err;
    bool fail(const std::string& why) { if (err->empty()) *err = "config.json: " + why; return false; }
    const JVal* obj(const JVal* v, const char* key, const std::string& where) {
        const JVal* o = v ? v->get(key) : nullptr;
        if (!o || o->kind != JVal::JOBJ) { fail(where + "." + key + " is missing"); return nullptr; }
        return o;
    }
    bool num(const JVal* v, const char* key, const std::string& where, double* out) {
        const JVal* n = v ? v->get(key) : nullptr;
        if (!n || n->kind != JVal::JNUM) return fail(where + "." + key + " is missing");
        *out = n->num;
        return true;
    }
    bool integer(const JVal* v, const char* key, const std::string& where, int lo, int hi, int* out) {
        double d;
        if (!num(v, key, where, &d)) return false;
        if (d != floor(d) || d < lo || d > hi) return fail(where + "." + key + " is out of range");
        *out = (int)d;
        return true;
    }
    bool real(const JVal* v, const char* key, const std::string& where, float* out) {
        double d;
        if (!num(v, key, where, &d)) return false;
        *out = (float)d;
        return true;
    }
};

bool is_set(const JVal* v) { return v && v->kind != JVal::JNULL; }

bool read_heads(Reader& r, const JVal* m, const std::string& w, int max_dim, int max_vdim, int* heads, int* kv, int* dim, int* vdim) {
    if (!r.integer(m, "heads", w, 1, 4096, heads) || !r.integer(m, "kv_heads", w, 1, 4096, kv) || !r.integer(m, "dim", w, 1, max_dim, dim) ||
        !r.integer(m, "vdim", w, 1, max_vdim, vdim))
        return false;
    return *heads % *kv == 0 || r.fail(w + ".heads is not a multiple of kv_heads");
}

bool read_rotation(Reader& r, const JVal* m, const std::string& w, int dim, int* dims, double* base) {
    const JVal* rot = m->get("rot");
    if (!is_set(rot)) return true;
    if (!r.integer(rot, "dims", w + ".rot", 0, dim, dims) || !r.num(rot, "base", w + ".rot", base)) return false;
    if (*dims % 2) return r.fail(w + ".rot.dims is odd");
    return *base > 0.0 || r.fail(w + ".rot.base is not positive");
}

/* sizes, score scale and rotation: what every attention has */
bool read_attention(Reader& r, const JVal* m, const std::string& w, TkAttnSpec* a) {
    return read_heads(r, m, w, TK_MAX_HEAD_DIM, TK_MAX_HEAD_DIM, &a->heads, &a->kv_heads, &a->dim, &a->vdim) && r.real(m, "scale", w, &a->scale) &&
           read_rotation(r, m, w, a->dim, &a->rot_dims, &a->rot_base);
}

bool read_window(Reader& r, const JVal* m, const std::string& w, TkAttnSpec* a) {
    if (const JVal* mask = m->get("mask"); is_set(mask)) {
        if (is_set(mask->get("size")) && !r.integer(mask, "size", w + ".mask", 1, 1 << 30, &a->window)) return false;
        if (is_set(mask->get("keep_first")) && !r.integer(mask, "keep_first", w + ".mask", 0, 1 << 30, &a->keep_first)) return false;
    }
    return true;
}

bool read_delta(Reader& r, const JVal* m, const std::string& w, TkDeltaSpec* d) {
    return read_heads(r, m, w, TK_MAX_DELTA_DIM, TK_MAX_DELTA_VDIM, &d->heads, &d->kv_heads, &d->dim, &d->vdim) &&
           r.integer(m, "conv", w, 1, TK_MAX_CONV_TAPS, &d->taps);
}

/* chunks, capped scores, a convolution ahead of the rotation */
bool read_chunks(Reader& r, const JVal* m, const std::string& w, TkAttnSpec* a) {
    if (const JVal* mask = m->get("mask"); is_set(mask) && is_set(mask->get("size")) && !r.integer(mask, "size", w + ".mask", 1, 1 << 30, &a->chunk)) return false;
    if (is_set(m->get("softcap")) && !r.real(m, "softcap", w, &a->softcap)) return false;
    if (is_set(m->get("conv")) && !r.integer(m, "conv", w, 1, TK_MAX_CONV_TAPS, &a->taps)) return false;
    return a->softcap >= 0.0f || r.fail(w + ".softcap is negative");
}

bool read_retention(Reader& r, const JVal* m, const std::string& w, TkRetentionSpec* o) {
    if (!r.integer(m, "heads", w, 1, 4096, &o->heads) || !r.integer(m, "dim", w, 1, TK_MAX_RETENTION_DIM, &o->dim) || !r.integer(m, "vdim", w, 1, TK_MAX_RETENTION_VDIM, &o->vdim) ||
        !read_rotation(r, m, w, o->dim, &o->rot_dims, &o->rot_base))
        return false;
    const JVal* d = m->get("decay");
    if (!d || d->kind != JVal::JARR || (int)d->arr.size() != o->heads) return r.fail(w + ".decay is not a list of one number per head");
    for (const JVal& v : d->arr) {
        if (v.kind != JVal::JNUM || !(v.num >= 0.0 && v.num <= 1.0)) return r.fail(w + ".decay has a value outside 0 .. 1");
        o->decay.push_back(v.num);
    }
    return true;
}

bool read_mlp(Reader& r, const JVal* m, const std::string& w, TkMlpSpec* o) {
    const JVal* kind = m->get("kind");
    if (!kind || kind->kind != JVal::JSTR) return r.fail(w + ".kind is missing");
    if (kind->str == "dense") {
        o->kind = TkMlpSpec::DENSE;
        return r.integer(m, "ff", w, 1, 1 << 24, &o->ff);
    }
    if (kind->str != "moe") return r.fail(w + ".kind '" + kind->str + "' is unknown");
    o->kind = TkMlpSpec::MOE;
    const JVal *ex = r.obj(m, "expert", w), *ro = r.obj(m, "router", w);
    if (!ex || !ro || !r.integer(ex, "ff", w + ".expert", 1, 1 << 24, &o->ff) || !r.integer(ro, "experts", w + ".router", 1, TK_MAX_EXPERTS, &o->experts) ||
        !r.integer(ro, "top", w + ".router", 1, TK_MAX_TOP, &o->top))
        return false;
    if (const JVal* g = ro->get("groups"); is_set(g)) {
        if (!r.integer(g, "count", w + ".router.groups", 1, 64, &o->groups) || !r.integer(g, "keep", w + ".router.groups", 1, 64, &o->keep)) return false;
        if (o->experts % o->groups || o->keep > o->groups) return r.fail(w + ".router.groups does not divide the experts");
    }
    return o->top <= o->experts / o->groups * o->keep || r.fail(w + ".router.top is larger than the experts that can be chosen");
}

/* what every design gives: width, vocabulary, norm constant; null or the list of layers */
const JVal* read_model(Reader& r, const JVal& root, TkLayeredConfig* c) {
    if (!r.integer(&root, "width", "config", 1, 1 << 20, &c->width) || !r.integer(&root, "vocab", "config", 1, 1 << 24, &c->vocab)) return nullptr;
    const JVal* norm = r.obj(&root, "norm", "config");
    if (!norm || !r.real(norm, "eps", "norm", &c->eps)) return nullptr;
    const JVal* layers = root.get("layers");
    if (!layers || layers->kind != JVal::JARR || layers->arr.empty()) { r.fail("layers is missing"); return nullptr; }
    return layers;
}

/* Vuvulorn: every layer runs window attention and a gated delta rule side by side on the un-normed stream; norms on the sublayers' outputs */
bool parse_vuvulorn(const JVal& root, TkLayeredConfig* c, std::string* err) {
    Reader r{err};
    const JVal* layers = read_model(r, root, c);
    if (!layers) return false;
    for (size_t i = 0; i < layers->arr.size(); ++i) {
        const JVal* L = &layers->arr[i];
        const std::string w = "layers[" + std::to_string(i) + "]", p = "l" + std::to_string(i) + ".";
        const JVal* type = L->get("type");
        if (!type || type->kind != JVal::JSTR || type->str != "parallel") return r.fail(w + ".type is unknown");
        const JVal* m = r.obj(L, "mixer", w);
        const JVal *left = m ? r.obj(m, "left", w + ".mixer") : nullptr, *right = m ? r.obj(m, "right", w + ".mixer") : nullptr;
        if (!left || !right) return false;
        TkLayerSpec s;
        s.norm1 = p + "norm1"; s.norm2 = p + "norm2";
        s.branches.resize(2);
        TkBranchSpec &a = s.branches[0], &d = s.branches[1];
        a.kind = TkBranchSpec::ATTENTION; a.prefix = p + "mix.left."; a.attn.bias = a.attn.qk_norm = true;
        d.kind = TkBranchSpec::DELTA; d.prefix = p + "mix.right.";
        if (!r.real(m, "left_scale", w + ".mixer", &a.scale) || !r.real(m, "right_scale", w + ".mixer", &d.scale) ||
            !read_attention(r, left, w + ".mixer.left", &a.attn) || !read_window(r, left, w + ".mixer.left", &a.attn) || !read_delta(r, right, w + ".mixer.right", &d.delta))
            return false;
        if (const JVal* mlp = L->get("mlp"); is_set(mlp)) {
            s.mlp.prefix = p + "mlp.";
            if (!read_mlp(r, mlp, w + ".mlp", &s.mlp)) return false;
        }
        c->layers.push_back(std::move(s));
    }
    return true;
}

/* do two layers' tensors have the same shapes? */
bool same_shapes(const TkLayerSpec& x, const TkLayerSpec& y) {
    if (x.branches.size() != y.branches.size()) return false;
    for (size_t i = 0; i < x.branches.size(); ++i) {
        const TkBranchSpec &a = x.branches[i], &b = y.branches[i];
        if (a.kind != b.kind || a.attn.heads != b.attn.heads || a.attn.kv_heads != b.attn.kv_heads || a.attn.dim != b.attn.dim || a.attn.vdim != b.attn.vdim ||
            a.attn.taps != b.attn.taps || a.delta.heads != b.delta.heads || a.delta.kv_heads != b.delta.kv_heads || a.delta.dim != b.delta.dim ||
            a.delta.vdim != b.delta.vdim || a.delta.taps != b.delta.taps || a.retention.heads != b.retention.heads || a.retention.dim != b.retention.dim ||
            a.retention.vdim != b.retention.vdim)
            return false;
    }
    return x.mlp.kind == y.mlp.kind && x.mlp.ff == y.mlp.ff && x.mlp.experts == y.mlp.experts;
}

/* Kaparax: retention and chunked attention layers in any order, layer norms before and after every sublayer, a clamped gate in the feed-forward
 * (or none), layers that run another layer's tensors once more */
bool parse_kaparax(const JVal& root, TkLayeredConfig* c, std::string* err) {
    Reader r{err};
    const JVal *layers = read_model(r, root, c), *embedding = layers ? r.obj(&root, "embedding", "config") : nullptr;
    if (!embedding || !r.real(embedding, "scale", "embedding", &c->embed_scale)) return false;
    c->norm = TkLayeredConfig::LAYER;
    const int n = (int)layers->arr.size();
    for (int i = 0; i < n; ++i) {
        const JVal* L = &layers->arr[i];
        const std::string w = "layers[" + std::to_string(i) + "]";
        TkLayerSpec s;
        int owner = i;
        for (int hops = 0; is_set(layers->arr[owner].get("weights_of")); ++hops) {
            const std::string at = "layers[" + std::to_string(owner) + "]";
            if (!r.integer(&layers->arr[owner], "weights_of", at, 0, n - 1, &owner)) return false;
            if (hops > n) return r.fail(w + ".weights_of leads back to itself");
        }
        if (owner != i) s.weights_of = owner;
        const std::string p = "l" + std::to_string(owner) + ".";
        s.pre1 = p + "norm1"; s.norm1 = p + "norm1b"; s.pre2 = p + "norm2"; s.norm2 = p + "norm2b";
        const JVal *type = L->get("type"), *m = r.obj(L, "mixer", w);
        if (!m) return false;
        s.branches.resize(1);
        TkBranchSpec& b = s.branches[0];
        b.prefix = p + "mix.";
        if (type && type->kind == JVal::JSTR && type->str == "retention") {
            b.kind = TkBranchSpec::RETENTION;
            if (!read_retention(r, m, w + ".mixer", &b.retention)) return false;
        } else if (type && type->kind == JVal::JSTR && type->str == "attention") {
            if (!read_attention(r, m, w + ".mixer", &b.attn) || !read_chunks(r, m, w + ".mixer", &b.attn)) return false;
        } else {
            return r.fail(w + ".type is unknown");
        }
        if (const JVal* mlp = L->get("mlp"); is_set(mlp)) {
            s.mlp.prefix = p + "mlp.";
            if (!read_mlp(r, mlp, w + ".mlp", &s.mlp) || !r.real(mlp, "limit", w + ".mlp", &s.mlp.limit)) return false;
            if (s.mlp.kind != TkMlpSpec::DENSE) return r.fail(w + ".mlp.kind is unknown");
            s.mlp.act = TkMlpSpec::CLAMPED;
            s.mlp.slope = 1.702f;
            s.mlp.shift = 1.0f;
        }
        c->layers.push_back(std::move(s));
    }
    for (int i = 0; i < n; ++i)
        if (c->layers[i].weights_of >= 0 && !same_shapes(c->layers[i], c->layers[c->layers[i].weights_of]))
            return r.fail("layers[" + std::to_string(i) + "] has other sizes than the layer whose weights it uses");
    return true;
}

struct Entry { const char* name; bool (*parse)(const JVal&, TkLayeredConfig*, std::string*); };
const Entry g_architectures[] = {{"Vuvulorn", parse_vuvulorn}, {"Kaparax", parse_kaparax}};

} // namespace

std::vector<std::string> tk_layered_architectures() {
    std::vector<std::string> v;
    for (const Entry& e : g_architectures) v.push_back(e.name);
    return v;
}

bool tk_layered_parse(const std::string& text, TkLayeredConfig* out, std::string* err) {
    err->clear();
    JVal root;
    JParser ps{text.data(), text.data() + text.size()};
    if (!ps.value(&root) || root.kind != JVal::JOBJ) { *err = "config.json is not a JSON object"; return false; }
    const JVal* a = root.get("architecture");
    if (!a || a->kind != JVal::JSTR) { *err = "config.json: architecture is missing"; return false; }
    for (const Entry& e : g_architectures)
        if (a->str == e.name) {
            *out = TkLayeredConfig();
            out->architecture = a->str;
            return e.parse(root, out, err);
        }
    *err = "config.json: architecture '" + a->str + "' is not registered";
    return false;
}
