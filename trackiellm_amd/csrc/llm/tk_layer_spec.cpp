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

bool read_attention(Reader& r, const JVal* m, const std::string& w, TkAttnSpec* a) {
    if (!read_heads(r, m, w, TK_MAX_HEAD_DIM, TK_MAX_HEAD_DIM, &a->heads, &a->kv_heads, &a->dim, &a->vdim) || !r.real(m, "scale", w, &a->scale)) return false;
    if (const JVal* rot = m->get("rot"); is_set(rot)) {
        if (!r.integer(rot, "dims", w + ".rot", 0, a->dim, &a->rot_dims) || !r.num(rot, "base", w + ".rot", &a->rot_base)) return false;
        if (a->rot_dims % 2) return r.fail(w + ".rot.dims is odd");
    }
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

/* Vuvulorn: every layer runs window attention and a gated delta rule side by side on the un-normed stream; norms on the sublayers' outputs */
bool parse_vuvulorn(const JVal& root, TkLayeredConfig* c, std::string* err) {
    Reader r{err};
    if (!r.integer(&root, "width", "config", 1, 1 << 20, &c->width) || !r.integer(&root, "vocab", "config", 1, 1 << 24, &c->vocab)) return false;
    const JVal* norm = r.obj(&root, "norm", "config");
    if (!norm || !r.real(norm, "eps", "norm", &c->eps)) return false;
    const JVal* layers = root.get("layers");
    if (!layers || layers->kind != JVal::JARR || layers->arr.empty()) return r.fail("layers is missing");
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
            !read_attention(r, left, w + ".mixer.left", &a.attn) || !read_delta(r, right, w + ".mixer.right", &d.delta))
            return false;
        if (const JVal* mlp = L->get("mlp"); is_set(mlp)) {
            s.mlp.prefix = p + "mlp.";
            if (!read_mlp(r, mlp, w + ".mlp", &s.mlp)) return false;
        }
        c->layers.push_back(std::move(s));
    }
    return true;
}

struct Entry { const char* name; bool (*parse)(const JVal&, TkLayeredConfig*, std::string*); };
const Entry g_architectures[] = {{"Vuvulorn", parse_vuvulorn}};

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
