"""Plain numpy restatement (float64) of the layer-list decoders, one function per mechanism: TEST INFRASTRUCTURE ONLY.

A model is (config dict, {tensor name: array}); nothing here is shared with the product.  Every function handles one whole sequence, token
by token where the mechanism is a recurrence, with no cache, no chunks and no batches: what the paged, chunked, batched product is compared with.
"""
import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rms(x, eps):
    """x over the root of its mean square (last axis)"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rotate_half(x, pos, dims, base):
    """x [T, heads, dim]: dimension i turns with i + dims / 2 by the angle pos * base^(-2 i / dims); dimensions >= dims stay"""
    half = dims // 2
    if half == 0:
        return x.copy()
    ang = pos[:, None] * base ** (-2.0 * np.arange(half) / dims)[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = x.copy()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def visible(i, j, size, keep):
    """may position i read position j: a sliding window of `size` positions (0: no window) plus the first `keep` positions"""
    return j <= i and (not size or i - j < size or j < keep)


def softmax_attention(q, k, v, scale, size, keep):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim]"""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    idx = np.arange(T)
    for i in range(T):
        m = (idx <= i) & ((idx < keep) | (i - idx < size) if size else True)
        for h in range(H):
            g = h // (H // G)
            sc = k[m, g] @ q[i, h] * scale
            w = np.exp(sc - sc.max())
            out[i, h] = (w / w.sum()) @ v[m, g]
    return out


def window_attention_mixer(cfg, w, p, h, eps):
    """softmax attention with per-head norms on q and k, partial rotation, a window and kept first positions"""
    T = h.shape[0]
    H, G, dim, vdim = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, dim)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, dim)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, vdim)
    q = rms(q, eps) * w[p + "q.norm"]
    k = rms(k, eps) * w[p + "k.norm"]
    pos = np.arange(T, dtype=np.float64)
    q = rotate_half(q, pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    k = rotate_half(k, pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    o = softmax_attention(q, k, v, cfg["scale"], cfg["mask"]["size"], cfg["mask"]["keep_first"])
    return o.reshape(T, H * vdim) @ w[p + "o"].T + w[p + "o.b"]


def causal_conv(x, taps):
    """x [T, C], taps [C, n]: y[t] = sum_j taps[:, j] x[t - (n - 1) + j], zeros before the start"""
    n = taps.shape[1]
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                y[t] += taps[:, j] * x[s]
    return y


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def gated_delta_rule(q, k, v, beta, g):
    """q, k, g [T, H, dim], v [T, H, vdim], beta [T, H]: state S [dim, vdim] per head, rows decayed by g, then the rank-one correction that moves
    S^T k towards v; the output reads the updated state"""
    T, H, dim = k.shape
    S = np.zeros((H, dim, v.shape[2]))
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            S[h] *= g[t, h][:, None]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] += np.outer(k[t, h], u)
            o[t, h] = S[h].T @ q[t, h]
    return o


def delta_gates(w, p, h, H, dim):
    """(beta [T, H], decay [T, H, dim])"""
    T = h.shape[0]
    beta = sigmoid(h @ w[p + "b"].T)
    a = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    g = np.exp(-np.exp(w[p + "A_log"])[None, :, None] * softplus(a).reshape(T, H, dim))
    return beta, g


def gated_head_norm(o, w, p, h, eps):
    T, H, vdim = o.shape
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(T, H, vdim)
    return rms(o, eps) * w[p + "norm"] * gate


def delta_mixer(cfg, w, p, h, eps):
    T = h.shape[0]
    H, G, dim, vdim = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = silu(causal_conv(h @ w[p + "q"].T, w[p + "q.conv"])).reshape(T, G, dim)
    k = silu(causal_conv(h @ w[p + "k"].T, w[p + "k.conv"])).reshape(T, G, dim)
    v = silu(causal_conv(h @ w[p + "v"].T, w[p + "v.conv"])).reshape(T, H, vdim)
    q, k = unit(q) * dim ** -0.5, unit(k)
    q, k = np.repeat(q, H // G, axis=1), np.repeat(k, H // G, axis=1)
    beta, g = delta_gates(w, p, h, H, dim)
    o = gated_delta_rule(q, k, v, beta, g)
    return gated_head_norm(o, w, p, h, eps).reshape(T, H * vdim) @ w[p + "o"].T


def swiglu(w, p, h):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(scores, top, count, keep):
    """scores [experts] -> chosen expert ids: groups ranked by the sum of their two best scores, then the `top` best experts of the kept groups"""
    E = len(scores)
    per = E // count
    rank = [np.sort(scores[i * per:(i + 1) * per])[::-1][:2].sum() for i in range(count)]
    groups = np.argsort(-np.array(rank), kind="stable")[:keep]
    cand = [e for e in range(E) if e // per in groups]
    return sorted(cand, key=lambda e: (-scores[e], e))[:top]


def moe(cfg, w, p, h):
    r = cfg["router"]
    grp = r.get("groups") or {"count": 1, "keep": 1}
    s = sigmoid(h @ w[p + "router"].T)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e in route(s[t], r["top"], grp["count"], grp["keep"]):
            out[t] += s[t, e] * swiglu(w, p + "e%d." % e, h[t])
    return out


def vuvulorn(cfg, w, tokens):
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    stream = []
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        if L["type"] != "parallel":
            raise ValueError("unknown layer type " + L["type"])
        y = m["left_scale"] * window_attention_mixer(m["left"], w, p + "mix.left.", x, eps) + \
            m["right_scale"] * delta_mixer(m["right"], w, p + "mix.right.", x, eps)
        x = x + rms(y, eps) * w[p + "norm1"]
        ff = L.get("mlp")
        if ff:
            y = swiglu(w, p + "mlp.", x) if ff["kind"] == "dense" else moe(ff, w, p + "mlp.", x)
            x = x + rms(y, eps) * w[p + "norm2"]
        stream.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T, np.array(stream)


# ---- Kaparax: retention and chunked attention layers between layer norms ----

def layer_norm(x, gain, shift, eps):
    """x less its mean, over the root of its variance, per row"""
    c = x - x.mean(axis=-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * gain + shift


def retention(q, k, v, decay):
    """q, k [T, H, dim], v [T, H, vdim], decay [H]: a state [dim, vdim] per head that fades by a constant and gains k v^T; read by q after the gain"""
    T, H, dim = k.shape
    S = np.zeros((H, dim, v.shape[2]))
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + np.outer(k[t, h], v[t, h])
            o[t, h] = q[t, h] @ S[h]
    return o


def retention_mixer(cfg, w, p, h, eps):
    T = h.shape[0]
    H, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    pos = np.arange(T, dtype=np.float64)
    q, k = ((h @ w[p + n].T).reshape(T, H, dim) for n in "qk")
    q, k = (rotate_half(z, pos, cfg["rot"]["dims"], cfg["rot"]["base"]) for z in (q, k))
    o = retention(q, k * dim ** -0.5, (h @ w[p + "v"].T).reshape(T, H, vdim), cfg["decay"])
    return (rms(o, eps).reshape(T, H * vdim) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def same_chunk(i, j, size):
    """may position i read position j: a chunk of `size` positions, counted from the sequence's start (0: no chunks), is closed to the next ones"""
    return j <= i and (not size or i // size == j // size)


def capped(score, cap):
    """scores pressed into (-cap, cap); None: left as they are"""
    return cap * np.tanh(score / cap) if cap else score


def chunked_attention(q, k, v, scale, size, cap):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim]"""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        js = [j for j in range(i + 1) if same_chunk(i, j, size)]
        for h in range(H):
            sc = capped(k[js, h // per] @ q[i, h] * scale, cap)
            e = np.exp(sc - sc.max())
            out[i, h] = (e / e.sum()) @ v[js, h // per]
    return out


def chunked_attention_mixer(cfg, w, p, h):
    T = h.shape[0]
    H, G, dim, vdim = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q, k, v = (causal_conv(h @ w[p + n].T, w[p + n + ".conv"]) for n in "qkv")
    pos = np.arange(T, dtype=np.float64)
    q = rotate_half(q.reshape(T, H, dim), pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    k = rotate_half(k.reshape(T, G, dim), pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    o = chunked_attention(q, k, v.reshape(T, G, vdim), cfg["scale"], (cfg.get("mask") or {}).get("size"), cfg.get("softcap"))
    return o.reshape(T, H * vdim) @ w[p + "o"].T


def clamped_glu(w, p, h, limit):
    """the gate is cut above, the linear side on both sides and moved by one"""
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def kaparax(cfg, w, tokens):
    eps = cfg["norm"]["eps"]

    def norm(name, z):
        return layer_norm(z, w[name], w[name + ".b"], eps)

    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    stream = []
    for i, L in enumerate(cfg["layers"]):
        while cfg["layers"][i].get("weights_of") is not None:
            i = cfg["layers"][i]["weights_of"]
        p = "l%d." % i
        h = norm(p + "norm1", x)
        y = retention_mixer(L["mixer"], w, p + "mix.", h, eps) if L["type"] == "retention" else chunked_attention_mixer(L["mixer"], w, p + "mix.", h)
        x = x + norm(p + "norm1b", y)
        if L.get("mlp"):
            x = x + norm(p + "norm2b", clamped_glu(w, p + "mlp.", norm(p + "norm2", x), L["mlp"]["limit"]))
        stream.append(x)
    return norm("final.norm", x) @ w["head"].T, np.array(stream)


def forward(cfg, w, tokens):
    """(logits [T, vocab], residual stream after every layer [layers, T, width]) of one sequence"""
    w = {k: np.asarray(v, np.float64) for k, v in w.items()}
    return {"Vuvulorn": vuvulorn, "Kaparax": kaparax}[cfg["architecture"]](cfg, w, tokens)
