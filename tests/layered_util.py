"""Small layer-list checkpoints for the tests: configurations, random weights, and the folder (config.json + model.safetensors) the loader reads."""
import json
import os
import struct
import sys

import numpy as np

sys.path.insert(0, os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "oracle"))
import layered_oracle as LO  # noqa: E402


def bf16_bits(x):
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_round(x):
    return (bf16_bits(x).astype(np.uint32) << 16).view(np.float32)


def attention(heads, kv, dim, vdim, rot, size, keep, scale=None, base=10000.0):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "rot": {"dims": rot, "base": base}, "scale": scale or dim ** -0.5,
            "mask": {"size": size, "keep_first": keep}}


def delta(heads, kv, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def layer(left, right, mlp, ls=1.0, rs=1.0):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": ls, "right_scale": rs}, "mlp": mlp}


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Vuvulorn", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


def retention(heads, dim, vdim, rot, decay, base=10000.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"dims": rot, "base": base}, "decay": list(decay)}


def chunked(heads, kv, dim, vdim, rot, size, conv, softcap, scale=None, base=10000.0):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "rot": {"dims": rot, "base": base}, "scale": scale or dim ** -0.5,
            "mask": {"size": size}, "conv": conv, "softcap": softcap}


def serial(mixer, mlp=None, weights_of=None):
    """a Kaparax layer; mlp: (ff, limit)"""
    L = {"type": "retention" if "decay" in mixer else "attention", "mixer": mixer, "mlp": mlp and {"kind": "dense", "ff": mlp[0], "limit": mlp[1]}}
    if weights_of is not None:
        L["weights_of"] = weights_of
    return L


def kaparax(width, vocab, layers, eps=1e-5, scale=1.0):
    return {"architecture": "Kaparax", "embedding": {"scale": scale}, "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


def kaparax_weights(cfg, seed, gain=1.0):
    """every tensor, values that bf16 holds exactly; gain: of the queries and keys of attention, and of the feed-forward's gates (caps and limits are reached)"""
    rng = np.random.default_rng(seed)
    D, w = cfg["width"], {}

    def mat(name, n, k, f=1.0):
        w[name] = f * rng.standard_normal((n, k)) / np.sqrt(k)

    def norm(name):
        w[name] = 1.0 + 0.2 * rng.standard_normal(D)
        w[name + ".b"] = 0.2 * rng.standard_normal(D)

    w["embed"] = rng.standard_normal((cfg["vocab"], D))
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, m = "l%d." % i, L["mixer"]
        norm(p + "norm1")
        norm(p + "norm1b")
        if L["type"] == "retention":
            for n, rows in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
                mat(p + "mix." + n, m["heads"] * rows, D)
        else:
            for n, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                mat(p + "mix." + n, rows, D, gain if n != "v" else 1.0)
                w[p + "mix." + n + ".conv"] = rng.standard_normal((rows, m["conv"])) / np.sqrt(m["conv"])
        mat(p + "mix.o", D, m["heads"] * m["vdim"])
        if L["mlp"]:
            norm(p + "norm2")
            norm(p + "norm2b")
            mat(p + "mlp.gate", L["mlp"]["ff"], D, gain)
            mat(p + "mlp.up", L["mlp"]["ff"], D, gain)
            mat(p + "mlp.down", D, L["mlp"]["ff"])
    norm("final.norm")
    mat("head", cfg["vocab"], D)
    return {k: bf16_round(v) for k, v in w.items()}


def random_weights(cfg, seed, rank_a=9, rank_g=13):
    """every tensor of the configuration, values that bf16 holds exactly"""
    if cfg["architecture"] == "Kaparax":
        return kaparax_weights(cfg, seed)
    rng = np.random.default_rng(seed)
    D, w = cfg["width"], {}

    def mat(name, n, k):
        w[name] = rng.standard_normal((n, k)) / np.sqrt(k)

    def near_one(name, n):
        w[name] = 1.0 + 0.2 * rng.standard_normal(n)

    w["embed"] = rng.standard_normal((cfg["vocab"], D))
    for i, L in enumerate(cfg["layers"]):
        p, a, d = "l%d." % i, L["mixer"]["left"], L["mixer"]["right"]
        l, r = p + "mix.left.", p + "mix.right."
        for n, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
            mat(l + n, rows, D)
            w[l + n + ".b"] = 0.3 * rng.standard_normal(rows)
        mat(l + "o", D, a["heads"] * a["vdim"])
        w[l + "o.b"] = 0.3 * rng.standard_normal(D)
        near_one(l + "q.norm", a["dim"])
        near_one(l + "k.norm", a["dim"])
        nk, nv = d["kv_heads"] * d["dim"], d["heads"] * d["vdim"]
        for n, rows in (("q", nk), ("k", nk), ("v", nv)):
            mat(r + n, rows, D)
            w[r + n + ".conv"] = rng.standard_normal((rows, d["conv"])) / np.sqrt(d["conv"])
        mat(r + "b", d["heads"], D)
        w[r + "A_log"] = np.log(rng.uniform(0.5, 6.0, d["heads"]))
        w[r + "dt_bias"] = rng.uniform(-5.0, -1.0, d["heads"] * d["dim"])
        mat(r + "a1", rank_a, D)
        mat(r + "a2", d["heads"] * d["dim"], rank_a)
        mat(r + "g1", rank_g, D)
        mat(r + "g2", nv, rank_g)
        near_one(r + "norm", d["vdim"])
        mat(r + "o", D, nv)
        near_one(p + "norm1", D)
        m = L["mlp"]
        if m:
            near_one(p + "norm2", D)
            if m["kind"] == "dense":
                names, ff = [p + "mlp."], m["ff"]
            else:
                names, ff = [p + "mlp.e%d." % e for e in range(m["router"]["experts"])], m["expert"]["ff"]
                mat(p + "mlp.router", m["router"]["experts"], D)
            for n in names:
                mat(n + "gate", ff, D)
                mat(n + "up", ff, D)
                mat(n + "down", D, ff)
    near_one("final.norm", D)
    mat("head", cfg["vocab"], D)
    return {k: bf16_round(v) for k, v in w.items()}


def write_folder(path, cfg, w):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, at, blobs = {}, 0, []
    for name, x in w.items():
        b = bf16_bits(x).tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(x)), "data_offsets": [at, at + len(b)]}
        at += len(b)
        blobs.append(b)
    h = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    return str(path)


def rel_rms(got, want, quantile=1.0):
    """root mean square difference over the vocabulary, mean taken off, in units of the logits' spread; the worst row (or a quantile of the rows)"""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    s = np.asarray(want, np.float64)
    s = np.sqrt(np.mean((s - s.mean(-1, keepdims=True)) ** 2))
    return float(np.quantile(np.sqrt((d * d).mean(-1)), quantile) / s)


def feed(session, slot, tokens, cuts, start=0):
    """the tokens of one sequence in portions; logits of every position"""
    out, at = [], start
    for n in cuts:
        r = range(at - start, at - start + n)
        lg, _ = session.forward_rows([slot] * n, range(at, at + n), [tokens[i] for i in r], range(n))
        out.append(lg)
        at += n
    assert at - start == len(tokens)
    return np.concatenate(out)


F32 = 2e-5   # worst row's rms difference in units of the logits' spread
BF16 = 0.06  # of nine rows in ten: where a router's choice is close, bf16 inputs may take another expert than the restatement


def close(got, want, tol):
    return rel_rms(got, want, 1.0 if tol < 1e-3 else 0.9) < tol


def tokens_for(cfg, n, seed=11):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


class Case:
    """a checkpoint on disk, its restatement, and models per dtype"""

    def __init__(self, tk, path, cfg, seed=7, w=None):
        self.tk, self.cfg = tk, cfg
        self.w = w if w is not None else random_weights(cfg, seed)
        self.dir = write_folder(path, cfg, self.w)
        self.models, self.known = {}, {}

    def session(self, dtype, max_seq=4, max_ctx=512, pool=0):
        if dtype not in self.models:
            self.models[dtype] = self.tk.LlmModel(folder=self.dir, dtype=dtype)
        return self.tk.LlmSession(self.models[dtype], max_seq, max_ctx, pool_tokens=pool)

    def want(self, tokens):
        k = tuple(tokens)
        if k not in self.known:
            self.known[k] = LO.forward(self.cfg, self.w, tokens)
        return self.known[k]


def greedy(session, slot, prompt, n):
    out, at, nxt = [], len(prompt), None
    _, ids = session.forward_rows([slot] * at, range(at), prompt, [at - 1], want_logits=False, want_ids=True)
    for _ in range(n):
        nxt = int(ids[0])
        out.append(nxt)
        _, ids = session.forward_rows([slot], [at], [nxt], [0], want_logits=False, want_ids=True)
        at += 1
    return out


def runner_ids(runner, prompt, n):
    runner.prepare_ids(prompt)
    out = []
    for _ in range(n):
        i = runner.pending_id
        if runner.next_token() is None:
            break
        out.append(i)
    return out


def no_end(ids, n):
    """what a runner yields of a greedy continuation: it stops at the end-of-sequence id"""
    return ids[:ids.index(2)] if 2 in ids[:n] else ids[:n]
