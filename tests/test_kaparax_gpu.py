"""GPU: Kaparax (retention and chunked attention layers) against the plain numpy restatement, and against itself cut and batched in other ways."""
import copy
import json
import os
import subprocess
import sys
import threading

import numpy as np
import pytest

import layered_util as U
from layered_util import LO, Case, chunked, greedy, kaparax, no_end, retention, runner_ids, serial, tokens_for

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": 1e-5, "bfloat16": 0.03}
DTYPES = sorted(TOL)

CONFIGS = {
    # nothing a multiple of anything; layers borrow tensors (one of them a borrower's); a decay of 1; caps and limits that bite
    "odd": kaparax(93, 131, [serial(retention(3, 20, 36, 12, [0.9, 1.0, 0.3])),
                             serial(chunked(4, 2, 24, 40, 12, 17, 3, 4.0), (70, 1.5)),
                             serial(retention(2, 33, 21, 0, [0.7, 0.97]), (50, 0.8)),
                             serial(chunked(4, 2, 24, 40, 12, 17, 3, 4.0), (70, 1.5), 1),
                             serial(retention(3, 20, 36, 12, [0.9, 1.0, 0.3]), None, 0),
                             serial(retention(3, 20, 36, 12, [0.9, 1.0, 0.3]), None, 4),
                             serial(chunked(2, 2, 18, 10, 4, 33, 1, 50.0))], eps=1e-3, scale=2.5),
    # wide heads, one head, one tap and many, chunks over more than one page
    "wide": kaparax(64, 96, [serial(retention(1, 160, 200, 32, [0.99]), (33, 2.0)),
                             serial(chunked(2, 1, 160, 200, 32, 140, 16, 20.0)),
                             serial(retention(2, 16, 256, 16, [0.5, 0.999], base=500.0)),
                             serial(chunked(1, 1, 128, 16, 128, 70, 2, 9.0, base=500.0), (40, 1.0))]),
    # sizes that fill the kernels' tiles exactly
    "full": kaparax(96, 80, [serial(retention(2, 64, 128, 64, [0.95, 0.99])),
                             serial(chunked(4, 2, 64, 64, 32, 48, 4, 15.0), (64, 2.0)),
                             serial(retention(1, 128, 64, 128, [0.98])),
                             serial(retention(1, 256, 256, 256, [0.9])),
                             serial(chunked(2, 1, 128, 128, 64, 128, 4, 25.0), (64, 3.0))], scale=0.5),
    # more query heads per key head than a tile has rows; many small heads
    "grouped": kaparax(80, 64, [serial(chunked(34, 2, 16, 16, 8, 130, 3, 6.0, scale=0.4), (48, 1.2)),
                                serial(retention(40, 4, 4, 2, np.linspace(0.2, 1.0, 40)))]),
}


def near(got, want, dtype, worst=8.0):
    """nine rows in ten within the tolerance, and none far from it: where a retention's output happens to be close to zero, its norm enlarges any rounding"""
    return U.rel_rms(got, want) < worst * TOL[dtype] and (len(got) < 50 or U.rel_rms(got, want, 0.9) < TOL[dtype])


@pytest.fixture(scope="module")
def cases(gpu, tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = Case(gpu, tmp_path_factory.mktemp(name), CONFIGS[name], w=U.kaparax_weights(CONFIGS[name], 7, gain=1.5))
        return made[name]
    return get


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_and_streams(cases, name, dtype):
    c = cases(name)
    toks = tokens_for(c.cfg, 330)
    want, streams = c.want(toks)
    s = c.session(dtype)
    assert near(U.feed(s, 0, toks, [330]), want, dtype)
    st = s.forward_streams([1] * 330, range(330), toks)
    for l in range(len(streams)):
        assert near(st[l], streams[l], dtype), "layer %d" % l


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_token_by_token(cases, name, dtype):
    """decoding through cache, histories and states (replayed graphs), position by position from the first one on"""
    c = cases(name)
    toks = tokens_for(c.cfg, 330)
    want = c.want(toks)[0]
    got = U.feed(c.session(dtype), 2, toks, [1] * 330)
    assert near(got, want, dtype)
    for n in (1, 2, 3):  # the first tokens, where a convolution reaches before the start
        assert near(got[:n], c.want(toks[:n])[0], dtype)


CUTS = [[2] * 75, [3] * 50, [63, 1, 1, 64, 2, 19], [64, 64, 22], [1, 16, 17, 33, 2, 2, 65, 14], [100, 2, 48], [129, 21]]


@pytest.mark.parametrize("cuts", CUTS)
def test_portions(cases, cuts):
    for name in ("odd", "wide"):
        c = cases(name)
        toks = tokens_for(c.cfg, 150)
        for dtype in DTYPES:
            assert near(U.feed(c.session(dtype), 1, toks, cuts), c.want(toks)[0], dtype)


def one(mixer, mlp=None, **kw):
    return kaparax(52, 61, [serial(mixer, mlp)], **kw)


MECHANISMS = {
    "retention": one(retention(3, 14, 22, 6, [0.95, 0.6, 1.0])),
    "retention without memory": one(retention(2, 14, 22, 6, [0.0, 0.0]), eps=0.01),
    "retention, all dimensions turn": one(retention(2, 32, 32, 32, [0.9, 0.99], base=100.0)),
    "attention": one(chunked(6, 3, 14, 22, 6, 41, 4, 10.0)),
    "attention without chunks": one(dict(chunked(2, 1, 14, 22, 6, 1, 4, 10.0), mask=None)),
    "attention without a cap": one(dict(chunked(2, 1, 14, 22, 14, 30, 2, 1.0), softcap=None)),
    "tight cap": one(chunked(2, 2, 14, 22, 6, 41, 4, 0.7, scale=2.0)),
    "feed-forward": one(retention(1, 4, 4, 0, [0.0]), (37, 0.6), eps=0.1),
}


@pytest.mark.parametrize("what", sorted(MECHANISMS))
def test_one_mechanism_at_a_time(gpu, tmp_path, what):
    cfg = MECHANISMS[what]
    c = Case(gpu, tmp_path, cfg, w=U.kaparax_weights(cfg, 23, gain=2.0))
    toks = tokens_for(cfg, 90, 3)
    want, streams = c.want(toks)
    for cuts in ([90], [1] * 90, [40, 2, 48]):
        assert near(U.feed(c.session("float32"), 0, toks, cuts), want, "float32")
    assert near(c.session("float32").forward_streams([0] * 90, range(90), toks)[0], streams[0], "float32")


@pytest.mark.parametrize("dim,vdim", [(20, 100), (64, 130), (64, 256), (70, 17), (128, 64), (100, 128), (128, 200), (130, 20), (256, 128), (200, 256)])
def test_retention_sizes(gpu, tmp_path, dim, vdim):
    """every form of the scan and of the step: segments of several blocks, of one, and of parts of one"""
    cfg = kaparax(40, 50, [serial(retention(2, dim, vdim, dim // 4 * 2, [0.97, 0.999]))])
    c = Case(gpu, tmp_path, cfg, seed=dim)
    toks = tokens_for(cfg, 200)
    want = c.want(toks)[0]
    for dtype in DTYPES:
        s = c.session(dtype)
        for cuts in ([200], [130, 1, 1, 2, 66], [33, 65, 64, 3, 35]):
            assert near(U.feed(s, 0, toks, cuts), want, dtype), cuts


def test_long_blocks(gpu, tmp_path):
    """so many heads that a scan's blocks are longer than one chunk, several segments in a pass, singles between them"""
    cfg = kaparax(32, 40, [serial(retention(64, 4, 8, 4, np.linspace(0.9, 0.9999, 64)))])
    c = Case(gpu, tmp_path, cfg)
    toks = [tokens_for(cfg, n, n) for n in (700, 1, 300, 1, 257)]
    s = c.session("float32", 5, 1024)
    seq = sum(([i] * len(t) for i, t in enumerate(toks)), [])
    lg, _ = s.forward_rows(seq, sum((list(range(len(t))) for t in toks), []), sum(toks, []), range(len(seq)))
    for i, t in enumerate(toks):
        assert near(lg[np.array(seq) == i], c.want(t)[0], "float32"), i
    for i, t in ((0, toks[0]), (4, toks[4])):  # and what the pass left behind
        got, _ = s.forward_rows([i, i], [len(t), len(t) + 1], [5, 6], [0, 1])
        assert near(got, c.want(t + [5, 6])[0][-2:], "float32")


# ---- keys that stand out: keys are made from one half of a token's (normed) embedding, queries from the other half by the same matrix, so a token
# whose second half repeats another token's first half asks for exactly that token: a wrong chunk edge or a wrong page shows ----

def edge_case(gpu, path, size, T, places):
    cfg = kaparax(64, 300, [serial(chunked(2, 1, 32, 32, 2, size, 3, 40.0, scale=0.5))])
    w = U.kaparax_weights(cfg, 5)
    for n in ("l0.norm1", "l0.norm1.b"):
        w[n] = np.full_like(w[n], 0.0 if n.endswith("b") else 1.0)
    for n in "qk":  # the convolutions pass their input through
        w["l0.mix.%s.conv" % n] = np.tile(np.array([0, 0, 1], np.float32), (len(w["l0.mix.%s.conv" % n]), 1))
    half = w["l0.mix.k"][:, :32] * 2.0
    w["l0.mix.k"] = U.bf16_round(np.concatenate([half, 0 * half], axis=1))
    w["l0.mix.q"] = U.bf16_round(np.concatenate([np.concatenate([0 * half, half], axis=1)] * 2))
    toks = list(range(2, T + 2))
    for i, at in enumerate(places):
        w["embed"][T + 2 + i, 32:] = w["embed"][toks[at], :32]
    return Case(gpu, path, cfg, w=w), toks


@pytest.mark.parametrize("size,T", [(40, 200), (64, 200), (64, 193), (65, 200), (1, 140), (130, 250), (100, 201), (7, 140)])
def test_edges_of_chunks_and_pages(gpu, tmp_path, size, T):
    last = T - 1
    edge = last // size * size
    places = sorted({p for p in (edge, edge + 1, edge - 1, edge - 2, edge - size, last - size, last - 1, 0, 63, 64, 127, 128) if 0 <= p < last})
    c, toks = edge_case(gpu, tmp_path, size, T, places)
    sessions = [(d, c.session(d)) for d in DTYPES]
    for i, at in enumerate(places):
        t = toks[:last] + [T + 2 + i]  # the last token asks for the one at `at`
        want = c.want(t)[0][last]
        for mistake in (size + 1, size - 1, last - at, 10 ** 6):
            if mistake < 1 or LO.same_chunk(last, at, mistake) == LO.same_chunk(last, at, size):
                continue
            bad = copy.deepcopy(c.cfg)
            bad["layers"][0]["mixer"]["mask"]["size"] = mistake
            assert U.rel_rms(LO.forward(bad, c.w, t)[0][last], want) > 0.1, "the mistake would not show"
        for dtype, s in sessions:
            for cuts in ([T], [last, 1], [last - 1, 2], [last - 70, 70, 1], [edge, T - edge] if edge else [T]):
                assert near(U.feed(s, 0, t, cuts)[last:], want[None], dtype, 1.0), (at, cuts)
                s.release(0)


def test_state_reaches_across_portions_and_restarts_at_zero(gpu, tmp_path):
    """a decay close to 1: the first token still shows in the last position's logits, through portions, blocks and single tokens; a slot used again starts clean"""
    cfg = kaparax(48, 60, [serial(retention(2, 12, 12, 4, [0.9995, 0.999]))])
    c = Case(gpu, tmp_path, cfg, seed=9)
    toks = tokens_for(cfg, 420, 4)
    changed = [(toks[0] + 1) % 60] + toks[1:]
    want, want2 = c.want(toks)[0], c.want(changed)[0]
    assert U.rel_rms(want2[-1], want[-1]) > 100 * TOL["float32"]
    s = c.session("float32")
    for cuts in ([420], [1] * 420, [2] * 210, [50, 2, 3, 300, 65]):
        assert near(U.feed(s, 0, toks, cuts)[-1], want[-1], "float32")
        assert near(U.feed(s, 0, changed, cuts)[-1], want2[-1], "float32")  # position 0 again: the slot starts anew


def test_history_reaches_across_portions(gpu, tmp_path):
    """a convolution that only reads its oldest tap: every portion and every token reads what the one before left behind"""
    cfg = kaparax(48, 60, [serial(chunked(2, 1, 12, 16, 4, 50, 5, 9.0))])
    w = U.kaparax_weights(cfg, 9)
    for n in "qkv":
        w["l0.mix.%s.conv" % n] = np.tile(np.array([1, 0, 0, 0, 0], np.float32), (len(w["l0.mix.%s.conv" % n]), 1))
    c = Case(gpu, tmp_path, cfg, w=w)
    toks = tokens_for(cfg, 120, 4)
    for dtype in DTYPES:
        s = c.session(dtype)
        for cuts in ([120], [1] * 120, [2] * 60, [3] * 40, [4] * 30, [5] * 24, [50, 2, 3, 65]):
            assert near(U.feed(s, 0, toks, cuts), c.want(toks)[0], dtype)


def test_borrowed_tensors_equal_copied_ones(cases, gpu, tmp_path):
    """a layer that uses another's tensors keeps a cache and a state of its own: the same as a model that holds the tensors twice"""
    c = cases("odd")
    cfg, w = copy.deepcopy(c.cfg), dict(c.w)
    for i, owner in ((3, 1), (4, 0), (5, 0)):
        del cfg["layers"][i]["weights_of"]
        w.update({"l%d.%s" % (i, k[len("l%d." % owner):]): v for k, v in c.w.items() if k.startswith("l%d." % owner)})
    twice = Case(gpu, tmp_path, cfg, w=w)
    toks = tokens_for(cfg, 100)
    for dtype in DTYPES:
        for cuts in ([100], [60] + [1] * 40):
            assert np.array_equal(U.feed(c.session(dtype), 0, toks, cuts), U.feed(twice.session(dtype), 0, toks, cuts))
    assert c.models["float32"].weight_bytes == twice.models["float32"].weight_bytes  # a step streams them as often


# ---- batches, pages, slots ----

@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_requests_share_passes_pages_and_slots(cases, dtype):
    """twelve requests of 1 .. 200 tokens over four slots and a pool that holds far fewer than all: portions of some beside single tokens of others,
    requests left out of steps, pages and slots used again"""
    c = cases("odd")
    rng = np.random.default_rng(31)
    s = c.session(dtype, 4, 256, pool=512)
    todo = [tokens_for(c.cfg, n, 100 + n) for n in (1, 200, 65, 2, 130, 64, 7, 63, 128, 33, 90, 3)]
    live, free, got, done = {}, [2, 0, 3, 1], {}, 0
    while todo or live:
        while todo and free and sum((len(t) + 63) // 64 for t, _, _ in live.values()) + (len(todo[0]) + 63) // 64 <= 8:
            t = todo.pop(0)
            live[free.pop()] = (t, 0, done)
            got[done] = (t, [])
            done += 1
        seq, pos, tok, who = [], [], [], []
        for slot, (t, at, i) in list(live.items()):
            if len(live) > 1 and rng.random() < 0.25:
                continue
            n = min(len(t) - at, int(rng.choice([1, 1, 2, 3, 17, 64, 70])))
            seq += [slot] * n
            pos += range(at, at + n)
            tok += t[at:at + n]
            who += [i] * n
            live[slot] = (t, at + n, i)
        if not seq:
            continue
        lg, ids = s.forward_rows(seq, pos, tok, range(len(seq)), want_ids=True)
        assert np.array_equal(ids, lg.argmax(1))
        for r, i in enumerate(who):
            got[i][1].append(lg[r])
        for slot, (t, at, i) in list(live.items()):
            if at == len(t):
                s.release(slot)
                free.append(slot)
                del live[slot]
    for t, rows in got.values():
        assert near(np.array(rows), c.want(t)[0], dtype)
    assert s.cache_usage() == (0, 8)


def test_many_sequences_decode_together(cases):
    """forty sequences of different lengths, four steps of one token each, against the restatement of every one"""
    c = cases("odd")
    toks = [tokens_for(c.cfg, 1 + 3 * i, i) for i in range(40)]
    s = c.session("float32", 40, 192)
    for i, t in enumerate(toks):
        U.feed(s, i, t, [len(t)])
    for k in range(4):
        lg, _ = s.forward_rows(range(40), [len(t) for t in toks], [7 + k] * 40, range(40))
        for t in toks:
            t.append(7 + k)
    want = np.array([LO.forward(c.cfg, c.w, t)[0][-1] for t in toks])
    assert near(lg, want, "float32")


def test_last_pass_can_be_taken_back(cases):
    c = cases("odd")
    toks, wrong = tokens_for(c.cfg, 80), tokens_for(c.cfg, 80, 99)
    s = c.session("float32")
    U.feed(s, 0, toks[:60], [60])
    for n in (1, 5, 1):
        s.forward_rows([0] * n, range(60, 60 + n), wrong[:n], [0])
    assert near(U.feed(s, 0, toks[60:], [2, 1, 1, 16], start=60), c.want(toks)[0][60:], "float32")


def test_more_rows_than_a_pass_holds(gpu, tmp_path):
    cfg = kaparax(32, 40, [serial(retention(2, 8, 8, 4, [0.99, 0.9999])), serial(chunked(2, 1, 8, 8, 4, 300, 4, 9.0), (16, 1.0))])
    c = Case(gpu, tmp_path, cfg)
    toks = tokens_for(cfg, 2300)
    s = c.session("float32", 2, 2400)
    assert s.row_capacity < 2300
    whole = U.feed(s, 0, toks, [2300])
    assert near(whole, U.feed(s, 1, toks, [700, 1, 2, 997, 600]), "float32")
    assert near(whole[:200], c.want(toks[:200])[0], "float32")


# ---- generation ----

@pytest.mark.parametrize("dtype", DTYPES)
def test_device_driven_decode_loop(cases, dtype, monkeypatch):
    """the captured loop against one pass per token and, in 32-bit, against the restatement, over 300 steps; and without graphs"""
    c = cases("odd")
    s = c.session(dtype, 3, 512)
    prompts = np.array([tokens_for(c.cfg, 50, 60 + i) for i in range(3)], np.int32)
    first = s.prefill(prompts)
    toks, _ = s.decode(3, 150)
    more, _ = s.decode(3, 151)
    got = np.concatenate([first[None], toks, more])
    ref = c.session(dtype, 3, 512)
    nxt = ref.prefill(prompts)
    for k in range(302):
        assert np.array_equal(nxt, got[k, :3])
        _, nxt = ref.forward_rows(range(3), [50 + k] * 3, nxt, range(3), want_logits=False, want_ids=True)
    if dtype == "float32":
        ids = prompts[0].tolist() + [int(t) for t in got[:, 0]]
        want = c.want(ids[:-1])[0]
        lg, _ = s.forward_rows([0], [len(ids) - 1], [ids[-1]], [0])  # the host takes over where the loop stopped
        assert near(lg, c.want(ids)[0][-1:], dtype)
        margin = np.sort(want[49:], axis=1)
        sure = margin[:, -1] - margin[:, -2] > 1e-3
        assert sure.sum() > 250 and np.array_equal(want[49:].argmax(1)[sure], got[:, 0][sure])
    monkeypatch.setenv("TK_MI355X_NO_GRAPH", "1")
    e = c.session(dtype, 3, 512)
    assert np.array_equal(e.prefill(prompts), first)
    assert np.array_equal(e.decode(3, 150)[0], toks)


def test_runners_share_the_scheduler(cases):
    """loader, registry, continuous batching with run-ahead rows: every runner on its thread sees what it would see alone"""
    c = cases("odd")
    tk = c.tk
    loader = tk.ModelLoader()
    h = loader.load(c.dir + "?dtype=float32")
    loader.set_runner_slots(h, 4)
    ref = c.session("float32", 1, 512)
    prompts = [tokens_for(c.cfg, n, 40 + n) for n in (5, 70, 129, 1)]
    want = [no_end(greedy(ref, 0, p, 60), 60) for p in prompts]
    runners = [tk.LlmRunner(h, context_size=512) for _ in prompts]
    got = [None] * 4

    def work(i):
        got[i] = [runner_ids(runners[i], prompts[i], 60) for _ in range(2)]
    th = [threading.Thread(target=work, args=(i,)) for i in range(4)]
    for t in th:
        t.start()
    for t in th:
        t.join()
    for i in range(4):
        assert got[i] == [want[i], want[i]], i
    for r in runners:
        r.close()
    r = tk.LlmRunner(h, context_size=512)  # a slot another runner gave back
    assert runner_ids(r, prompts[1], 30) == no_end(want[1], 30)
    r.close()
    loader.close()


# ---- loading, command line ----

def test_loader_names_what_is_wrong_with_a_folder(gpu, tmp_path):
    cfg = CONFIGS["grouped"]
    w = U.random_weights(cfg, 1)
    for i, name in enumerate(("l0.norm1b.b", "l0.mix.k.conv", "l1.mix.g", "final.norm.b")):
        with pytest.raises(gpu.TkError, match=name):
            gpu.LlmModel(folder=U.write_folder(tmp_path / str(i), cfg, {k: v for k, v in w.items() if k != name}))


def test_random_weights_model(gpu):
    m = gpu.LlmModel(config=CONFIGS["wide"], seed=3)
    s = gpu.LlmSession(m, 2, 128)
    lg, ids = s.forward_rows([0] * 40, range(40), tokens_for(CONFIGS["wide"], 40), range(40), want_ids=True)
    assert np.isfinite(lg).all() and len(set(ids.tolist())) > 3


def test_trace_runner(cases, tmp_path):
    c = cases("wide")
    a, b = tokens_for(c.cfg, 90, 1), tokens_for(c.cfg, 33, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:70], "want": [69, 3, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": b[:31]}, {"id": "x", "tokens": a[70:71], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[71:], "want": [18]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "y", "tokens": b[31:], "want": [1, 0]}], "end": ["y"]}]
    for dtype in DTYPES:
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", c.dir, "--dtype", dtype, "--out", str(out), "--max-tokens", "192"],
                           input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr
        A, B = c.want(a)[0], c.want(b)[0]
        read = lambda i: np.fromfile(out / ("%d.f32" % i), "<f4").reshape(-1, c.cfg["vocab"])
        assert near(read(0), A[[69, 3, 3]], dtype) and near(read(1), A[[70]], dtype)
        assert near(read(2), A[[89]], dtype) and near(read(3), B[[32, 31]], dtype)
