"""GPU: layer-list decoders (Vuvulorn) against the plain numpy restatement, and against themselves cut and batched in other ways."""
import json
import os
import subprocess
import sys
import threading

import numpy as np
import pytest

import layered_util as U
from layered_util import BF16, F32, LO, Case, attention, close, config, delta, dense, greedy, layer, moe, no_end, runner_ids, tokens_for

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

CONFIGS = {
    # nothing a multiple of anything: padded tiles in every product
    "odd": config(93, 131, [layer(attention(4, 2, 24, 40, 12, 17, 3), delta(4, 2, 20, 36, 3), dense(70), 1.2, 0.7),
                            layer(attention(4, 4, 18, 10, 4, 33, 0), delta(3, 1, 9, 7, 5), moe(40, 6, 3, (3, 2)), 0.9, 1.3),
                            layer(attention(2, 1, 24, 24, 0, 9, 1), delta(2, 2, 33, 21, 2), None)], eps=1e-3),
    # wide heads, one head, one tap, experts without groups, kept positions over more than one page
    "wide": config(64, 96, [layer(attention(1, 1, 128, 16, 128, 70, 5, base=500.0), delta(3, 3, 130, 8, 1), moe(16, 4, 1)),
                            layer(attention(2, 1, 160, 200, 32, 40, 70), delta(1, 1, 16, 256, 4), moe(33, 8, 4, (4, 4)), 0.5, 2.0)]),
    # head sizes that fill the attention kernels' tiles exactly
    "full": config(72, 80, [layer(attention(4, 2, 64, 64, 16, 50, 4), delta(2, 1, 32, 64, 4), dense(64)),
                            layer(attention(2, 1, 128, 128, 64, 90, 1), delta(1, 1, 64, 128, 4), None),
                            layer(attention(1, 1, 256, 256, 256, 66, 0), delta(1, 1, 128, 128, 4), moe(24, 4, 2))]),
    # more query heads per key head than a tile has rows, a large state
    "grouped": config(80, 64, [layer(attention(34, 2, 16, 16, 8, 130, 2, scale=0.4), delta(2, 1, 256, 256, 6), dense(48), 1.0, 1.0)]),
}


@pytest.fixture(scope="module")
def cases(gpu, tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = Case(gpu, tmp_path_factory.mktemp(name), CONFIGS[name])
        return made[name]
    return get


@pytest.mark.parametrize("dtype,tol", [("float32", F32), ("bfloat16", BF16)])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_and_streams(cases, name, dtype, tol):
    c = cases(name)
    toks = tokens_for(c.cfg, 150)
    want, streams = c.want(toks)
    s = c.session(dtype)
    got = U.feed(s, 0, toks, [150])
    assert close(got, want, tol)
    st = s.forward_streams([1] * 150, range(150), toks)
    for l in range(len(streams)):
        assert close(st[l], streams[l], tol), "layer %d" % l


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_token_by_token(cases, name):
    """decoding through the cache and the state (replayed graphs), position by position"""
    c = cases(name)
    toks = tokens_for(c.cfg, 150)
    for dtype, tol in (("float32", F32), ("bfloat16", BF16)):
        assert close(U.feed(c.session(dtype), 2, toks, [1] * 150), c.want(toks)[0], tol)


@pytest.mark.parametrize("cuts", [[2] * 75, [3] * 50, [63, 1, 1, 64, 2, 19], [64, 64, 22], [1, 16, 17, 33, 2, 2, 65, 14], [100, 2, 48]])
def test_portions(cases, cuts):
    for name in ("odd", "wide"):
        c = cases(name)
        toks = tokens_for(c.cfg, 150)
        assert close(U.feed(c.session("float32"), 1, toks, cuts), c.want(toks)[0], F32)
    toks = tokens_for(cases("odd").cfg, 150)
    assert close(U.feed(cases("odd").session("bfloat16"), 1, toks, cuts), cases("odd").want(toks)[0], BF16)


def variant(base, **parts):
    """one layer with one mechanism left"""
    c = json.loads(json.dumps(base))
    L = c["layers"][0]
    L["mixer"]["left_scale"], L["mixer"]["right_scale"] = parts.get("scales", (1.0, 1.0))
    if "mlp" in parts:
        L["mlp"] = parts["mlp"]
    c["layers"] = [L]
    return c


@pytest.mark.parametrize("what,parts", [("attention", {"scales": (1.0, 0.0), "mlp": None}), ("delta", {"scales": (0.0, 1.0), "mlp": None}),
                                        ("dense", {"scales": (0.01, 0.0), "mlp": dense(50)}), ("moe", {"scales": (0.01, 0.0), "mlp": moe(20, 12, 5, (4, 2))})])
def test_one_mechanism_at_a_time(gpu, tmp_path, what, parts):
    cfg = variant(CONFIGS["odd"], **parts)
    c = Case(gpu, tmp_path, cfg, seed=23)
    toks = tokens_for(cfg, 90, 3)
    want, streams = c.want(toks)
    for cuts in ([90], [1] * 90, [40, 2, 48]):
        s = c.session("float32")
        assert close(U.feed(s, 0, toks, cuts), want, F32)
    assert close(c.session("float32").forward_streams([0] * 90, range(90), toks)[0], streams[0], F32)


# ---- keys that stand out: keys are made from one half of an embedding, queries from the other half by the same matrix, so a token whose second
# half repeats another token's first half asks for exactly that token: a wrong window edge, a lost first position or a wrong page shows ----

def edge_case(gpu, path, size, keep, T, places):
    cfg = config(64, 300, [layer(attention(2, 1, 32, 32, 2, size, keep, scale=1.2), delta(1, 1, 8, 8, 2), None, 1.0, 0.0)])
    w = U.random_weights(cfg, 5)
    p = "l0.mix.left."
    half = w[p + "k"][:, :32] * 1.5
    w[p + "k"] = U.bf16_round(np.concatenate([half, 0 * half], axis=1))
    w[p + "q"] = np.concatenate([np.concatenate([0 * half, half], axis=1)] * 2)
    w[p + "q"] = U.bf16_round(w[p + "q"])
    w[p + "q.b"], w[p + "k.b"] = 0 * w[p + "q.b"], 0 * w[p + "k.b"]
    w[p + "q.norm"] = w[p + "k.norm"]
    toks = list(range(2, T + 2))
    for i, at in enumerate(places):
        w["embed"][T + 2 + i, 32:] = w["embed"][toks[at], :32]
    return Case(gpu, path, cfg, w=w), toks


@pytest.mark.parametrize("size,keep,T", [(40, 6, 200), (64, 1, 200), (65, 64, 200), (1, 3, 140), (130, 66, 250)])
def test_edges_of_windows_pages_and_kept_positions(gpu, tmp_path, size, keep, T):
    last = T - 1
    places = sorted({p for p in (last - size + 1, last - size, last - size + 2, 0, keep - 1, keep, 63, 64, 127, 128) if 0 <= p < last})
    c, toks = edge_case(gpu, tmp_path, size, keep, T, places)
    asks = [(at, toks[:last] + [T + 2 + i]) for i, at in enumerate(places)]  # the last token asks for the one at `at`
    s32, s16 = c.session("float32"), c.session("bfloat16")
    for at, t in asks:
        want = c.want(t)[0][last]
        other = LO.visible(last, at, size, keep)
        for mistake in ((size + 1, keep), (size - 1, keep), (size, keep + 1), (size, max(keep - 1, 0))):
            if LO.visible(last, at, *mistake) == other or not mistake[0]:
                continue
            bad = json.loads(json.dumps(c.cfg))
            bad["layers"][0]["mixer"]["left"]["mask"] = {"size": mistake[0], "keep_first": mistake[1]}
            assert U.rel_rms(LO.forward(bad, c.w, t)[0][last], want) > 0.2, "the mistake would not show"
        for s, tol in ((s32, F32), (s16, BF16)):
            for cuts in ([T], [last, 1], [last - 1, 2], [last - 70, 70, 1]):
                got = U.feed(s, 0, t, cuts)[last]
                assert close(got, want, tol), (at, cuts)
                s.release(0)


def test_state_reaches_across_portions_and_restarts_at_zero(gpu, tmp_path):
    """slow decays: the first token still shows in the last position's logits, through portions and single tokens; a slot used again starts clean"""
    cfg = config(48, 60, [layer(attention(1, 1, 8, 8, 4, 4, 0), delta(2, 1, 12, 12, 4), None, 0.0, 1.0)])
    w = U.random_weights(cfg, 9)
    w["l0.mix.right.dt_bias"] = np.full_like(w["l0.mix.right.dt_bias"], -12.0)
    w["l0.mix.right.a2"] *= 0.0
    c = Case(gpu, tmp_path, cfg, w=w)
    toks = tokens_for(cfg, 120, 4)
    changed = [(toks[0] + 1) % 60] + toks[1:]
    want, want2 = c.want(toks)[0], c.want(changed)[0]
    assert U.rel_rms(want2[-1], want[-1]) > 100 * F32
    s = c.session("float32")
    for cuts in ([120], [1] * 120, [2] * 60, [50, 2, 3, 65]):
        assert close(U.feed(s, 0, toks, cuts)[-1], want[-1], F32)
        assert close(U.feed(s, 0, changed, cuts)[-1], want2[-1], F32)  # position 0 again: the slot starts anew


# ---- batches, pages, slots ----

@pytest.mark.parametrize("dtype,tol", [("float32", F32), ("bfloat16", BF16)])
def test_unequal_requests_share_passes_pages_and_slots(cases, dtype, tol):
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
        assert close(np.array(rows), c.want(t)[0], tol)
    assert s.cache_usage() == (0, 8)


@pytest.mark.parametrize("dim,vdim", [(20, 20), (40, 36), (70, 17), (130, 20)])
def test_many_heads_and_sequences(gpu, tmp_path, dim, vdim):
    """the recurrence's form for many columns at once: eight sequences of unequal length x 32 heads in one pass, then portions and single tokens"""
    cfg = config(40, 50, [layer(attention(2, 2, 8, 8, 4, 7, 1), delta(32, 16, dim, vdim, 4), dense(24))])
    c = Case(gpu, tmp_path, cfg, seed=dim)
    prompts = [tokens_for(cfg, 21 + 5 * i, i) for i in range(8)]
    s = c.session("float32", 8, 64)
    got = [[] for _ in prompts]
    for lo, hi in ((0, 19), (19, 21), (21, 60)):
        seq, pos, tok = [], [], []
        for i, p in enumerate(prompts):
            part = p[lo:hi]
            seq += [i] * len(part)
            pos += range(lo, lo + len(part))
            tok += part
        if lo == 21:  # the first sequence has ended
            assert 0 not in seq
        lg, _ = s.forward_rows(seq, pos, tok, range(len(seq)))
        for r, i in enumerate(seq):
            got[i].append(lg[r])
    for p, rows in zip(prompts, got):
        assert close(np.array(rows), c.want(p)[0], F32)


def test_wanted_rows_only(cases):
    c = cases("odd")
    toks = tokens_for(c.cfg, 100)
    s = c.session("float32")
    lg, ids = s.forward_rows([0] * 100, range(100), toks, [3, 50, 99], want_ids=True)
    want = c.want(toks)[0]
    assert close(lg, want[[3, 50, 99]], F32) and np.array_equal(ids, lg.argmax(1))
    none, _ = s.forward_rows([1] * 40, range(40), toks[:40], [], want_logits=False)
    assert none is None
    lg, _ = s.forward_rows([1] * 60, range(40, 100), toks[40:], [59])
    assert close(lg, want[[99]], F32)


def test_last_pass_can_be_taken_back(cases):
    """rows at the position where a sequence's last pass began replace that pass: cache, convolution history and state"""
    c = cases("odd")
    toks, wrong = tokens_for(c.cfg, 80), tokens_for(c.cfg, 80, 99)
    want = c.want(toks)[0]
    s = c.session("float32")
    U.feed(s, 0, toks[:60], [60])
    for n in (1, 5, 1):  # replaced again and again
        s.forward_rows([0] * n, range(60, 60 + n), wrong[:n], [0])
    got = U.feed(s, 0, toks[60:], [2, 1, 1, 16], start=60)
    assert close(got, want[60:], F32)
    s.forward_rows([0], [80], [1], [0])
    with pytest.raises(c.tk.TkError):  # two passes back is gone
        s.forward_rows([0], [64], [1], [0])
    got, _ = s.forward_rows([0], [0], toks[:1], [0])
    assert close(got, want[:1], F32)


def test_what_a_pass_refuses(cases):
    c = cases("odd")
    s = c.session("float32", 2, 128, pool=128)
    with pytest.raises(c.tk.TkError, match="stands at"):
        s.forward_rows([0], [5], [1], [0])
    with pytest.raises(c.tk.TkError, match="one run"):
        s.forward_rows([0, 1, 0], [0, 0, 1], [1, 2, 3], [0])
    with pytest.raises(c.tk.TkError, match="out of range"):
        s.forward_rows([0], [0], [c.cfg["vocab"]], [0])
    with pytest.raises(c.tk.TkError, match="out of range"):
        s.forward_rows([0], [128], [0], [0])
    with pytest.raises(c.tk.TkError, match="ascending"):
        s.forward_rows([0, 0], [0, 1], [1, 2], [1, 0])
    toks = tokens_for(c.cfg, 100)
    U.feed(s, 0, toks, [100])
    with pytest.raises(c.tk.TkError, match="exhausted"):
        s.forward_rows([1], [0], [1], [0])
    s.release(0)
    assert close(U.feed(s, 1, toks, [100]), c.want(toks)[0], F32)


def test_more_rows_than_a_pass_holds(gpu, tmp_path):
    cfg = config(32, 40, [layer(attention(2, 1, 8, 8, 4, 300, 2), delta(1, 1, 8, 8, 3), moe(16, 4, 2))])
    c = Case(gpu, tmp_path, cfg)
    toks = tokens_for(cfg, 2300)
    s = c.session("float32", 2, 2400)
    assert s.row_capacity < 2300
    whole = U.feed(s, 0, toks, [2300])
    parts = U.feed(s, 1, toks, [700, 1, 2, 997, 600])
    assert close(whole, parts, F32)
    assert close(whole[:200], c.want(toks[:200])[0], F32)


# ---- generation ----

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_device_driven_decode_loop(cases, dtype, monkeypatch):
    """the captured loop against one pass per token, over 300 steps and several replays, with passes of the host in between; and without graphs"""
    c = cases("odd")
    s = c.session(dtype, 3, 512)
    prompts = np.array([tokens_for(c.cfg, 50, 60 + i) for i in range(3)], np.int32)
    first = s.prefill(prompts)
    toks, ms = s.decode(3, 150)
    more, _ = s.decode(3, 151)
    got = np.concatenate([first[None], toks, more])
    ref = c.session(dtype, 3, 512)
    for i in range(3):
        assert greedy(ref, i, prompts[i].tolist(), 302) == got[:, i].tolist()
    # the host takes over where the loop stopped
    ids = [int(t) for t in got[-1]]
    a, _ = s.forward_rows([0, 1, 2], [50 + 301] * 3, ids, range(3))
    for i in range(3):
        b, _ = ref.forward_rows([i], [50 + 302], [int(a[i].argmax())], [0])
        d, _ = s.forward_rows([i], [50 + 302], [int(a[i].argmax())], [0])
        assert close(d, b, F32 if dtype == "float32" else BF16)
    monkeypatch.setenv("TK_MI355X_NO_GRAPH", "1")
    e = c.session(dtype, 3, 512)
    assert np.array_equal(e.prefill(prompts), first)
    assert np.array_equal(e.decode(3, 150)[0], toks)


def test_decode_loop_keeps_to_what_it_continues(cases):
    c = cases("odd")
    s = c.session("float32", 2, 128)
    s.prefill(np.array([tokens_for(c.cfg, 8, 1), tokens_for(c.cfg, 8, 2)], np.int32))
    s.release(1)
    with pytest.raises(c.tk.TkError, match="released"):
        s.decode(2, 3)
    s.forward_rows([0, 0], [0, 1], [1, 2], [1])
    with pytest.raises(c.tk.TkError, match="continues"):
        s.decode(1, 3)


def test_runners_share_the_scheduler(cases):
    """tk_llm_runner_* on threads: loader, registry, continuous batching with run-ahead rows; every runner sees what it would see alone"""
    c = cases("odd")
    tk = c.tk
    loader = tk.ModelLoader()
    h = loader.load(c.dir + "?dtype=float32")
    assert loader.load(c.dir + "?dtype=float32").value == h.value
    loader.set_runner_slots(h, 4)
    ref = c.session("float32", 1, 512)
    prompts = [tokens_for(c.cfg, n, 40 + n) for n in (5, 70, 129, 1)]
    want = [no_end(greedy(ref, 0, p, 60), 60) for p in prompts]
    runners = [tk.LlmRunner(h, context_size=512) for _ in prompts]
    got = [None] * 4

    def work(i):
        got[i] = [runner_ids(runners[i], prompts[i], 60) for _ in range(2)]  # the second round starts the slot anew
    th = [threading.Thread(target=work, args=(i,)) for i in range(4)]
    for t in th:
        t.start()
    for t in th:
        t.join()
    for i in range(4):
        assert got[i] == [want[i], want[i]], i
    # a runner that stops early, and one that goes another way than the row that ran ahead of it
    r = runners[1]
    r.prepare_ids(prompts[1])
    for _ in range(3):
        r.next_token()
    tk.check(tk.lib().tk_llm_runner_add_tool_response(r.h, b"t", b"x"))
    text = b'[TOOL_RESULT] name: "t", output: x [/TOOL_RESULT]'
    inserted = [min(3 + b, 10 ** 9) if 3 + b < c.cfg["vocab"] else 0 for b in text]
    cont = prompts[1] + want[1][:3] + inserted
    if len(want[1]) >= 3:
        assert r.pending_id == greedy(ref, 0, cont, 1)[0]
    assert runner_ids(runners[0], prompts[2], 20) == no_end(want[2], 20)
    for r in runners:
        r.close()
    r = tk.LlmRunner(h, context_size=512)  # a slot another runner gave back
    assert runner_ids(r, prompts[1], 30) == no_end(want[1], 30)
    r.prepare("a text prompt")
    r.close()
    loader.close()


def test_sampling_chain(cases):
    """the shared sampler on this session: top_k 1 is the arg max, a seed is reproducible, rows keep their own state"""
    c = cases("odd")
    s = c.session("float32", 3, 128)
    toks = tokens_for(c.cfg, 30)
    seq, pos = [0] * 30 + [1] * 30, list(range(30)) * 2
    hot = [(1.5, 40, 0.95, 0.0, 5, r) for r in range(60)]
    lg, a = s.forward_sampled(seq, pos, toks * 2, hot)
    _, b = s.forward_sampled(seq, pos, toks * 2, hot)
    assert np.array_equal(a, b) and not np.array_equal(a, lg.argmax(1))
    _, one = s.forward_sampled(seq, pos, toks * 2, [(1.5, 1, 1.0, 0.0, 5, r) for r in range(60)])
    assert np.array_equal(one, lg.argmax(1))
    _, mixed = s.forward_sampled([2, 0], [0, 0], [1, 2], [(0.0, 0, 1.0, 0.0, 0, 0), (2.0, 40, 0.9, 0.0, 3, 1)])
    assert len(mixed) == 2


# ---- loading ----

def test_loader_names_what_is_wrong_with_a_folder(gpu, tmp_path):
    cfg = CONFIGS["grouped"]
    w = U.random_weights(cfg, 1)
    with pytest.raises(gpu.TkError, match="config.json"):
        gpu.LlmModel(folder=str(tmp_path / "nowhere"))
    missing = {k: v for k, v in w.items() if k != "l0.mlp.up"}
    with pytest.raises(gpu.TkError, match="l0.mlp.up"):
        gpu.LlmModel(folder=U.write_folder(tmp_path / "a", cfg, missing))
    bent = dict(w)
    bent["l0.norm1"] = w["l0.norm1"][:-1]
    with pytest.raises(gpu.TkError, match="l0.norm1"):
        gpu.LlmModel(folder=U.write_folder(tmp_path / "b", cfg, bent))
    d = U.write_folder(tmp_path / "c", cfg, w)
    with pytest.raises(gpu.TkError, match="dtype"):
        gpu.LlmModel(folder=d, dtype="float16")
    with open(os.path.join(d, "model.safetensors"), "r+b") as f:
        f.truncate(4000)
    with pytest.raises(gpu.TkError):
        gpu.LlmModel(folder=d)


def test_random_weights_model(gpu):
    m = gpu.LlmModel(config=CONFIGS["wide"], gate_rank=8, seed=3)
    s = gpu.LlmSession(m, 2, 128)
    lg, ids = s.forward_rows([0] * 40, range(40), tokens_for(CONFIGS["wide"], 40), range(40), want_ids=True)
    assert np.isfinite(lg).all() and len(set(ids.tolist())) > 3
    assert m.weight_bytes > 0


def test_trace_runner(cases, tmp_path):
    c = cases("wide")
    a, b = tokens_for(c.cfg, 90, 1), tokens_for(c.cfg, 33, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:70], "want": [69, 3, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": b[:31]}, {"id": "x", "tokens": a[70:71], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[71:], "want": [18]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "y", "tokens": b[31:], "want": [1, 0]}], "end": ["y"]}]
    for dtype, tol in (("float32", F32), ("bfloat16", BF16)):
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", c.dir, "--dtype", dtype, "--out", str(out), "--max-tokens", "192"],
                           input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr
        assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(4)]
        A, B = c.want(a)[0], c.want(b)[0]
        read = lambda i: np.fromfile(out / ("%d.f32" % i), "<f4").reshape(-1, c.cfg["vocab"])
        assert close(read(0), A[[69, 3, 3]], tol) and close(read(1), A[[70]], tol)
        assert close(read(2), A[[89]], tol) and close(read(3), B[[32, 31]], tol)
