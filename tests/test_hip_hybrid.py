"""The hybrid decoder (Nilivik design) on the GPU against the plain implementation of tests/hybrid_oracle.py: small models with random
weights, float32 compute for sharp comparisons (differences of rounding size only) and bfloat16 compute for the serving path."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from crabml_amd import synth_hybrid as sh
from tests import hybrid_oracle as ho

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# root mean square of the logits' difference over that of the logits
TOL = {True: 2e-5, False: 2e-2}


class Model:
    def __init__(self, config, folder, seed=0, tensors=None):
        self.config = config
        bits = tensors if tensors is not None else sh.random_tensors(config, seed)
        self.tensors = {k: sh.from_bf16(v) for k, v in bits.items()}
        self.folder = sh.write_model(config, bits, str(folder))

    def oracle(self, tokens, config=None, tensors=None):
        return ho.forward(config or self.config, tensors or self.tensors, tokens)

    def runner(self, ca, hdev, f32, seq_len=1024, **kw):
        return ca.load_model(self.folder, hdev, seq_len=seq_len, f32=f32, **kw)

    def tokens(self, n, seed=1):
        return [int(t) for t in np.random.default_rng(seed).integers(0, self.config["vocab"], n)]


def err(got, want):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape
    assert np.isfinite(got).all()
    d = got - want
    return float(np.max(np.sqrt((d * d).mean(axis=-1)) / np.sqrt((want * want).mean())))


def close(got, want, f32, factor=1.0):
    e = err(got, want)
    assert e <= factor * TOL[f32], e


def whole(r, tokens):
    s = r.open()
    lg = r.step([(s, tokens, list(range(len(tokens))))])
    r.close(s)
    return lg


# sizes on purpose unlike one another, unaligned, equal or 1: (width, vocab, layers, loop)
CONFIGS = {
    "plain": sh.config(128, 300, [sh.layer(4, 2, 32, 32, 24, 3, 16, 24, 96), sh.layer(4, 2, 32, 32, 24, 3, 16, 24, 96)]),
    "odd": sh.config(84, 131, [sh.layer(6, 3, 20, 12, 7, 5, 12, 20, 75), sh.layer(3, 1, 36, 44, 50, 2, 28, 36, None)],
                     loop={"start": 0, "stop": 1, "times": 3}, softcap=4.0),
    "loop": sh.config(96, 257, [sh.layer(2, 2, 16, 48, 1000, 1, 64, 8, 50, decay=[1.0]), sh.layer(1, 1, 8, 8, 1, 4, 8, 8, None),
                                sh.layer(10, 1, 24, 24, 33, 2, 40, 72, 130), sh.layer(2, 1, 64, 64, 64, 2, 64, 64, 64)],
                      loop={"start": 1, "stop": 3, "times": 2}),
    "all-loop": sh.config(64, 64, [sh.layer(2, 1, 16, 16, 16, 2, 16, 16, 32)], loop={"start": 0, "stop": 1, "times": 1}),
    "wide-heads": sh.config(160, 200, [sh.layer(2, 1, 136, 100, 90, 2, 144, 48, 200), sh.layer(18, 2, 200, 256, 40, 1, 256, 130, 64)],
                            loop={"start": 1, "stop": 2, "times": 2}),
    "no-mlp": sh.config(72, 99, [sh.layer(4, 4, 24, 8, 12, 4, 8, 16, None), sh.layer(4, 4, 24, 8, 30, 4, 8, 16, None)]),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    base = tmp_path_factory.mktemp("hybrid")
    cache = {}

    def get(name):
        if name not in cache:
            cache[name] = Model(CONFIGS[name], base / name, seed=len(name))
        return cache[name]
    return get


# ---- whole models --------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_every_position(ca, hdev, models, name, f32):
    m = models(name)
    r = m.runner(ca, hdev, f32)
    for n in (1, 2, 3, 65, 150):
        t = m.tokens(n, seed=n)
        close(whole(r, t), m.oracle(t), f32)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_then_token_by_token(ca, hdev, models, name, f32):
    """every logit of the decode step, from the first token on and behind a prompt, over several chunk borders"""
    m = models(name)
    r = m.runner(ca, hdev, f32)
    t = m.tokens(110, seed=5)
    want = m.oracle(t)
    a, b = r.open(), r.open()
    got_a = [r.step([(a, [x], [0])])[0] for x in t[:60]]
    close(got_a, want[:60], f32)
    close(r.step([(b, t[:70], [3, 69])]), want[[3, 69]], f32)
    got_b = [r.step([(b, [x], [0])])[0] for x in t[70:]]
    close(got_b, want[70:], f32)
    assert r.length(a) == 60 and r.length(b) == 110


@pytest.mark.parametrize("name", ["odd", "loop", "plain"])
def test_portions_of_a_prompt(ca, hdev, models, name):
    m = models(name)
    r = m.runner(ca, hdev, True)
    t = m.tokens(140, seed=6)
    want = m.oracle(t)
    for size in (2, 3, 16, 63, 64, 65, 128):
        s, got = r.open(), []
        for i in range(0, len(t), size):
            p = t[i:i + size]
            got.append(r.step([(s, p, list(range(len(p))))]))
        r.close(s)
        close(np.concatenate(got), want, True)


def test_internal_passes_cut_prompts_too(ca, hdev, models):
    """pass_rows far below the batch: entries are split over passes, some passes hold the end of one and the start of another"""
    m = models("odd")
    r = m.runner(ca, hdev, True, pass_rows=50)
    lens = [70, 1, 33, 121, 2]
    prompts = [m.tokens(n, seed=20 + n) for n in lens]
    seqs = [r.open() for _ in lens]
    got = r.step([(s, p, list(range(len(p)))) for s, p in zip(seqs, prompts)])
    close(got, np.concatenate([m.oracle(p) for p in prompts]), True)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("name", ["plain", "loop"])
def test_unequal_batch_against_each_alone(ca, hdev, models, name, f32):
    """prompts of different lengths as one batch, decoded together; shorter ones leave early; then more sequences than a decode step
    takes, and a step that mixes portions with single tokens"""
    m = models(name)
    r = m.runner(ca, hdev, f32)
    lens = [1, 66, 23, 100, 7]
    toks = [m.tokens(n + 12, seed=30 + n) for n in lens]
    want = [m.oracle(t) for t in toks]
    seqs = [r.open() for _ in lens]
    close(r.step([(s, t[:n], [n - 1]) for s, t, n in zip(seqs, toks, lens)]), [w[n - 1] for w, n in zip(want, lens)], f32)
    live = list(range(len(lens)))
    for k in range(12):
        if k in (4, 8):
            r.close(seqs[live.pop(0)])
        got = r.step([(seqs[i], [toks[i][lens[i] + k]], [0]) for i in live])
        close(got, [want[i][lens[i] + k] for i in live], f32)
    for i in live:
        r.close(seqs[i])
    many = [m.tokens(9 + i, seed=60 + i) for i in range(21)]
    want = [m.oracle(t) for t in many]
    seqs = [r.open() for _ in many]
    r.step([(s, t[:-4], []) for s, t in zip(seqs, many)])
    for k in (4, 3):
        got = r.step([(s, [t[-k]], [0]) for s, t in zip(seqs, many)])
        close(got, [w[-k] for w in want], f32)
    got = r.step([(s, t[-2:] if i % 2 else [t[-2]], [0]) for i, (s, t) in enumerate(zip(seqs, many))])
    close(got, [w[-2] for w in want], f32)


def test_rows_of_a_batch_do_not_change_each_other(ca, hdev, models):
    """the same sequence in the same step function: its logits do not move when others are added or leave"""
    m = models("plain")
    r = m.runner(ca, hdev, True)
    t = m.tokens(40, seed=70)
    alone = whole(r, t)
    others = [m.tokens(n, seed=80 + n) for n in (5, 90)]
    seqs = [r.open() for _ in range(3)]
    got = r.step([(seqs[0], others[0], []), (seqs[1], t, list(range(40))), (seqs[2], others[1], [])])
    close(got, alone, True, 0.2)


def test_slabs_are_reused_clean(ca, hdev, models):
    """a sequence opened on a slab that another one has filled starts from nothing: prompt and decode"""
    m = models("loop")
    r = m.runner(ca, hdev, True)
    t = m.tokens(50, seed=90)
    want = m.oracle(t)
    for start in (1, 40):
        for filler in (m.tokens(200, seed=91), m.tokens(3, seed=92)):
            a = r.open()
            r.step([(a, filler, [])])
            r.close(a)
            b = r.open()
            close(r.step([(b, t[:start], [start - 1])]), want[start - 1:start], True)
            close([r.step([(b, [x], [0])])[0] for x in t[start:]], want[start:], True)
            r.close(b)


def test_graph_replays_equal_eager_steps(ca, hdev, models):
    m = models("odd")
    g, e = m.runner(ca, hdev, False), m.runner(ca, hdev, False, use_graph=False)
    t = m.tokens(60, seed=95)
    sg, se = [g.open() for _ in range(3)], [e.open() for _ in range(3)]
    for i, x in enumerate(t):
        n = 3 if i % 4 else 2  # two batch sizes in turn, the program's own eager work (prompt passes) in between
        a = g.step([(s, [x], [0]) for s in sg[:n]])
        b = e.step([(s, [x], [0]) for s in se[:n]])
        assert np.array_equal(a.view(np.uint32), b.view(np.uint32)), i
        if i % 10 == 9:
            assert np.array_equal(whole(g, t[:5]).view(np.uint32), whole(e, t[:5]).view(np.uint32))


def test_long_decoding(ca, hdev, models):
    """hundreds of decoded tokens: the recurrence and many chunks in a row"""
    m = models("odd")
    for f32 in (True, False):
        r = m.runner(ca, hdev, f32, seq_len=600)
        t = m.tokens(500, seed=96)
        want = m.oracle(t)
        s = r.open()
        r.step([(s, t[:2], [])])
        got = [r.step([(s, [x], [0] if i % 7 == 0 or i > 470 else [])]) for i, x in enumerate(t[2:])]
        at = [i + 2 for i in range(498) if len(got[i])]
        close(np.concatenate(got), want[at], f32)


# ---- single mechanisms: one layer, one branch -------------------------------------------------------------------------------------------
def attention_only(chunk, heads=2, kv=1, dim=32, vdim=32, width=128, vocab=40, **kw):
    return sh.config(width, vocab, [sh.layer(heads, kv, dim, vdim, chunk, 1, 8, 8, None, left_scale=1.0, right_scale=0.0, **kw)],
                     embed_scale=8.0, softcap=50.0)


def linear_only(decay, dim=16, vdim=16, width=64, vocab=40):
    return sh.config(width, vocab, [sh.layer(1, 1, 8, 8, 64, len(decay), dim, vdim, None, decay=decay, left_scale=0.0, right_scale=1.0)], softcap=50.0)


def pointed_at(config, seed, key_token, query_token, gain):
    """random weights in which query_token's query (every head) points at key_token's key: that score stands far above all others"""
    bits = sh.random_tensors(config, seed)
    w = {k: sh.from_bf16(v).astype(np.float64) for k, v in bits.items()}
    a = config["layers"][0]["mixer"]["left"]
    unit = lambda v: v / np.sqrt((v * v).mean())
    ek, eq = unit(w["embed"][key_token]), unit(w["embed"][query_token])
    for h in range(a["heads"]):
        g = h // (a["heads"] // a["kv_heads"])
        k = w["l0.mix.left.k"][g * a["dim"]:(g + 1) * a["dim"]] @ ek
        rows = slice(h * a["dim"], (h + 1) * a["dim"])
        w["l0.mix.left.q"][rows] += gain * np.outer(k / np.linalg.norm(k), eq) / len(eq)
    bits["l0.mix.left.q"] = sh.to_bf16(w["l0.mix.left.q"].astype(np.float32))
    bits["l0.mix.left.r1"] = sh.to_bf16(np.full(a["heads"], 0.3, np.float32))
    return bits


@pytest.mark.parametrize("chunk", [16, 37, 64, 100, 256])
def test_one_key_at_every_edge(ca, hdev, tmp_path, chunk):
    """A query that looks for one key, the key moved around: first of the chunk and last of the one before, next to the query, a whole
    chunk away -- seen in a prompt, in a portion, and decoded through the cache.  The oracle itself says that the key's visibility shows:
    with a chunk border that is one token off it gives something else."""
    KEY, QUERY = 38, 39
    c = attention_only(chunk)
    m = Model(c, tmp_path / "m", tensors=pointed_at(c, chunk, KEY, QUERY, 14.0))
    rng = np.random.default_rng(chunk)
    base = [int(x) for x in rng.integers(0, 38, 3 * chunk + 5)]
    cases = [(chunk, 2 * chunk - 1), (chunk - 1, 2 * chunk - 1), (chunk - 1, chunk), (chunk, chunk), (2 * chunk - 1, 2 * chunk - 1), (0, chunk - 1),
             (0, chunk), (chunk, 2 * chunk), (2 * chunk, 2 * chunk + chunk // 2), (2 * chunk - 1, 2 * chunk + 1), (2 * chunk + 1, 3 * chunk + 3),
             (2 * chunk, 3 * chunk - 1), (3 * chunk - 1, 3 * chunk)]
    r = {f: m.runner(ca, hdev, f) for f in (True, False)}
    shows = 0
    for key, query in cases:
        t = list(base)
        t[key] = KEY
        t[query] = QUERY
        t = t[:query + 1]
        want = m.oracle(t)[-1]
        for size in (chunk - 1, chunk + 1):
            off = json.loads(json.dumps(c))
            off["layers"][0]["mixer"]["left"]["mask"]["size"] = size
            if size > 0 and err([m.oracle(t, config=off)[-1]], [want]) > 20 * TOL[True]:
                shows += 1
        for f32 in (True, False):
            s = r[f32].open()
            close(r[f32].step([(s, t, [query])])[0], want, f32)
            r[f32].close(s)
            s = r[f32].open()
            if query > 0:
                r[f32].step([(s, t[:query], [])])
            close(r[f32].step([(s, t[query:], [0])])[0], want, f32)
            r[f32].close(s)
            if query > 3:
                s = r[f32].open()
                r[f32].step([(s, t[:query - 3], [])])
                close(r[f32].step([(s, t[query - 3:], [3])])[0], want, f32)
                r[f32].close(s)
    assert shows >= len(cases)


@pytest.mark.parametrize("heads,kv", [(1, 1), (6, 2), (12, 1), (4, 4)])
def test_grouped_heads(ca, hdev, tmp_path, heads, kv):
    c = attention_only(48, heads=heads, kv=kv, dim=24, vdim=40)
    m = Model(c, tmp_path / "m", seed=heads)
    t = m.tokens(120, seed=3)
    want = m.oracle(t)
    for f32 in (True, False):
        r = m.runner(ca, hdev, f32)
        close(whole(r, t), want, f32)
        s = r.open()
        close([r.step([(s, [x], [0])])[0] for x in t], want, f32)


@pytest.mark.parametrize("what", ["sink", "r1", "r2", "g", "scale"])
def test_parts_of_the_attention_show(ca, hdev, tmp_path, what):
    """sink, distance penalty, gate, score scale: the GPU agrees with the oracle that has them, and not with one that lacks the part"""
    c = attention_only(64, heads=4, kv=2)
    m = Model(c, tmp_path / "m", seed=17)
    bits = sh.random_tensors(c, 17)
    bits["l0.mix.left.sink"] = sh.to_bf16(np.array([3.0, -1.0, 5.0, 0.5], np.float32))
    m = Model(c, tmp_path / "n", tensors=bits)
    t = m.tokens(90, seed=4)
    want = m.oracle(t)
    w, broken = dict(m.tensors), json.loads(json.dumps(c))
    name = "l0.mix.left." + what
    if what == "sink":
        w[name] = np.full(4, -1e4)
    elif what == "scale":
        broken["layers"][0]["mixer"]["left"]["scale"] *= 1.01
    else:
        w[name] = np.zeros_like(w[name])
    wrong = m.oracle(t, config=broken, tensors=w)
    assert err(wrong, want) > 10 * TOL[True]
    r = m.runner(ca, hdev, True)
    close(whole(r, t), want, True)
    s = r.open()
    close([r.step([(s, [x], [0])])[0] for x in t], want, True)


def test_linear_branch_alone_and_far_memory(ca, hdev, tmp_path):
    """decays from forgetful to none at all; a token hundreds of places back still counts, and its absence shows"""
    c = linear_only([0.2, 0.9, 0.999, 1.0])
    m = Model(c, tmp_path / "m", seed=8)
    t = m.tokens(400, seed=9)
    want = m.oracle(t)
    other = list(t)
    other[3] = (t[3] + 1) % 40
    assert err(m.oracle(other)[-1:], want[-1:]) > 20 * TOL[True]
    for f32 in (True, False):
        r = m.runner(ca, hdev, f32)
        close(whole(r, t), want, f32)
        s = r.open()
        r.step([(s, t[:130], [])])
        close([r.step([(s, [x], [0])])[0] for x in t[130:260]], want[130:260], f32)
        close(r.step([(s, t[260:], list(range(140)))]), want[260:], f32)


def test_feed_forward_alone(ca, hdev, tmp_path):
    """both sides of xIELU, with curvatures from small to large"""
    c = sh.config(64, 50, [sh.layer(1, 1, 8, 8, 4, 1, 8, 8, 200, left_scale=0.0, right_scale=0.0)])
    for act in ([-6.0, 3.0], [2.5, -5.0], [0.0, 0.0]):
        bits = sh.random_tensors(c, 3)
        bits["l0.mlp.act"] = sh.to_bf16(np.array(act, np.float32))
        m = Model(c, tmp_path / str(act[0]), tensors=bits)
        t = m.tokens(20, seed=2)
        want = m.oracle(t)
        for f32 in (True, False):
            r = m.runner(ca, hdev, f32)
            close(whole(r, t), want, f32)
            s = r.open()
            close([r.step([(s, [x], [0])])[0] for x in t], want, f32)


def test_positions_far_out(ca, hdev, tmp_path):
    """the position vectors of the embedding thousands of places in"""
    c = sh.config(64, 50, [sh.layer(1, 1, 8, 8, 128, 1, 8, 8, None, decay=[0.5])], embed_scale=0.1)
    m = Model(c, tmp_path / "m", seed=4)
    t = m.tokens(5000, seed=5)
    want = m.oracle(t)
    r = m.runner(ca, hdev, True, seq_len=6000)
    s = r.open()
    at = [0, 1, 2046, 2047, 2048, 2049, 4095, 4096, 4990]
    close(r.step([(s, t[:4991], at)]), want[at], True)
    close([r.step([(s, [x], [0])])[0] for x in t[4991:]], want[4991:], True)


def test_many_wanted_rows_and_none(ca, hdev, models):
    m = models("plain")
    r = m.runner(ca, hdev, True)
    t = m.tokens(600, seed=40)
    want = m.oracle(t)
    close(whole(r, t), want, True)  # several batches of classifier rows
    s = r.open()
    assert len(r.step([(s, t[:300], [])])) == 0
    close(r.step([(s, t[300:], [299])]), want[-1:], True)


# ---- generation ------------------------------------------------------------------------------------------------------------------------
def greedy_oracle(m, prompt, steps):
    t, out, margin = list(prompt), [], np.inf
    for _ in range(steps):
        lg = m.oracle(t)[-1]
        top = np.sort(lg)[-2:]
        margin = min(margin, (top[1] - top[0]) / np.sqrt((lg * lg).mean()))
        out.append(int(len(lg) - 1 - np.argmax(lg[::-1])))
        t.append(out[-1])
    return out, margin


def test_generate_schedules_more_prompts_than_places(ca, hdev, models):
    """the runner's own entry point: 19 prompts of unequal lengths and step counts through 16 places, against the oracle"""
    m = models("plain")
    r = m.runner(ca, hdev, True)
    prompts = [m.tokens(1 + 5 * (i % 7), seed=100 + i) for i in range(19)]
    steps = [1 + i % 9 for i in range(19)]
    steps[4] = 0
    got = r.generate(prompts, steps)
    sure = 0
    for p, n, g in zip(prompts, steps, got):
        want, margin = greedy_oracle(m, p, n)
        assert len(g) == n
        if margin > 1e-3:
            sure += 1
            assert g == want
    assert sure >= 15
    assert r.generate(prompts[:3], steps[:3]) == got[:3]


def test_single_sequence_entry_points(ca, hdev, models):
    """ModelRunner: prefill / forward / decode_greedy / reset, and the device-sampled tokens against the host's choice"""
    m = models("loop")
    r = m.runner(ca, hdev, True)
    assert isinstance(r, ca.ModelRunner) and r.architecture == "Nilivik" and r.vocab_size == m.config["vocab"]
    p = m.tokens(45, seed=50)
    lg = r.prefill(p)
    close(lg, m.oracle(p)[-1], True)
    first = ca.sample_argmax(lg)
    ids = r.decode_greedy(first, 30)
    assert r.kv_cache_len() == 75
    r.reset()
    assert r.kv_cache_len() == 0
    lg, t = r.prefill(p), first
    for i in range(30):
        t = ca.sample_argmax(r.forward(t, 45 + i))
        assert t == ids[i]
    with pytest.raises(ca.CrabmlError):
        r.forward(1, 3)


def test_errors_leave_the_runner_usable(ca, hdev, models):
    m = models("plain")
    r = m.runner(ca, hdev, True, seq_len=64)
    s = r.open()
    for bad in ([(s + 5, [1], [])], [(s, [], [])], [(s, [m.config["vocab"]], [])], [(s, [1], [1])], [(s, [1, 2], [1, 0])], [(s, [1] * 65, [])],
                [(s, [1], []), (s, [2], [])]):
        with pytest.raises(ca.CrabmlError):
            r.step(bad)
    assert r.length(s) == 0
    t = m.tokens(64, seed=11)
    close(r.step([(s, t, [63])]), m.oracle(t)[-1:], True)
    with pytest.raises(ca.CrabmlError):
        r.step([(s, [1], [0])])
    r.close(s)
    with pytest.raises(ca.CrabmlError):
        r.close(s)


def test_command_lines(ca, models, tmp_path):
    """bin/trace_run and tools/generate.py as processes of their own"""
    m = models("plain")
    t = m.tokens(30, seed=12)
    u = m.tokens(12, seed=13)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:29], "want": [0, 28]}, {"id": "b", "tokens": u[:11], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t[29:], "want": [0]}, {"id": "b", "tokens": u[11:], "want": [0]}], "end": ["a", "b"]}]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", m.folder, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "42"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert p.stdout.split() == ["done", "0", "done", "1"]
    a, b = m.oracle(t), m.oracle(u)
    v = m.config["vocab"]
    close(np.fromfile(tmp_path / "0.f32", "<f4").reshape(-1, v), a[[0, 28]], True)
    close(np.fromfile(tmp_path / "1.f32", "<f4").reshape(-1, v), [a[29], b[11]], True)
    p = subprocess.run([sys.executable, os.path.join(ROOT, "tools", "generate.py"), m.folder, "--prompt", ",".join(map(str, t)), "--steps", "4", "--f32"],
                       capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    want, margin = greedy_oracle(m, t, 4)
    if margin > 1e-3:
        assert "tokens: " + ",".join(map(str, want)) in p.stdout


# ---- bfloat16 as a weight format of the Tensor path ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("m,k", [(1, 8), (3, 100), (70, 256), (513, 2056), (2050, 640)])
def test_matmul_vec_bf16(ca, hdev, m, k):
    rng = np.random.default_rng(m)
    bits = sh.to_bf16(rng.standard_normal((m, k)).astype(np.float32))
    w = sh.from_bf16(bits).astype(np.float64)
    t = ca.HipTensor.from_cpu(bits.view(np.uint8).reshape(-1), [m, k], ca.GGMLType.BF16, hdev)
    for b in (1, 2, 3, 8, 17):
        x = rng.standard_normal((b, k)).astype(np.float32)
        got = t.matmul_vec(ca.HipTensor.new(x.reshape(-1), [b, k], hdev)).export().reshape(b, m)
        want = x.astype(np.float64) @ w.T
        bound = 2e-6 * (np.abs(x).astype(np.float64) @ np.abs(w).T)
        assert (np.abs(got - want) <= bound).all()
    row = ca.HipTensor.alloc([k], ca.GGMLType.F32, hdev)
    row.copy_rows_from(t, [m - 1])
    assert np.array_equal(row.export(), sh.from_bf16(bits[m - 1]))
