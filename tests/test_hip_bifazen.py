"""The Bifazen design on the hybrid decoder, on the GPU against the plain implementation of tests/bifazen_oracle.py: small models with
random weights, float32 compute for sharp comparisons (differences of rounding size only) and bfloat16 compute for the serving path."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from crabml_amd import synth_bifazen as sb
from crabml_amd import synth_hybrid as sh
from tests import bifazen_oracle as bo

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# root mean square of the logits' difference over that of the logits
TOL = {True: 2e-5, False: 2.5e-2}


class Model:
    def __init__(self, config, folder, seed=0, tensors=None):
        self.config = config
        bits = tensors if tensors is not None else sb.random_tensors(config, seed)
        self.tensors = {k: sh.from_bf16(v) for k, v in bits.items()}
        self.folder = sh.write_model(config, bits, str(folder))

    def oracle(self, tokens, config=None, tensors=None):
        return bo.forward(config or self.config, tensors or self.tensors, tokens)

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


def decoded(r, tokens, start=0):
    """logits of tokens[start:], one by one"""
    s = r.open()
    if start:
        r.step([(s, tokens[:start], [])])
    got = [r.step([(s, [x], [0])])[0] for x in tokens[start:]]
    r.close(s)
    return got


# sizes on purpose unlike one another, unaligned, equal or 1
CONFIGS = {
    "plain": sb.config(128, 300, [sb.latent(4, 32, 16, 32, 64, 40, 96), sb.attention(4, 2, 32, 32, 24, 96), sb.latent(4, 32, 16, 32, 64, 40, 96),
                                  sb.attention(4, 2, 32, 32, 24, 96)], streams=4),
    "odd": sb.config(84, 131, [sb.attention(6, 3, 20, 10, 50, 75, v_mix=False), sb.latent(5, 20, 6, 12, 37, 7, None, base=500.0),
                               sb.attention(3, 3, 36, 10, 9, None), sb.latent(3, 12, 2, 44, 100, 33, 50, base=31.0), sb.attention(12, 3, 8, 10, 1, 23)],
                     streams=3, eps=1e-3),
    "ones": sb.config(40, 30, [sb.latent(1, 8, 2, 8, 8, 1, 1), sb.attention(1, 1, 1, 1, 2, 8), sb.attention(1, 1, 2, 1, 1000, 8)], streams=1),
    "latent-only": sb.config(96, 90, [sb.latent(20, 16, 8, 24, 40, 70, 64), sb.latent(2, 64, 64, 64, 128, 12, 64)], streams=2),
    "attention-only": sb.config(64, 64, [sb.attention(2, 1, 16, 16, 17, 32), sb.attention(2, 1, 24, 16, 30, 32)], streams=2),
    "wide": sb.config(160, 200, [sb.latent(3, 128, 64, 128, 300, 90, 200), sb.attention(18, 2, 136, 100, 100, 64), sb.latent(2, 200, 40, 136, 520, 33, 64),
                                 sb.attention(36, 2, 40, 100, 64, None)], streams=8),
}


# ("ones" in bfloat16: an RMS norm over one number is its sign, which rounding decides where the number is small)
CASES = [(n, f32) for n in sorted(CONFIGS) for f32 in (True, False) if f32 or n != "ones"]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    base = tmp_path_factory.mktemp("bifazen")
    cache = {}

    def get(name):
        if name not in cache:
            cache[name] = Model(CONFIGS[name], base / name, seed=len(name))
        return cache[name]
    return get


# ---- whole models --------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name,f32", CASES)
def test_whole_prompt_every_position(ca, hdev, models, name, f32):
    m = models(name)
    r = m.runner(ca, hdev, f32)
    for n in (1, 2, 3, 65, 150):
        t = m.tokens(n, seed=n)
        close(whole(r, t), m.oracle(t), f32)


@pytest.mark.parametrize("name,f32", CASES)
def test_prompt_then_token_by_token(ca, hdev, models, name, f32):
    """every logit of the decode step, from the first token on and behind a prompt, with windows that fill, and that have gone round"""
    m = models(name)
    r = m.runner(ca, hdev, f32)
    t = m.tokens(125, seed=5)
    want = m.oracle(t)
    close(decoded(r, t), want, f32)
    close(decoded(r, t, 70), want[70:], f32)


@pytest.mark.parametrize("name", ["odd", "plain", "wide", "ones"])
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


@pytest.mark.parametrize("f32", [True, False])
def test_internal_passes_cut_prompts_too(ca, hdev, models, f32):
    """pass_rows far below the batch: entries are split over passes, some passes hold the end of one and the start of another"""
    m = models("odd")
    r = m.runner(ca, hdev, f32, pass_rows=50)
    lens = [70, 1, 33, 121, 2]
    prompts = [m.tokens(n, seed=20 + n) for n in lens]
    seqs = [r.open() for _ in lens]
    got = r.step([(s, p, list(range(len(p)))) for s, p in zip(seqs, prompts)])
    close(got, np.concatenate([m.oracle(p) for p in prompts]), f32)


def test_many_portions_whose_earlier_rows_exceed_a_pass(ca, hdev, tmp_path):
    """sequences that all go on by two tokens: the earlier rows they read again (a window's worth each) are cut into passes too"""
    c = sb.config(48, 60, [sb.latent(2, 16, 8, 16, 24, 200, 32), sb.attention(2, 1, 16, 16, 150, 32)], streams=2)
    m = Model(c, tmp_path / "m", seed=2)
    r = m.runner(ca, hdev, True, pass_rows=256)
    toks = [m.tokens(150 + 23 * i, seed=200 + i) for i in range(9)]
    want = [m.oracle(t) for t in toks]
    seqs = [r.open() for _ in toks]
    r.step([(s, t[:-4], []) for s, t in zip(seqs, toks)])
    got = r.step([(s, t[-4:-2], [0, 1]) for s, t in zip(seqs, toks)])
    close(got, np.concatenate([w[-4:-2] for w in want]), True)
    got = r.step([(s, t[-2:-1], [0]) for s, t in zip(seqs, toks)])
    close(got, [w[-2] for w in want], True)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("name", ["plain", "odd"])
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
    many = [m.tokens(9 + 3 * i, seed=60 + i) for i in range(21)]
    want = [m.oracle(t) for t in many]
    seqs = [r.open() for _ in many]
    r.step([(s, t[:-4], []) for s, t in zip(seqs, many)])
    for k in (4, 3):
        got = r.step([(s, [t[-k]], [0]) for s, t in zip(seqs, many)])
        close(got, [w[-k] for w in want], f32)
    got = r.step([(s, t[-2:] if i % 2 else [t[-2]], [0]) for i, (s, t) in enumerate(zip(seqs, many))])
    close(got, [w[-2] for w in want], f32)


@pytest.mark.parametrize("f32", [True, False])
def test_many_heads_times_many_sequences(ca, hdev, tmp_path, f32):
    """enough (head, sequence) pairs to fill the chip: the decode attention of latents then runs in fewer, longer pieces"""
    c = sb.config(48, 60, [sb.latent(36, 16, 8, 24, 72, 400, 32)], streams=2)
    m = Model(c, tmp_path / "m", seed=2)
    r = m.runner(ca, hdev, f32)
    toks = [m.tokens(20 + 41 * i, seed=300 + i) for i in range(15)]
    want = [m.oracle(t) for t in toks]
    seqs = [r.open() for _ in toks]
    r.step([(s, t[:-3], []) for s, t in zip(seqs, toks)])
    for k in (3, 2, 1):
        close(r.step([(s, [t[-k]], [0]) for s, t in zip(seqs, toks)]), [w[-k] for w in want], f32)


def test_rows_of_a_batch_do_not_change_each_other(ca, hdev, models):
    m = models("plain")
    r = m.runner(ca, hdev, True)
    t = m.tokens(60, seed=70)
    alone = whole(r, t)
    others = [m.tokens(n, seed=80 + n) for n in (5, 90)]
    seqs = [r.open() for _ in range(3)]
    got = r.step([(seqs[0], others[0], []), (seqs[1], t, list(range(60))), (seqs[2], others[1], [])])
    close(got, alone, True, 0.2)


def test_slabs_are_reused_clean(ca, hdev, models):
    """a sequence opened on a slab that another one has filled starts from nothing: prompt and decode"""
    m = models("plain")
    r = m.runner(ca, hdev, True)
    t = m.tokens(60, seed=90)
    want = m.oracle(t)
    for start in (1, 45):
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


@pytest.mark.parametrize("window,n,start", [(23, 500, 2), (700, 1100, 640), (1500, 1700, 1480)])
def test_long_decoding(ca, hdev, tmp_path, window, n, start):
    """hundreds of decoded tokens: windows that go round many times; windows of so many rows that a workgroup takes several tiles of them"""
    c = sb.config(48, 70, [sb.latent(2, 16, 8, 16, 24, window, 32), sb.attention(2, 1, 16, 16, window, 32)], streams=2)
    m = Model(c, tmp_path / "m", seed=3)
    t = m.tokens(n, seed=96)
    want = m.oracle(t)
    for f32 in (True, False):
        r = m.runner(ca, hdev, f32, seq_len=n + 10)
        s = r.open()
        r.step([(s, t[:start], [])])
        got = [r.step([(s, [x], [0] if i % 7 == 0 or i > n - start - 30 else [])]) for i, x in enumerate(t[start:])]
        at = [i + start for i in range(n - start) if len(got[i])]
        close(np.concatenate(got), want[at], f32)


# ---- single mechanisms -----------------------------------------------------------------------------------------------------------------
def pointed_at(config, seed, key_token, query_token):
    """random weights of a one-layer model in which query_token's query (every head) points at key_token's key"""
    bits = sb.random_tensors(config, seed)
    for t in ("in", "out", "mix"):
        bits["l0.hc1." + t] = sh.to_bf16(np.ones_like(bits["l0.hc1." + t], np.float32))
    w = {k: sh.from_bf16(v).astype(np.float64) for k, v in bits.items()}
    m, lat = config["layers"][0]["mixer"], config["layers"][0]["type"] == "latent_attention"
    eps = config["norm"]["eps"]
    hk, hq = (bo.rms_norm(w["embed"][x], 1 + w["l0.norm1"], eps) for x in (key_token, query_token))
    rot = m["rot_dim"] if lat else 0
    if lat:
        c = bo.rms_norm((w["l0.mix.dkv"] @ hk)[:m["kv_rank"]], w["l0.mix.dkv.norm"], eps)
        keys = (w["l0.mix.uk"] @ c).reshape(m["heads"], m["dim"])
    else:
        k = bo.rms_norm(w["l0.mix.k"] @ hk + w["l0.mix.k.b"], w["l0.mix.k.norm"], eps).reshape(m["kv_heads"], m["dim"])
        keys = np.repeat(k, m["heads"] // m["kv_heads"], axis=0)
    for h in range(m["heads"]):
        rows = slice(h * (m["dim"] + rot), h * (m["dim"] + rot) + m["dim"])
        w["l0.mix.q"][rows] += 4 * np.sqrt(m["dim"]) * np.outer(keys[h] / np.linalg.norm(keys[h]), hq) / (hq @ hq)
    bits["l0.mix.q"] = sh.to_bf16(w["l0.mix.q"].astype(np.float32))
    return bits


@pytest.mark.parametrize("window", [1, 2, 16, 37, 64, 100, 256])
@pytest.mark.parametrize("kind", ["latent", "attention"])
def test_one_key_at_every_edge(ca, hdev, tmp_path, kind, window):
    """A query that looks for one key, the key moved around: just inside the window and just outside, next to the query, at the cache's
    wrap, first of the sequence -- seen in a prompt, in a portion, and decoded through the cache.  The oracle itself says that the key's
    visibility shows: with a window that is one token off it gives something else."""
    KEY, QUERY = 38, 39
    layer = sb.latent(2, 32, 8, 32, 48, window, None, scale=0.6) if kind == "latent" else sb.attention(2, 1, 32, 32, window, None, scale=0.6)
    c = sb.config(128, 40, [layer], streams=1)
    m = Model(c, tmp_path / "m", tensors=pointed_at(c, window, KEY, QUERY))
    base = [int(x) for x in np.random.default_rng(window).integers(0, 38, 3 * window + 8)]
    at = sorted({window, 2 * window - 1, 2 * window, 3 * window + 2})
    r = {f: m.runner(ca, hdev, f) for f in (True, False)}
    shows, edges = 0, 0
    for query in at:
        for back in sorted({window - 1, window, window + 1, 1, window // 2}):
            key = query - back
            if key < 0 or back == 0:
                continue
            t = list(base)
            t[key] = KEY
            t[query] = QUERY
            t = t[:query + 1]
            want = m.oracle(t)[-1]
            if back in (window - 1, window):
                edges += 1
                off = json.loads(json.dumps(c))
                off["layers"][0]["mixer"]["mask"]["size"] = window + (1 if back == window else -1)
                shows += err([m.oracle(t, config=off)[-1]], [want]) > 20 * TOL[True]
            for f32 in (True, False):
                s = r[f32].open()
                close(r[f32].step([(s, t, [query])])[0], want, f32)
                r[f32].close(s)
                s = r[f32].open()
                r[f32].step([(s, t[:query], [])])
                close(r[f32].step([(s, t[query:], [0])])[0], want, f32)
                r[f32].close(s)
                if query > 3:
                    s = r[f32].open()
                    r[f32].step([(s, t[:query - 3], [])])
                    close(r[f32].step([(s, t[query - 3:], [3])])[0], want, f32)
                    r[f32].close(s)
    assert edges and shows == edges


PARTS = ["l0.mix.q.b", "l0.mix.k.b", "l0.mix.v.b", "l0.mix.o.b", "l0.mix.q.norm", "l0.mix.k.norm", "l0.mix.g", "l0.norm1", "l0.norm2", "l0.hc1.in", "l0.hc1.out",
         "l0.hc1.mix", "l0.hc2.in", "l0.hc2.out", "l0.hc2.mix", "l0.mlp.gate", "l0.mlp.up", "l1.mix.dkv.norm", "l1.mix.uk", "l1.mix.uv", "l1.hc1.mix", "l2.mix.vmix",
         "l2.mix.k.b", "final.norm"]


def test_every_part_shows(ca, hdev, tmp_path):
    """the GPU agrees with the oracle that has every part, and each part makes a difference far above the tolerance: without it, and the
    mixing matrix read the other way round, the first layer's unused mixing factor used, scales, bases, eps and streams changed"""
    c = sb.config(64, 80, [sb.attention(4, 2, 16, 16, 30, 48), sb.latent(4, 16, 8, 16, 24, 25, 48), sb.attention(4, 2, 16, 16, 12, 48), sb.attention(4, 2, 16, 16, 40, None)],
                  streams=3, eps=1e-3)
    m = Model(c, tmp_path / "m", seed=17)
    t = m.tokens(90, seed=4)
    want = m.oracle(t)
    wrong = {}
    for p in PARTS:
        w = dict(m.tensors)
        w[p] = np.ones_like(w[p]) if p.endswith((".q.norm", ".k.norm", ".dkv.norm", "hc1.in", "hc1.out", "hc2.in", "hc2.out")) else np.zeros_like(w[p])
        wrong[p] = m.oracle(t, tensors=w)
    for q in ("hc1", "hc2"):
        w = dict(m.tensors)
        w["l0.%s.mix" % q] = w["l0.%s.mix" % q].T
        wrong[q + " transposed"] = m.oracle(t, tensors=w)

    def changed(name, *path, by):
        off = json.loads(json.dumps(c))
        at = off
        for p in path[:-1]:
            at = at[p]
        at[path[-1]] = by(at[path[-1]])
        wrong[name] = m.oracle(t, config=off)
    changed("eps", "norm", "eps", by=lambda x: x / 10)
    changed("scale", "layers", 0, "mixer", "scale", by=lambda x: x * 1.01)
    changed("latent scale", "layers", 1, "mixer", "scale", by=lambda x: x * 1.01)
    changed("base", "layers", 1, "mixer", "rot", "base", by=lambda x: x * 1.1)
    changed("mixing switched off", "layers", 2, "mixer", "v_mix", by=lambda x: False)
    changed("mixing from the second layer on", "layers", 0, "mixer", "v_mix", by=lambda x: False)
    for name, lg in wrong.items():
        assert err(lg, want) > 10 * TOL[True], name
    unused = dict(m.tensors)
    unused["l0.mix.vmix"] = np.float32(0.9)
    assert np.array_equal(m.oracle(t, tensors=unused), want)
    for f32 in (True, False):
        r = m.runner(ca, hdev, f32)
        close(whole(r, t), want, f32)
        close(decoded(r, t), want, f32)


@pytest.mark.parametrize("heads,kv", [(1, 1), (6, 2), (12, 1), (4, 4), (34, 2)])
def test_grouped_heads(ca, hdev, tmp_path, heads, kv):
    c = sb.config(128, 40, [sb.attention(heads, kv, 24, 40, 48, None), sb.latent(heads, 24, 8, 40, 56, 48, None)], streams=2)
    m = Model(c, tmp_path / "m", seed=heads)
    t = m.tokens(120, seed=3)
    want = m.oracle(t)
    for f32 in (True, False):
        r = m.runner(ca, hdev, f32)
        close(whole(r, t), want, f32)
        close(decoded(r, t), want, f32)


def test_rotation_far_out(ca, hdev, tmp_path):
    """thousands of places in, where an angle that was formed carelessly has lost its digits; prompts longer than a pass"""
    c = sb.config(64, 50, [sb.latent(2, 8, 32, 32, 32, 60, None, base=50.0)], streams=1)
    m = Model(c, tmp_path / "m", seed=4)
    t = m.tokens(5000, seed=5)
    want = m.oracle(t)
    r = m.runner(ca, hdev, True, seq_len=6000)
    s = r.open()
    at = [0, 1, 2046, 2047, 2048, 2049, 2107, 2108, 4095, 4096, 4990]
    close(r.step([(s, t[:4991], at)]), want[at], True)
    close([r.step([(s, [x], [0])])[0] for x in t[4991:]], want[4991:], True)


def test_a_far_key_among_hundreds(ca, hdev, tmp_path):
    """one early token in a wide window decides; replaced, the logits move"""
    KEY, QUERY = 38, 39
    for layer in (sb.latent(2, 32, 8, 32, 48, 900, None, scale=0.6), sb.attention(2, 1, 32, 32, 900, None, scale=0.6)):
        c = sb.config(128, 40, [layer], streams=1)
        m = Model(c, tmp_path / layer["type"], tensors=pointed_at(c, 5, KEY, QUERY))
        t = [int(x) for x in np.random.default_rng(6).integers(0, 38, 801)]
        t[3], t[800] = KEY, QUERY
        want = m.oracle(t)[-1]
        other = list(t)
        other[3] = 7
        assert err([m.oracle(other)[-1]], [want]) > 20 * TOL[True]
        for f32 in (True, False):
            r = m.runner(ca, hdev, f32)
            close(whole(r, t)[-1], want, f32)
            close(decoded(r, t, 800)[0], want, f32)


def test_more_wanted_rows_than_a_batch_of_them_and_none(ca, hdev, models):
    m = models("plain")
    r = m.runner(ca, hdev, True)
    t = m.tokens(600, seed=40)
    want = m.oracle(t)
    close(whole(r, t), want, True)
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
    prompts = [m.tokens(1 + 7 * (i % 7), seed=100 + i) for i in range(19)]
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
    m = models("plain")
    r = m.runner(ca, hdev, True)
    assert isinstance(r, ca.ModelRunner) and r.architecture == "Bifazen" and r.vocab_size == m.config["vocab"]
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


def test_command_lines(ca, models, tmp_path):
    """bin/trace_run and tools/generate.py as processes of their own"""
    m = models("odd")
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
    p = subprocess.run([sys.executable, os.path.join(ROOT, "tools", "generate.py"), m.folder, "--prompt", ",".join(map(str, t)), "--prompt", ",".join(map(str, u)),
                        "--steps", "4", "--f32"], capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    for prompt in (t, u):
        want, margin = greedy_oracle(m, prompt, 4)
        if margin > 1e-3:
            assert "tokens: " + ",".join(map(str, want)) in p.stdout
