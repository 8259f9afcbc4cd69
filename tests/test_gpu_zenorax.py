"""Zenorax on the device against the float64 oracle: every mechanism alone over sizes, prompts against token-by-token decoding,
portions, mixed batches, reused pages and slots, keys far away and at page borders, lost states, long decoding, generation through the
scheduler."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from helpers import layered_build as B
from helpers import layered_ref as R
from helpers.device import ROOT, dev
from helpers.layered_model import Model, check, err, feed, greedy, margin

pytestmark = pytest.mark.gpu
DT = pytest.mark.parametrize("dt", ["f32", "bf16"])


@pytest.fixture(scope="module")
def cai():
    return dev()


MIXED = dict(layers=[B.zlayer(B.forget(heads=3, dim=20, vdim=28), B.zmoe(experts=9, top=4, ff=17, count=3, keep=2)),
                     B.zlayer(B.lat(heads=6, dim=20, rot_dim=12, vdim=44, kv_rank=52, q_rank=30), B.zmoe(experts=6, top=2, ff=40, count=6, keep=4)),
                     B.zlayer(B.keyval(heads=6, kv_heads=2, dim=28, rot=10), B.zmoe(experts=5, top=5, ff=33, count=1, keep=1)),
                     B.zlayer(B.lat(heads=1, dim=33, rot_dim=7, rot=6, vdim=9, kv_rank=17, q_rank=21, yarn=None)),
                     B.zlayer(B.forget(heads=1, dim=33, vdim=9)),
                     B.zlayer(B.keyval(heads=3, kv_heads=3, dim=9, rot=0, factor=None), B.zmoe())], width=100, vocab=211, taps=4)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """bf16: the choice of experts is decided by far, so that the oracle and 16-bit activations cannot part there"""
    cfg = B.zconfig(**MIXED)
    return {dt: Model(tmp_path_factory.mktemp("zenorax"), cfg, seed=21, edit=B.steady_groups if dt == "bf16" else None) for dt in ("f32", "bf16")}


# ---------------------------------------------------------------- each mechanism alone
LAT = [B.lat(*a, yarn=y) for a, y in (
    ((1, 8, 8, 8, 8, 8, 0.4), None), ((4, 24, 8, 40, 64, 48, 0.2, 4), (2.0, 300, 16.0, 2.0)), ((6, 64, 32, 64, 128, 96, 0.1), (8.0, 1000, 32.0, 1.0)), ((8, 130, 66, 70, 200, 130, 0.07), (1.0, 64, 4.0, 1.0)),
    ((10, 128, 64, 128, 512, 300, 0.07), (4.0, 2000, 32.0, 1.0)), ((3, 18, 10, 9, 20, 7, 0.3, 0), None), ((5, 200, 56, 256, 130, 64, 0.06), (16.0, 100, 2.0, 0.5)), ((9, 31, 2, 33, 67, 65, 0.25), (0.5, 500, 30.0, 3.0)),
    ((2, 250, 20, 300, 40, 50, 0.1), None))]
KEYVAL = [B.keyval(*a) for a in ((1, 1, 8, 0.5, 8), (4, 4, 24, 0.3, 24, 50.0, 1.0), (6, 2, 48, 0.2, 20), (8, 1, 130, 0.1, 64), (10, 2, 256, 0.06, 256, 1e4, 8.0), (2, 1, 64, 0.2, 2, 300.0, 0.5), (3, 1, 18, 0.4, 0), (15, 3, 72, 0.15, 36))]
FORGET = [B.forget(*a) for a in ((1, 8, 8), (4, 24, 40), (3, 48, 96), (8, 130, 70), (2, 256, 256), (5, 18, 9), (16, 64, 20), (2, 3, 130), (7, 65, 33))]
MOE = [B.zmoe(*a) for a in ((4, 1, 16, 2, 1), (8, 8, 33, 4, 4), (36, 5, 20, 4, 2), (130, 6, 9, 13, 3), (512, 3, 5, 64, 2), (66, 64, 3, 1, 1), (16, 2, 70, 16, 5), (64, 4, 24, 8, 1), (256, 8, 4, 8, 4))]


@DT
@pytest.mark.parametrize("i", range(len(LAT)))
def test_latent_attention_alone(cai, tmp_path, i, dt):
    m = Model(tmp_path, B.zconfig([B.zlayer(LAT[i])], width=40 + 8 * i, vocab=67, eps=10.0 ** -(2 + i % 5), scale=0.5 + i), seed=i)
    tok = m.tokens(150, i)
    dec = m.open(cai, 192, 1, dt)
    for cuts in ([150], [100, 1], [64, 65, 2, 1], [9, 40, 31, 32, 33, 3]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("i", range(len(KEYVAL)))
def test_keys_as_values_alone(cai, tmp_path, i, dt):
    m = Model(tmp_path, B.zconfig([B.zlayer(KEYVAL[i])], width=42 + 9 * i, vocab=67, eps=10.0 ** -(2 + i % 5), cap=4.0 + i), seed=i)
    tok = m.tokens(150, i)
    dec = m.open(cai, 192, 1, dt)
    for cuts in ([150], [100, 1], [64, 65, 2, 1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("gates", ["mixed", "strong", "weak"])
@pytest.mark.parametrize("i", range(len(FORGET)))
def test_forget_gates_alone(cai, tmp_path, i, gates, dt):
    """strong: gates near and at zero within a chunk, sums of them far below the smallest float; weak: a state that hardly forgets"""
    def edit(w):
        if gates == "strong":
            w["l0.mix.f.b"] -= np.linspace(0, 90, len(w["l0.mix.f.b"])); w["l0.mix.lower"][::2] = 0
        if gates == "weak":
            w["l0.mix.f.b"] += 7.0; w["l0.mix.lower"][::3] = 0.996
    m = Model(tmp_path, B.zconfig([B.zlayer(FORGET[i])], width=40 + 9 * i, vocab=67, eps=10.0 ** -(3 + i % 4)), seed=50 + i, edit=edit)
    tok = m.tokens(140, i)
    dec = m.open(cai, 64, 2, dt)
    for cuts in ([140], [100, 1], [16, 17, 15, 2, 1], [3, 30, 31]):
        dec.reset(1)
        check(feed(dec, tok, cuts, 1), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("i", range(len(MOE)))
def test_experts_alone(cai, tmp_path, i, dt):
    """one layer whose mixer adds nothing, so that every token stands alone; tokens whose choice of experts or groups is close are left out"""
    def edit(w):
        w["l0.norm1b"] *= 0
        if i % 2:
            w["l0.mlp.correction"] -= 2.0              # negative choice scores
    m = Model(tmp_path, B.zconfig([B.zlayer(B.forget(1, 8, 8), MOE[i])], width=56 + 12 * i, vocab=400, scale=2.0), seed=30 + i, edit=edit)
    r, w = MOE[i]["router"], m.w
    x = w["embed"] * 2.0
    z = R.linear(w["l0.mlp.router"], R.rms_norm(x, 1e-5) * w["l0.norm2"])
    c = R.sigmoid(z) + w["l0.mlp.correction"]
    n, count, keep = r["experts"], r["groups"]["count"], r["groups"]["keep"]
    g = c.reshape(400, count, n // count)
    score = np.sort(np.sort(g, axis=2)[:, :, -2:].sum(2), axis=1)[:, ::-1]
    lead = np.full(400, np.inf)
    if keep < count:
        lead = np.minimum(lead, score[:, keep - 1] - score[:, keep])
    for t in range(400):
        best = np.argsort(-np.sort(g[t], axis=1)[:, -2:].sum(1), kind="stable")[:keep]
        s = np.sort(g[t][best].reshape(-1))[::-1]
        if r["top"] < len(s):
            lead[t] = min(lead[t], s[r["top"] - 1] - s[r["top"]])
    clear = np.nonzero(lead > (1e-5 if dt == "f32" else 8e-3))[0]
    assert len(clear) > 8
    tok = np.random.default_rng(i).choice(clear, 90).tolist()
    dec = m.open(cai, 128, 1, dt)
    for cuts in ([90], [9, 8, 3, 1], [5, 2, 30]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("what", ["sink", "convolution", "depth", "lower bound", "correction", "eps", "soft cap", "turned part", "gate"])
def test_one_mechanism_made_strong(cai, tmp_path, what, dt):
    """the others neutral, this one large enough to carry the result: leaving it out in the oracle moves the logits far"""
    cfg = B.zconfig([B.zlayer(B.keyval()), B.zlayer(B.forget(), B.zmoe()), B.zlayer(B.lat())], width=64, vocab=90, cap=2.0 if what == "soft cap" else 1e4, eps=0.5 if what == "eps" else 1e-6)

    def neutral(w, keep=None):
        for n in w:
            if n.endswith("canon1") and keep != "convolution" or n.endswith("lower") and keep != "lower bound" or n.endswith("correction") and keep != "correction":
                w[n] = w[n] * 0
            if n.endswith("dwa") and keep != "depth":
                w[n] = np.eye(len(w[n]))[-1]
            if n.endswith("sink") and keep != "sink":
                w[n] = w[n] * 0 - 30.0
            if n.endswith(".g") and keep != "gate":
                w[n] = w[n] * 0
            if n.endswith("dkv") and keep != "turned part":
                w[n] = w[n].copy(); w[n][36:] = 0

    def edit(w):
        B.steady_groups(w) if what != "correction" else None
        neutral(w, None if what == "correction" else what)
        if what == "sink":
            w["l0.mix.sink"] = np.array([9.0, 2.0, -1.0, 14.0])
        if what == "convolution":
            for i in range(3):
                w["l%d.canon1" % i][:, 0] += 2.0
        if what == "depth":
            w["l1.dwa"] = np.array([1.5, -0.7, 0.5]); w["l2.dwa"] = np.array([-0.5, 1.0, 0.6, 0.9])
        if what == "turned part":
            w["l2.mix.dkv"][36:] *= 3
        if what == "gate":
            w["l2.mix.g"] *= 5
        if what == "correction":
            w["l1.mlp.correction"] = np.array([0, 9.0, 3.0, -4.0, 0, 0, 8.0, 7.0])
        else:
            w["l1.mlp.router"] *= 0                    # one choice for all
    m = Model(tmp_path, cfg, seed=9, edit=edit)
    tok = m.tokens(140, 4)
    plain = dict(m.w)
    neutral(plain)
    bare = json.loads(json.dumps(cfg)); bare["norm"]["eps"] = 1e-6; bare["logit_softcap"] = 1e4
    assert err(R.forward(bare, plain, np.array(tok)), m.ref(tok)) > 0.15
    dec = m.open(cai, 192, 1, dt)
    for cuts in ([140], [90, 1], [1], [3, 2, 40]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 9])
@pytest.mark.parametrize("width", [60, 97])
def test_input_convolution_of_any_length(cai, tmp_path, taps, width, dt):
    """portions shorter than the convolution looks back, two sequences whose rings alternate"""
    m = Model(tmp_path, B.zconfig([B.zlayer(B.keyval()), B.zlayer(B.forget())], width=width, vocab=90, taps=taps), seed=taps)
    a, b = m.tokens(60, 2), m.tokens(60, 3)
    dec = m.open(cai, 128, 2, dt)
    for cuts in ([60], [2], [1], [3, 1, 2, 20], [11, 4]):
        dec.reset(0); dec.reset(1)
        check(feed(dec, a, cuts, 0), m.ref(a), dt)
        check(feed(dec, b, cuts, 1), m.ref(b), dt)
    dec.reset(0); dec.reset(1)
    got, at = [[], []], [0, 0]
    while at[0] < 60:
        n = [min(k, 60 - i) for k, i in zip((1 + at[0] % 3, 1 + (at[0] + 1) % 2), at)]
        entries = [(s, (a, b)[s][at[s]:at[s] + n[s]], range(n[s])) for s in (1, 0) if n[s]]
        lg = dec.step_batch(entries)[1]
        for s, t, w in entries:
            got[s].append(lg[:len(t)]); lg = lg[len(t):]; at[s] += len(t)
    check(np.concatenate(got[0]), m.ref(a), dt); check(np.concatenate(got[1]), m.ref(b)[:at[1]], dt)
    dec.close()


# ---------------------------------------------------------------- whole models
@DT
@pytest.mark.parametrize("cuts", [[300], [1], [2], [3, 2, 65, 1, 1, 16, 17, 2], [64], [130, 1], [5, 9, 7], [31, 33, 32]], ids=str)
def test_portions_and_decoding_agree_with_the_whole(cai, models, cuts, dt):
    m = models[dt]
    tok = m.tokens(150, 3)
    dec = m.open(cai, 192, 1, dt)
    check(feed(dec, tok, cuts), m.ref(tok), dt)
    assert dec.len() == 150 and dec.cache_rows() == 150
    dec.close()


@DT
def test_first_tokens(cai, models, dt):
    m = models[dt]
    dec = m.open(cai, 64, 1, dt)
    for n in range(1, 8):
        tok = m.tokens(n, 40 + n)
        for cuts in ([n], [1], [2]):
            dec.reset()
            check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
def test_mixed_batches_with_reused_slots_and_pages(cai, models, dt):
    """eight requests over three slots; portions of some beside single tokens of others; a pool that the live ones nearly fill"""
    m = models[dt]
    rng = np.random.default_rng(5)
    lens = [70, 9, 131, 1, 64, 33, 90, 200]
    reqs = [m.tokens(n, 120 + i) for i, n in enumerate(lens)]
    dec = m.open(cai, 448, 3, dt)
    todo, live, free = list(range(8)), {}, [0, 1, 2]
    got = {i: [] for i in todo}
    while todo or live:
        while free and todo:
            live[todo.pop(0)] = [free.pop(int(rng.integers(len(free)))), 0]
        pick = [i for i in live if rng.random() < 0.8] or list(live)
        rng.shuffle(pick)
        entries, where = [], []
        for i in pick:
            slot, at = live[i]
            n = min(int(rng.choice([1, 1, 1, 2, 3, 17, 40, 64])), lens[i] - at)
            entries.append((slot, reqs[i][at:at + n], range(n))); where.append((i, n))
        lg = dec.step_batch(entries)[1]
        r0 = 0
        for i, n in where:
            got[i].append(lg[r0:r0 + n]); r0 += n
            live[i][1] += n
            if live[i][1] == lens[i]:
                slot = live.pop(i)[0]
                dec.reset(slot); free.append(slot)
    for i in got:
        check(np.concatenate(got[i]), m.ref(reqs[i]), dt)
    assert dec.room(0) == 448                     # every page came back
    dec.close()


@DT
@pytest.mark.parametrize("rows", [2, 3, 5, 8, 11])
def test_decoding_together_agrees_with_each_request_alone(cai, models, rows, dt):
    """single tokens of many requests at different lengths: captured steps of up to eight rows, and wider ones"""
    m = models[dt]
    reqs = [m.tokens(10 + 7 * b, 200 + b) for b in range(rows)]
    dec = m.open(cai, 64 * 2 * rows, rows, dt)
    for b in range(rows):
        dec.step_batch([(b, reqs[b][:-4], [])])
    for k in range(4, 0, -1):
        lg = dec.step_batch([(b, reqs[b][len(reqs[b]) - k:][:1], [0]) for b in range(rows)])[1]
        check(lg, np.stack([m.ref(reqs[b])[-k] for b in range(rows)]), dt)
    dec.close()


@pytest.fixture(scope="module")
def wide(tmp_path_factory):
    """wider than the streaming products stage at once for eight rows, rows split between waves, a width that is no multiple of the padding"""
    cfg = B.zconfig([B.zlayer(B.lat(heads=12, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=768, scale=0.07), B.zmoe(experts=8, top=2, ff=300, count=2, keep=1)),
                     B.zlayer(B.forget(heads=8, dim=128, vdim=128), B.zmoe(experts=4, top=2, ff=700, count=2, keep=2)), B.zlayer(B.keyval(heads=8, kv_heads=2, dim=128, rot=64, scale=0.1))], width=2100, vocab=50)
    return Model(tmp_path_factory.mktemp("wide"), cfg, seed=2, edit=B.steady_groups)


@DT
@pytest.mark.parametrize("rows", [1, 2, 3, 4, 5, 6, 7, 8, 9])
def test_wide_layers_in_small_batches(cai, wide, rows, dt):
    reqs = [wide.tokens(4 + b, 500 + b) for b in range(rows)]
    dec = wide.open(cai, 64 * rows, rows, dt)
    got = [[] for _ in reqs]
    for k in range(2):                            # one token each, twice
        lg = dec.step_batch([(b, reqs[b][k:k + 1], [0]) for b in range(rows)])[1]
        for b in range(rows):
            got[b].append(lg[b:b + 1])
    for b in range(rows):                         # the rest in a portion of one to ten tokens
        got[b].append(dec.step_batch([(b, reqs[b][2:], range(len(reqs[b]) - 2))])[1])
        check(np.concatenate(got[b]), wide.ref(reqs[b]), dt)
    dec.close()


@DT
def test_wide_layers_in_prompts(cai, wide, dt):
    tok = wide.tokens(200, 7)
    dec = wide.open(cai, 256, 1, dt)
    for cuts in ([200], [90, 70, 1], [20, 33, 64]):
        dec.reset()
        check(feed(dec, tok, cuts), wide.ref(tok), dt)
    dec.close()


@pytest.mark.parametrize("width", [1026, 1030, 2052, 4100])
def test_widths_of_every_stream_launch(cai, tmp_path, width):
    m = Model(tmp_path, B.zconfig([B.zlayer(B.keyval()), B.zlayer(B.forget(), B.zmoe(ff=9))], width=width, vocab=40), seed=3, edit=B.steady_groups)
    tok = m.tokens(80, 2)
    dec = m.open(cai, 128, 1)
    for cuts in ([80], [70, 1], [6, 3]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), "f32")
    dec.close()


def test_batches_agree_with_each_request_alone_to_rounding(cai, models):
    m = models["f32"]
    reqs = [m.tokens(n, 60 + n) for n in (21, 90, 2, 1)]
    dec = m.open(cai, 512, 4)
    alone = []
    for r in reqs:
        alone.append(feed(dec, r, [len(r)])); dec.reset()
    lg = dec.step_batch([(3 - i, r, range(len(r))) for i, r in enumerate(reqs)])[1]
    assert err(lg.astype(np.float64), np.concatenate(alone).astype(np.float64)) < 8e-6
    dec.close()


# ---------------------------------------------------------------- far tokens, page borders
def pointed(kind, heads=2):
    """token 400 + t asks for token t: keys carry a sign vector in the first half of the width, askers the same one in the second, keys
    are made of the first half and queries of the second, so that one score stands far above all others"""
    mix = B.keyval(heads=heads, kv_heads=1, dim=64, scale=0.2, rot=2) if kind == "keys" else B.lat(heads=heads, dim=64, rot_dim=8, vdim=24, kv_rank=64, q_rank=64, scale=0.2)
    cfg = B.zconfig([B.zlayer(mix)], width=128, vocab=800, cap=20.0)

    def edit(w):
        sign = np.sign(np.random.default_rng(77).standard_normal((400, 64)))
        w["embed"] = np.zeros((800, 128)); w["embed"][:400, :64] = sign; w["embed"][400:, 64:] = sign
        a = "l0.mix."
        w["l0.norm1"] = np.ones(128); w["l0.canon1"] *= 0; w["l0.norm1b"] *= 2
        if kind == "keys":
            w[a + "k"] = np.eye(64, 128); w[a + "q"] = np.concatenate([np.eye(64, 128, 64)] * heads); w[a + "sink"] = np.full(heads, 2.0)
        else:
            w[a + "dq"] = np.eye(64, 128, 64); w[a + "dq.norm"] = np.ones(64); w[a + "dkv.norm"] = np.ones(64)
            w[a + "dkv"][:64] = np.eye(64, 128); w[a + "dkv"][64:] *= 0.3
            w[a + "uk"] = np.concatenate([np.eye(64)] * heads)
            w[a + "uq"] = np.concatenate([np.concatenate([np.eye(64), 0.3 * w[a + "uq"][:8]])] * heads)
    return cfg, edit


@DT
@pytest.mark.parametrize("kind", ["keys", "latents"])
def test_far_keys_and_page_borders(cai, tmp_path, kind, dt):
    """a key that outweighs all others, first and last in its page, asked for from beside it, from across a border and from hundreds
    of tokens later, in prompts, in portions and decoded; and asked for too early, when it must not be seen yet"""
    cfg, edit = pointed(kind)
    m = Model(tmp_path, cfg, seed=3, edit=edit)
    T = 390
    keys = np.random.default_rng(2).permutation(400)[:T]
    tok = keys.copy()
    asks = {1: 0, 64: 63, 66: 64, 70: 2, 127: 126, 128: 65, 129: 127, 150: 20, 192: 191, 200: 128, 255: 193, 256: 60, 260: 3, 318: 130, 319: 190, 320: 0, 321: 257, 384: 65, 387: 253, 389: 4}
    for at, key in asks.items():
        tok[at] = 400 + keys[key]
    early = {30: 31, 62: 63, 100: 190, 191: 194}
    for at, key in early.items():
        tok[at] = 400 + keys[key]
    want = m.ref(tok)
    for at, key in asks.items():                  # the oracle tells: without the key the asker's logits are others
        if key not in asks and key not in early:
            lost = tok.copy(); lost[key] = keys[(key + 7) % 390] if (key + 7) % 390 not in asks else 399
            assert err(R.forward(cfg, m.w, lost[:at + 1])[at:], want[at:at + 1]) > 0.08, (at, key)
    dec = m.open(cai, 448, 1, dt)
    for cuts in ([T], [60, 1], [2, 100, 3], [65, 63, 20, 1, 1, 40], [256, 1]):
        dec.reset()
        check(feed(dec, tok.tolist(), cuts), want, dt)
    dec.close()


@DT
def test_a_state_that_is_lost_shows(cai, tmp_path, dt):
    """one token writes under gates that hardly forget and later ones write little: hundreds of tokens on, whatever the portions, what is
    read is its value"""
    def edit(w):
        w["l0.canon1"] *= 0; w["l0.norm1"] = np.ones(64)
        w["embed"][:, 0] = -4.0; w["embed"][7, 0] = 4.0
        f = np.zeros((60, 64)); f[:, 0] = -6.0
        w["l0.mix.f"] = f; w["l0.mix.f.b"] = np.full(60, -2.0); w["l0.mix.lower"] = np.full(60, 0.02)
    m = Model(tmp_path, B.zconfig([B.zlayer(B.forget(heads=3, dim=20, vdim=28))], width=64, vocab=90, cap=20.0), seed=4, edit=edit)
    tok = [int(t) if t != 7 else 8 for t in m.tokens(300, 5)]
    tok[5] = 7
    other = list(tok); other[5] = 9
    assert err(m.ref(other)[-1:], m.ref(tok)[-1:]) > 0.1
    dec = m.open(cai, 64, 1, dt)
    for cuts in ([300], [1], [6, 1, 16, 15, 2, 64], [5, 2, 100]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


# ---------------------------------------------------------------- long decoding, generation, sessions
@DT
def test_long_decoding(cai, models, dt):
    """token by token across page borders and every size of the captured steps' launches"""
    m = models[dt]
    tok = m.tokens(580, 8)
    dec = m.open(cai, 640, 1, dt)
    check(feed(dec, tok, [1]), m.ref(tok), dt)
    dec.close()


@DT
def test_thousands_of_keys(cai, tmp_path, dt):
    """soft-max over many slices, 32-bit rows in turns; positions past the length the rotation was made for"""
    m = Model(tmp_path, B.zconfig([B.zlayer(B.lat(heads=16, dim=16, rot_dim=16, vdim=16, kv_rank=256, scale=0.25)), B.zlayer(B.keyval(heads=8, kv_heads=2, dim=32, rot=32, scale=0.3))], width=32, vocab=60), seed=8)
    tok = m.tokens(2100, 3)
    want = m.ref(tok)
    dec = m.open(cai, 2112, 1, dt)
    check(feed(dec, tok, [2100]), want, dt)
    dec.reset()
    check(feed(dec, tok, [1500, 560, 3, 1]), want, dt)
    dec.close()


def test_the_pool_bounds_what_is_held(cai, models):
    m = models["f32"]
    dec = m.open(cai, 192, 2)
    tok = m.tokens(200, 3)
    feed(dec, tok[:128], [128])
    assert dec.room(0) == 64 and dec.room(1) == 64
    feed(dec, tok[:64], [64], 1)
    with pytest.raises(cai.CaiError):
        dec.step_batch([(0, tok[128:129], [0])])
    dec.reset(1)
    check(feed(dec, tok[128:192], [1]), m.ref(tok[:192])[128:], "f32")
    dec.close()


def test_greedy_generation_through_every_entry_point(cai, models):
    m = models["f32"]
    prompts = [m.tokens(n, 70 + n) for n in (30, 3, 77, 12, 64)]
    dec = m.open(cai, 384, 2)
    want = []
    for p in prompts:
        want.append(greedy(dec, p, 40)); dec.reset()
        margin(m, p, want[-1])
    am, _ = dec.prefill(prompts[2])               # the captured device-side loop, across page borders
    assert [am] + dec.generate(am, 77, 39).tolist() == want[2]
    dec.reset()
    am, lg = dec.step_window(prompts[1], 0)
    check(lg, m.ref(prompts[1]), "f32")
    am, lg = dec.step([want[1][0]], [3])
    check(lg, m.ref(prompts[1] + want[1][:1])[3:], "f32")
    dec.reset()
    sched = cai.Scheduler(dec, max_rows=24, portion=10)
    ids = [sched.submit(p, 40) for p in prompts]
    live, waiting = sched.step()
    assert live == 2 and waiting == 3
    sched.run()
    assert [sched.result(i) for i in ids] == [(w, True) for w in want]
    stop = want[0][5]
    a = sched.submit(prompts[0], 40, eos=stop); b = sched.submit(prompts[1], 40); sched.step(); sched.drop(b); sched.run()
    assert sched.result(a)[0] == want[0][:want[0].index(stop) + 1]
    c = sched.submit(prompts[0], 12, temperature=1.2, top_k=8, seed=3); sched.run()
    assert len(sched.result(c)[0]) == 12
    sched.close(); dec.close()


def test_long_generation_on_the_device(cai, models):
    """hundreds of tokens through the captured loop, which is captured anew as the sequence grows"""
    m = models["f32"]
    p = m.tokens(230, 5)
    dec = m.open(cai, 640)
    am, _ = dec.prefill(p)
    got = [am] + dec.generate(am, 230, 330).tolist()
    lg = m.ref(p + got[:-1])[229:]
    chosen = lg[np.arange(len(got)), got]
    assert (lg.max(1) - chosen).max() < 1e-3 * np.abs(lg).max()
    dec.close()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_a_captured_step_repeats(cai, models, dt):
    """the same captured steps over other sequences, lengths and pages, with other work in between"""
    m = models[dt]
    dec = m.open(cai, 640, 4, dt)
    for rnd in range(3):
        reqs = [m.tokens(40 + 9 * b + rnd, 300 + 10 * rnd + b) for b in range(3)]
        seqs = [(b + rnd) % 4 for b in range(3)]
        for b in range(3):
            dec.step_batch([(seqs[b], reqs[b][:30], [])])
        for t in range(30, 38):
            lg = dec.step_batch([(seqs[b], reqs[b][t:t + 1], [0]) for b in range(3)])[1]
            check(lg, np.stack([m.ref(reqs[b])[t] for b in range(3)]), dt)
        for s in seqs:
            dec.reset(s)
    dec.close()


@DT
def test_snapshot_restore_fork_and_hidden_state(cai, models, dt):
    m = models[dt]
    tok = m.tokens(120, 31)
    dec = m.open(cai, 448, 2, dt)
    feed(dec, tok[:80], [80])
    snap = dec.snapshot()
    dec.fork(0, 1)
    check(feed(dec, tok[80:], [7], 0), m.ref(tok)[80:], dt); check(feed(dec, tok[80:], [1], 1), m.ref(tok)[80:], dt)
    dec.reset(1)
    dec.restore(snap, 1)
    check(feed(dec, tok[80:], [40], 1), m.ref(tok)[80:], dt)
    read = lambda h: R.soft_cap(R.linear(m.w["embed"], h.astype(np.float64))[None], m.cfg["logit_softcap"])
    check(read(dec.hidden_state(39)), m.ref(tok)[-1:], dt)
    more = tok + [5]
    dec.step_batch([(1, [5], [0])])
    check(read(dec.hidden_state(0)), m.ref(more)[-1:], dt)
    cai.load().cai_kv_snap_destroy(snap)
    dec.close()


def mixer(l, **kw):
    return lambda c, w: c["layers"][l]["mixer"].update(**kw)


def groups(**kw):
    return lambda c, w: c["layers"][0]["mlp"]["router"]["groups"].update(**kw)


@pytest.mark.parametrize("name, change", [
    ("heads", mixer(1, heads=3)), ("vdim", mixer(1, vdim=20)), ("type", lambda c, w: c["layers"][0].update(type="delta")), ("mix.g", mixer(0, heads=2)), ("rot.dims", mixer(0, rot=dict(dims=14, base=3.0))),
    ("rot.dims", mixer(1, rot=dict(dims=3, base=9.0))), ("rot.base", mixer(1, rot=dict(dims=4))), ("scaling.slow", mixer(0, rot=dict(dims=4, base=9.0, scaling=dict(factor=2.0, original=9, fast=2.0)))),
    ("scaling.factor", mixer(1, rot=dict(dims=4, base=9.0, scaling=dict(factor=0)))), ("scale", lambda c, w: c["layers"][0]["mixer"].pop("scale")), ("kv_rank", mixer(0, kv_rank=4096)), ("dkv", mixer(0, kv_rank=35)),
    ("sink", lambda c, w: w.pop("l1.mix.sink")), ("lower", lambda c, w: w.pop("l2.mix.lower")), ("f.b", lambda c, w: w.pop("l2.mix.f.b")), ("canon1", lambda c, w: w.pop("l1.canon1")), ("canon1", lambda c, w: c["canon"].update(taps=2)),
    ("canon.taps", lambda c, w: c.pop("canon")), ("dwa", lambda c, w: w.update({"l1.dwa": np.ones(2)})), ("norm2b", lambda c, w: w.pop("l0.norm2b")), ("norm1b", lambda c, w: w.pop("l2.norm1b")),
    ("router.top", lambda c, w: c["layers"][0]["mlp"]["router"].update(top=9)), ("groups", groups(count=3)), ("groups", groups(keep=1)), ("groups.keep", groups(keep=5)), ("groups.count", lambda c, w: c["layers"][0]["mlp"]["router"].pop("groups")),
    ("e5", lambda c, w: w.pop("l0.mlp.e5.up")), ("correction", lambda c, w: w.pop("l0.mlp.correction")), ("kind", lambda c, w: c["layers"][0]["mlp"].update(kind="dense")), ("logit_softcap", lambda c, w: c.pop("logit_softcap")),
    ("embedding.scale", lambda c, w: c.pop("embedding")), ("norm.eps", lambda c, w: c.pop("norm")), ("final.norm", lambda c, w: w.pop("final.norm"))])
def test_loader_names_what_is_wrong(cai, tmp_path, name, change):
    cfg = B.zconfig([B.zlayer(B.lat(), B.zmoe()), B.zlayer(B.keyval()), B.zlayer(B.forget())])
    w = B.weights(cfg)
    change(cfg, w)
    B.write(str(tmp_path), cfg, w)
    with pytest.raises(cai.CaiError) as e:
        cai.Decoder.load(str(tmp_path), 64)
    assert name in str(e.value)


# ---------------------------------------------------------------- programs
def test_command_line_generation(cai, models):
    m = models["f32"]
    prompts = [m.tokens(9, 1), m.tokens(20, 2)]
    dec = m.open(cai, 192)
    want = []
    for p in prompts:
        want.append(greedy(dec, p, 7)); dec.reset()
    dec.close()
    exe = os.path.join(ROOT, "neural-api_amd", "host", "caihip_run")
    both = subprocess.run([exe, m.folder, "7", "--dtype", "float32", "--portion", "4"] + [str(t) for t in prompts[0]] + ["--"] + [str(t) for t in prompts[1]],
                          capture_output=True, text=True, timeout=100)
    assert [[int(t) for t in s.split()] for s in both.stdout.splitlines()] == want, both.stdout + both.stderr


@pytest.mark.parametrize("dt, name", [("f32", "float32"), ("bf16", "bfloat16")])
def test_trace_replay(cai, models, tmp_path, dt, name):
    m = models[dt]
    a, b = m.tokens(50, 6), m.tokens(30, 7)
    steps = [dict(step=0, entries=[dict(id="x", tokens=a[:40], want=[39, 0])], end=[]), dict(step=1, entries=[dict(id="y", tokens=b[:2], want=[])], end=[]),
             dict(step=2, entries=[dict(id="y", tokens=b[2:], want=[27]), dict(id="x", tokens=a[40:41], want=[0])], end=["y"]),
             dict(step=3, entries=[dict(id="z", tokens=b, want=[29]), dict(id="x", tokens=a[41:], want=[8, 7])], end=["x", "z"])]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", m.folder, "--dtype", name, "--out", str(tmp_path), "--max-tokens", "128"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done %d" % i for i in range(4)], r.stderr
    got = lambda i: np.fromfile(tmp_path / ("%d.f32" % i), "<f4").reshape(-1, m.cfg["vocab"])
    check(got(0), m.ref(a)[[39, 0]], dt)
    assert not os.path.exists(tmp_path / "1.f32")
    check(got(2), np.stack([m.ref(b)[29], m.ref(a)[40]]), dt)
    check(got(3), np.stack([m.ref(b)[29], m.ref(a)[49], m.ref(a)[48]]), dt)
