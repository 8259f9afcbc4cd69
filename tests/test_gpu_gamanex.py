"""Gamanex on the device against the float64 oracle: every mechanism alone over sizes, prompts against token-by-token decoding,
portions, mixed batches, reused pages and slots, keys far away and at page borders, keys of another layer, long decoding, generation
through the scheduler."""
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


MIXED = dict(layers=[B.glayer(B.sig(heads=6, kv_heads=2, dim=20, vdim=44, every=11), B.gmoe(experts=9, top=4, ff=17)),
                     B.glayer(B.sig(heads=3, kv_heads=3, dim=33, vdim=9, every=1, coef=0.2, scale=0.3), 52),
                     B.glayer(B.sig(heads=6, kv_heads=2, dim=20, vdim=44, every=3, coef=0.6, scale=0.15, kv_from=0)),
                     B.glayer(B.sig(heads=3, kv_heads=3, dim=33, vdim=9, every=64, scale=0.2, kv_from=1), B.gmoe(experts=5, top=5, ff=40)),
                     B.glayer(B.sig(heads=5, kv_heads=1, dim=16, vdim=24), 31)], width=100, vocab=211, logit_scale=1.3)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """bf16: the choice of experts is decided by far, so that the oracle and 16-bit activations cannot part there"""
    cfg = B.gconfig(**MIXED)
    return {dt: Model(tmp_path_factory.mktemp("gamanex"), cfg, seed=21, edit=B.steady_experts(cfg) if dt == "bf16" else None) for dt in ("f32", "bf16")}


# ---------------------------------------------------------------- each mechanism alone
SIG = [B.sig(h, g, d, dv, sc, coef, every) for h, g, d, dv, sc, coef, every in (
    (1, 1, 8, 8, 0.5, 0.5, 1), (4, 4, 24, 40, 0.3, 0.3, 2), (6, 2, 48, 96, 0.2, 0.1, 64), (8, 1, 130, 70, 0.1, 0.7, 65),
    (10, 2, 256, 256, 0.06, 0.2, 33), (2, 1, 64, 20, 0.2, 1.1, 1000), (3, 1, 18, 9, 0.4, 0.4, 63), (15, 3, 72, 64, 0.15, 0.05, 128), (16, 8, 32, 128, 0.25, 0.0, 5))]
MOE = [B.gmoe(n, top, ff) for n, top, ff in ((4, 1, 16), (8, 8, 33), (37, 5, 20), (130, 6, 9), (512, 3, 5), (66, 64, 3), (16, 2, 70))]


@DT
@pytest.mark.parametrize("i", range(len(SIG)))
def test_sigmoid_attention_alone(cai, tmp_path, i, dt):
    m = Model(tmp_path, B.gconfig([B.glayer(SIG[i])], width=40 + 8 * i, vocab=67, eps=10.0 ** -(2 + i % 5), logit_scale=0.5 + i), seed=i)
    tok = m.tokens(150, i)
    dec = m.open(cai, 192, 1, dt)
    for cuts in ([150], [100, 1], [64, 65, 2, 1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("what", ["distance", "temperature", "head number", "norm over all heads", "layer scale", "gate", "eps"])
def test_one_mechanism_made_strong(cai, tmp_path, what, dt):
    """the others neutral, this one large enough to carry the result: leaving it out in the oracle moves the logits far"""
    cfg = B.gconfig([B.glayer(B.sig(heads=4, kv_heads=2, coef=1.5 if what == "temperature" else 0.0, every=10), 40)], width=64, vocab=90, logit_scale=1.0, eps=0.5 if what == "eps" else 1e-6)

    def neutral(w, keep=None):
        one = {"distance": ("l0.mix.r1",), "head number": ("l0.mix.pb",), "layer scale": ("l0.ls1", "l0.ls2"), "gate": ("l0.rg1", "l0.rg1.b", "l0.rg2", "l0.rg2.b")}.get(keep, ())
        for n in w:
            if n in one:
                continue
            if n.endswith((".r1", ".pb", ".rg1", ".rg2", ".b")):
                w[n] = w[n] * 0
            elif n.endswith((".ls1", ".ls2", "norm1", "norm2")) or (n.endswith("q.norm") and keep != "norm over all heads"):
                w[n] = np.ones_like(w[n])

    def edit(w):
        neutral(w, what)
        if what == "distance":
            w["l0.mix.r1"] = np.array([3.0, 0.5, 1.0, 2.0]); w["l0.mix.r2"] = np.array([0.05, 4.0, 1.0, 0.3])
        if what == "norm over all heads":          # a head far larger than the others: a norm per head would level them
            w["l0.mix.q"][:24] *= 6; w["l0.mix.k"][24:] *= 5
    m = Model(tmp_path, cfg, seed=9, edit=edit)
    tok = m.tokens(140, 4)
    plain = dict(m.w)
    if what == "norm over all heads":
        plain["l0.mix.q"] = plain["l0.mix.q"].copy(); plain["l0.mix.q"][:24] /= 6; plain["l0.mix.k"] = plain["l0.mix.k"].copy(); plain["l0.mix.k"][24:] /= 5
    else:
        neutral(plain)
    bare = json.loads(json.dumps(cfg)); bare["layers"][0]["mixer"]["q_temp"]["coef"] = 0.0; bare["norm"]["eps"] = 1e-6
    assert err(R.forward(bare, plain, np.array(tok)), m.ref(tok)) > 0.15
    dec = m.open(cai, 192, 1, dt)
    for cuts in ([140], [90, 1], [1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("i", range(len(MOE)))
def test_experts_alone(cai, tmp_path, i, dt):
    """one layer whose mixer adds nothing, so that every token stands alone; tokens whose choice of experts is close are left out"""
    def edit(w):
        w["l0.ls1"] *= 0
    m = Model(tmp_path, B.gconfig([B.glayer(B.sig(heads=1, kv_heads=1, dim=8, vdim=8), MOE[i])], width=56 + 12 * i, vocab=400), seed=30 + i, edit=edit)
    r, w = MOE[i]["router"], m.w
    h = R.rms_norm(w["embed"], 1e-5) * w["l0.norm2"]
    z = R.linear(w["l0.mlp.router"], h) + w["l0.mlp.router.b"]
    top = np.sort(z, axis=1)[:, ::-1]
    clear = np.arange(400)
    if r["top"] < r["experts"]:
        clear = clear[top[:, r["top"] - 1] - top[:, r["top"]] > (1e-5 if dt == "f32" else 3e-2)]
    assert len(clear) > 12
    tok = np.random.default_rng(i).choice(clear, 90).tolist()
    dec = m.open(cai, 128, 1, dt)
    for cuts in ([90], [9, 8, 3, 1], [5, 2, 30]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("mlp", [None, 1, 31, 64, 200], ids=str)
def test_feed_forward_beside_the_mixer(cai, tmp_path, mlp, dt):
    """none at all, one row, widths around the padding; a second layer of another width leaves the padding of the first one dirty"""
    m = Model(tmp_path, B.gconfig([B.glayer(B.sig(), mlp), B.glayer(B.sig(), 130), B.glayer(B.sig(), mlp)], width=60, vocab=90), seed=5)
    tok = m.tokens(70, 2)
    dec = m.open(cai, 128, 1, dt)
    for cuts in ([60, 1], [8, 5, 2, 1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("frm", [(None, 0, 0, 0), (None, None, 0, 1, 0), (None, 0, None, 2, 0, 2)], ids=str)
def test_keys_and_values_of_an_earlier_layer(cai, tmp_path, frm, dt):
    """neighbours and layers further back, several readers of one layer, in turns with layers that keep their own"""
    cfg = B.gconfig([B.glayer(B.sig(kv_from=f, scale=0.15 + 0.03 * i, every=4 + i, coef=0.1 * i), 40 if i % 2 else None) for i, f in enumerate(frm)], width=70)
    m = Model(tmp_path, cfg, seed=len(frm))
    tok = m.tokens(140, 1)
    dec = m.open(cai, 192, 2, dt)
    for cuts in ([140], [40, 1], [33, 2, 70, 5]):
        dec.reset(1)
        check(feed(dec, tok, cuts, 1), m.ref(tok), dt)
    dec.close()


# ---------------------------------------------------------------- whole models
@DT
@pytest.mark.parametrize("cuts", [[300], [1], [2], [3, 2, 65, 1, 1, 16, 17, 2], [64], [130, 1], [5, 9, 7]], ids=str)
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
    for n in range(1, 7):
        tok = m.tokens(n, 40 + n)
        for cuts in ([n], [1]):
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
    cfg = B.gconfig([B.glayer(B.sig(heads=4, kv_heads=2, dim=130, vdim=136), 2600), B.glayer(B.sig(heads=4, kv_heads=2, dim=130, vdim=136, kv_from=0), B.gmoe(experts=4, top=2, ff=300))], width=2100, vocab=50)
    return Model(tmp_path_factory.mktemp("wide"), cfg, seed=2, edit=B.steady_experts(cfg))


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
    for b in range(rows):                         # the rest in a portion of one to eight tokens
        got[b].append(dec.step_batch([(b, reqs[b][2:], range(len(reqs[b]) - 2))])[1])
        check(np.concatenate(got[b]), wide.ref(reqs[b]), dt)
    dec.close()


def test_batches_agree_with_each_request_alone_to_rounding(cai, models):
    m = models["f32"]
    reqs = [m.tokens(n, 60 + n) for n in (21, 90, 2, 1)]
    dec = m.open(cai, 512, 4)
    alone = []
    for r in reqs:
        alone.append(feed(dec, r, [len(r)])); dec.reset()
    lg = dec.step_batch([(3 - i, r, range(len(r))) for i, r in enumerate(reqs)])[1]
    assert err(lg.astype(np.float64), np.concatenate(alone).astype(np.float64)) < 4e-6
    dec.close()


# ---------------------------------------------------------------- far tokens, page borders
def pointed(heads=2, layers=1):
    """token 400 + t asks for token t: keys carry a sign vector in the first half of the width, askers the same one in the second,
    W_k reads the first half and W_q the second, so that one score stands far above all others.  With two layers the second one
    reads the first one's keys."""
    cfg = B.gconfig([B.glayer(B.sig(heads=heads, kv_heads=1, dim=64, vdim=24, scale=0.17, coef=0.05, every=100, kv_from=0 if i else None)) for i in range(layers)], width=128, vocab=800)

    def edit(w):
        sign = np.sign(np.random.default_rng(77).standard_normal((400, 64)))
        w["embed"] = np.zeros((800, 128)); w["embed"][:400, :64] = sign; w["embed"][400:, 64:] = sign
        w["l0.mix.k"] = np.eye(64, 128); w["l0.mix.k.norm"] = np.ones(64); w["l0.mix.v"] *= 3
        for i in range(layers):
            p = "l%d." % i
            w[p + "norm1"] = np.ones(128); w[p + "mix.q"] = np.concatenate([np.eye(64, 128, 64)] * heads); w[p + "mix.q.norm"] = np.ones(64 * heads)
            w[p + "mix.pb"] = np.full(heads, -7.0); w[p + "mix.r1"] = np.full(heads, 0.3); w[p + "mix.r2"] = np.full(heads, 0.5)
            w[p + "mix.o"] *= 2
            w[p + "ls1"] = np.ones(128)
            if i + 1 < layers:                     # the first layer's own result stays out of the way
                w[p + "ls1"] *= 0
    return cfg, edit


@DT
@pytest.mark.parametrize("layers", [1, 2])
def test_far_keys_and_page_borders(cai, tmp_path, layers, dt):
    """a key that outweighs all others, first and last in its page, asked for from beside it, from across a border and from hundreds
    of tokens later, in prompts, in portions and decoded; and asked for too early, when it must not be seen yet"""
    cfg, edit = pointed(layers=layers)
    m = Model(tmp_path, cfg, seed=3, edit=edit)
    T = 390
    keys = np.random.default_rng(2).permutation(400)[:T]
    tok = keys.copy()
    asks = {1: 0, 64: 63, 66: 64, 70: 2, 127: 126, 128: 65, 129: 127, 150: 20, 192: 191, 200: 128, 255: 192, 256: 60, 260: 3, 318: 129, 319: 190, 320: 0, 321: 257, 384: 65, 387: 253, 389: 4}
    for at, key in asks.items():
        tok[at] = 400 + keys[key]
    early = {30: 31, 62: 64, 100: 190, 191: 193}
    for at, key in early.items():
        tok[at] = 400 + keys[key]
    want = m.ref(tok)
    for at, key in asks.items():                  # the oracle tells: without the key the asker's logits are others
        if key not in asks and key not in early:
            lost = tok.copy(); lost[key] = keys[(key + 7) % 390] if (key + 7) % 390 not in asks else 399
            assert err(R.forward(cfg, m.w, lost[:at + 1])[at:], want[at:at + 1]) > 0.1, (at, key)
    dec = m.open(cai, 448, 1, dt)
    for cuts in ([T], [60, 1], [2, 100, 3], [65, 63, 20, 1, 1, 40], [256, 1]):
        dec.reset()
        check(feed(dec, tok.tolist(), cuts), want, dt)
    dec.close()


@DT
def test_long_sums_over_thousands_of_keys(cai, tmp_path, dt):
    """no normalisation: thousands of small weights must add up, near and far, and 32-bit rows over many slices go in turns"""
    def edit(w):
        w["l0.mix.pb"] = np.linspace(-6.0, -3.0, 16); w["l0.mix.v"] += 0.05
    m = Model(tmp_path, B.gconfig([B.glayer(B.sig(heads=16, kv_heads=1, dim=16, vdim=256, every=500))], width=32, vocab=60), seed=8, edit=edit)
    tok = m.tokens(2100, 3)
    want = m.ref(tok)
    dec = m.open(cai, 2112, 1, dt)
    check(feed(dec, tok, [2100]), want, dt)
    dec.reset()
    check(feed(dec, tok, [1500, 560, 3, 1]), want, dt)
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


def test_a_captured_step_repeats(cai, models):
    """the same captured steps over other sequences, lengths and pages, with other work in between"""
    m = models["f32"]
    dec = m.open(cai, 640, 4)
    for rnd in range(3):
        reqs = [m.tokens(40 + 9 * b + rnd, 300 + 10 * rnd + b) for b in range(3)]
        seqs = [(b + rnd) % 4 for b in range(3)]
        for b in range(3):
            dec.step_batch([(seqs[b], reqs[b][:30], [])])
        for t in range(30, 38):
            lg = dec.step_batch([(seqs[b], reqs[b][t:t + 1], [0]) for b in range(3)])[1]
            check(lg, np.stack([m.ref(reqs[b])[t] for b in range(3)]), "f32")
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
    read = lambda h: R.linear(m.w["head"], h.astype(np.float64))[None] * m.cfg["logit_scale"]
    check(read(dec.hidden_state(39)), m.ref(tok)[-1:], dt)
    more = tok + [5]
    dec.step_batch([(1, [5], [0])])
    check(read(dec.hidden_state(0)), m.ref(more)[-1:], dt)
    cai.load().cai_kv_snap_destroy(snap)
    dec.close()


def mixer(l, **kw):
    return lambda c, w: c["layers"][l]["mixer"].update(**kw)


@pytest.mark.parametrize("name, change", [
    ("heads", mixer(0, heads=3, kv_heads=2)), ("type", lambda c, w: c["layers"][0].update(type="delta")), ("mix.q", mixer(0, heads=2)), ("q_temp.every", mixer(0, q_temp=dict(coef=1.0))),
    ("q_temp.coef", mixer(0, q_temp=dict(every=3))), ("scale", lambda c, w: c["layers"][0]["mixer"].pop("scale")), ("kv_from", mixer(1, kv_from=1)), ("kv_from", mixer(2, kv_from=1)),
    ("kv_from", mixer(0, kv_from=0)), ("kv_from", mixer(1, kv_heads=4)), ("mix.v", lambda c, w: w.pop("l0.mix.v")), ("r2", lambda c, w: w.pop("l1.mix.r2")), ("pb", lambda c, w: w.pop("l2.mix.pb")),
    ("ls2", lambda c, w: w.pop("l1.ls2")), ("rg1.b", lambda c, w: w.pop("l0.rg1.b")), ("rg2", lambda c, w: w.pop("l0.rg2")), ("norm2", lambda c, w: w.pop("l0.norm2")),
    ("router.top", lambda c, w: c["layers"][1]["mlp"]["router"].update(top=7)), ("e5", lambda c, w: w.pop("l1.mlp.e5.up")), ("router.b", lambda c, w: w.pop("l1.mlp.router.b")),
    ("kind", lambda c, w: c["layers"][0]["mlp"].update(kind="other")), ("mlp.up", lambda c, w: c["layers"][0]["mlp"].update(ff=41)), ("logit_scale", lambda c, w: c.pop("logit_scale")),
    ("norm.eps", lambda c, w: c.pop("norm")), ("final.norm", lambda c, w: w.pop("final.norm"))])
def test_loader_names_what_is_wrong(cai, tmp_path, name, change):
    cfg = B.gconfig([B.glayer(B.sig(), 40), B.glayer(B.sig(kv_from=0), B.gmoe()), B.glayer(B.sig())])
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
