"""Kiruvik on the device against the float64 oracle: every mechanism alone over sizes, prompts against token-by-token decoding,
portions, mixed batches, reused pages and slots, block edges, far tokens, long decoding, generation through the scheduler."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from helpers import layered_build as B
from helpers import layered_ref as R
from helpers.device import ROOT, dev
from helpers.layered_model import TOL, Model, check, err, feed, greedy, margin

pytestmark = pytest.mark.gpu
DT = pytest.mark.parametrize("dt", ["f32", "bf16"])


@pytest.fixture(scope="module")
def cai():
    return dev()


MIXED = dict(layers=[B.klayer(B.ssd()), B.klayer(B.rotary(heads=6, kv_heads=2, dim=20, vdim=44, block=11, rot=8), B.moe()),
                     B.klayer(B.ssd(heads=3, vdim=37, state=35, groups=1, conv=5, norm_groups=1), B.moe(experts=9, top=4, ff=17, shared_ff=70)),
                     B.klayer(B.rotary(heads=3, kv_heads=3, dim=33, vdim=9, block=70, rot=32, base=90.0), 52), B.klayer(B.ssd(heads=6, vdim=8, state=65, groups=3, conv=1, norm_groups=6), 17)],
             width=100, vocab=211, loop=dict(start=1, stop=4, times=2))


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """bf16: the choice of experts is decided by far, so that the oracle and 16-bit activations cannot part there"""
    return {dt: Model(tmp_path_factory.mktemp("kiruvik"), B.kconfig(**MIXED), seed=21, edit=B.steady_choice if dt == "bf16" else None) for dt in ("f32", "bf16")}


# ---------------------------------------------------------------- each mechanism alone
ROTARY = [B.rotary(h, g, d, dv, blk, sc, rot, base) for h, g, d, dv, blk, sc, rot, base in (
    (1, 1, 8, 8, 1, 0.5, 8, 10.0), (4, 4, 24, 40, 2, 0.3, 2, 1e4), (6, 2, 48, 96, 64, 0.2, 48, 300.0), (8, 1, 130, 70, 65, 0.1, 100, 1e6),
    (10, 2, 256, 256, 33, 0.06, 256, 77.0), (2, 1, 64, 20, 1000, 0.2, 30, 1e4), (3, 1, 18, 9, 63, 0.4, 6, 2.0), (15, 3, 72, 64, 128, 0.15, 64, 1e3))]
SSD = [B.ssd(h, p, n, g, t, ng) for h, p, n, g, t, ng in (
    (1, 8, 8, 1, 1, 1), (4, 16, 16, 2, 4, 2), (6, 20, 33, 3, 3, 4), (2, 130, 129, 1, 5, 1), (8, 64, 128, 2, 4, 8), (3, 256, 256, 3, 2, 3), (24, 35, 48, 1, 4, 5), (16, 9, 70, 4, 7, 1))]
MOE = [B.moe(n, top, ff, sc, lim, sff, slim) for n, top, ff, sc, lim, sff, slim in (
    (4, 1, 16, 1.0, 0.3, 16, 9.0), (8, 8, 33, 2.5, 0.8, 7, 0.4), (37, 5, 20, 0.6, 1.5, 64, 1.0), (130, 6, 9, 1.3, 7.0, 90, 0.7), (512, 3, 5, 1.0, 1.0, 40, 2.0), (66, 64, 3, 1.0, 0.5, 5, 0.2))]


@DT
@pytest.mark.parametrize("i", range(len(ROTARY)))
def test_rotary_block_attention_alone(cai, tmp_path, i, dt):
    m = Model(tmp_path, B.kconfig([B.klayer(ROTARY[i])], width=40 + 8 * i, vocab=67, mult=1.0 + i / 8), seed=i)
    tok = m.tokens(150, i)
    dec = m.open(cai, 192, 1, dt)
    for cuts in ([150], [100, 1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("i", range(len(SSD)))
def test_state_space_duality_alone(cai, tmp_path, i, dt):
    m = Model(tmp_path, B.kconfig([B.klayer(SSD[i])], width=40 + 8 * i, vocab=67, eps=10.0 ** -(2 + i)), seed=i)
    tok = m.tokens(150, i)
    dec = m.open(cai, 192, 1, dt)
    for cuts in ([150], [100, 1], [64, 65, 2, 1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


def test_strong_and_weak_decay(cai, tmp_path):
    """decays from almost none to e^-60 a token, alternating within a chunk: running sums must not cost accuracy"""
    cfg = B.kconfig([B.klayer(B.ssd(heads=6, vdim=16, state=24, groups=2, conv=2, norm_groups=2))], width=64, vocab=90)

    def edit(w):
        w["l0.mix.A_log"] = np.log(np.array([1e-5, 0.1, 1.0, 8.0, 30.0, 60.0])); w["l0.mix.dt_bias"] = np.array([0.0, 1.0, -1.0, 0.5, 0.0, 1.0])
        w["l0.mix.in"][-6:] *= 4
    m = Model(tmp_path, cfg, seed=3, edit=edit)
    tok = m.tokens(200, 1)
    dec = m.open(cai, 256)
    for cuts in ([200], [1], [30, 2]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), "f32")
    dec.close()


@DT
@pytest.mark.parametrize("i", range(len(MOE)))
def test_experts_alone(cai, tmp_path, i, dt):
    """one layer whose mixer adds nothing, so that every token stands alone; tokens whose choice of experts is close are left out"""
    def edit(w):
        w["l0.norm1b"] *= 0; w["l0.norm1b.b"] *= 0
    m = Model(tmp_path, B.kconfig([B.klayer(B.ssd(heads=1, vdim=4, state=4, groups=1, conv=1, norm_groups=1), MOE[i])], width=56 + 12 * i, vocab=400), seed=30 + i, edit=edit)
    r = MOE[i]["router"]
    w, all_tok = m.w, np.arange(400)
    h = R.dynamic_tanh(w["embed"], w["l0.norm2.alpha"], w["l0.norm2"], w["l0.norm2.b"])
    s = R.softmax_rows(R.linear(w["l0.mlp.router"], h)) + w["l0.mlp.correction"]
    top = np.sort(s, axis=1)[:, ::-1]
    clear = all_tok[top[:, r["top"] - 1] - top[:, r["top"]] > (1e-6 if dt == "f32" else 2e-3)] if r["top"] < r["experts"] else all_tok
    assert len(clear) > 12
    plain = np.argsort(-(s - w["l0.mlp.correction"]), axis=1)[:, :r["top"]]
    assert r["top"] > 1 or (np.sort(plain, 1) != np.sort(np.argsort(-s, axis=1)[:, :r["top"]], 1)).any()      # the corrections do change choices
    tok = np.random.default_rng(i).choice(clear, 90).tolist()
    dec = m.open(cai, 128, 1, dt)
    for cuts in ([90], [9, 8, 3, 1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("what", ["gelu", "squash", "multiplier"])
def test_feed_forward_norms_and_multiplier(cai, tmp_path, what, dt):
    def edit(w):
        for n in w:
            if what == "squash" and n.endswith(".alpha"):
                w[n] = w[n] * (3 if dt == "f32" else 1.5)
            if what == "gelu" and n.endswith("norm1b"):
                w[n] = w[n] * 0
    m = Model(tmp_path, B.kconfig([B.klayer(B.ssd(), 48), B.klayer(B.rotary(), 31)], width=60, vocab=90, mult=2.3 if what == "multiplier" else 1.0), seed=5, edit=edit)
    tok = m.tokens(70, 2)
    dec = m.open(cai, 128, 1, dt)
    check(feed(dec, tok, [60, 1]), m.ref(tok), dt)
    dec.close()


@DT
@pytest.mark.parametrize("loop", [None, (0, 3, 1), (0, 3, 2), (2, 3, 3), (0, 1, 4), (1, 1, 5), (1, 2, 1), (0, 2, 2)], ids=str)
def test_repeated_layers(cai, tmp_path, loop, dt):
    """stretches at the start, in the middle, at the end, of one layer, empty and run once: the matrix comes before every pass, the
    first one too, and each pass has cache and state of its own"""
    cfg = B.kconfig([B.klayer(B.ssd(), 40), B.klayer(B.rotary(block=5)), B.klayer(B.rotary(heads=2, block=70), B.moe(experts=3, top=3))],
                    loop=loop and dict(start=loop[0], stop=loop[1], times=loop[2]), width=70)
    m = Model(tmp_path, cfg, seed=4)
    tok = m.tokens(100, 1)
    dec = m.open(cai, 128, 1, dt)
    for cuts in ([100], [40, 1], [33, 2, 5]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


# ---------------------------------------------------------------- whole models
@DT
@pytest.mark.parametrize("cuts", [[300], [1], [2], [3, 2, 65, 1, 1, 16, 17, 2], [64], [130, 1], [5, 9, 7]], ids=str)
def test_portions_and_decoding_agree_with_the_whole(cai, models, cuts, dt):
    m = models[dt]
    tok = m.tokens(150, 3)
    dec = m.open(cai, 192, 1, dt)
    check(feed(dec, tok, cuts), m.ref(tok), dt)
    assert dec.len() == 150 and dec.cache_rows() <= 128
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
    dec = m.open(cai, 320, 3, dt)
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
    assert dec.room(0) == 320                     # every page came back
    dec.close()


@pytest.mark.parametrize("rows", [2, 5, 8, 11])
def test_decoding_together_agrees_with_each_request_alone(cai, models, rows):
    """single tokens of many requests at different lengths: captured steps of up to eight rows, and wider ones"""
    m = models["f32"]
    reqs = [m.tokens(10 + 7 * b, 200 + b) for b in range(rows)]
    dec = m.open(cai, 64 * 2 * rows, rows)
    for b in range(rows):
        dec.step_batch([(b, reqs[b][:-4], [])])
    for k in range(4, 0, -1):
        lg = dec.step_batch([(b, reqs[b][len(reqs[b]) - k:][:1], [0]) for b in range(rows)])[1]
        check(lg, np.stack([m.ref(reqs[b])[-k] for b in range(rows)]), "f32")
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


# ---------------------------------------------------------------- block edges, far tokens
def pointed(block, heads=2):
    """token 400 + t asks for token t: keys carry a sign vector in the first half of the width, askers the same one in the second,
    W_k reads the first half and W_q the second, so that one score stands far above all others; two of 64 dimensions turn"""
    cfg = B.kconfig([B.klayer(B.rotary(heads=heads, kv_heads=1, dim=64, vdim=24, block=block, scale=0.15, rot=2, base=50.0))], width=128, vocab=800)

    def edit(w):
        sign = np.sign(np.random.default_rng(77).standard_normal((400, 64)))
        w["embed"] = np.zeros((800, 128)); w["embed"][:400, :64] = sign; w["embed"][400:, 64:] = sign
        w["l0.norm1"] = np.ones(128); w["l0.norm1.b"] = np.zeros(128); w["l0.norm1.alpha"] = np.asarray(1.5)
        w["l0.mix.k"] = np.eye(64, 128); w["l0.mix.q"] = np.concatenate([np.eye(64, 128, 64)] * heads) * 1.5
        w["l0.mix.q.b"] *= 0; w["l0.mix.k.b"] *= 0; w["l0.mix.v"] *= 3; w["l0.mix.o"] *= 2
    return cfg, edit


@DT
@pytest.mark.parametrize("block", [2, 3, 63, 64, 65, 100, 128, 200])
def test_block_edges(cai, tmp_path, block, dt):
    """a key that outweighs all others, the last one of the block before and the first one of the asker's own block: asked for in a
    prompt, in portions and decoded, where blocks and pages begin together and elsewhere"""
    cfg, edit = pointed(block)
    m = Model(tmp_path, cfg, seed=block, edit=edit)
    T = 330
    keys = np.random.default_rng(block).permutation(400)[:T]
    inside, outside = keys.copy(), keys.copy()
    starts = list(range(block, T, max(block, 37) if block < 37 else block))
    starts = [s // block * block for s in starts]
    rows_in, rows_out = [], []
    for s in starts:
        e = min(s + block, T) - 1                  # the block's last place
        if e > s:
            inside[e] = 400 + keys[s]; rows_in.append(e)         # sees its block's first key
        outside[s] = 400 + keys[s - 1]; rows_out.append(s)       # the block's first token does not see the key just before it
        if e > s + 1:
            outside[e] = 400 + keys[s - 1]; rows_out.append(e)
    # the oracle tells the edges apart: against blocks that begin one place earlier
    def shifted(tok):
        real = R.chunk_attention

        def moved(q, k, v, scale, size):
            T_, G, H = q.shape[0], k.shape[1], q.shape[1]
            i, j = np.arange(T_)[:, None], np.arange(T_)[None, :]
            seen = (j <= i) & ((i + 1) // size == (j + 1) // size) | (i == j)
            return np.stack([R.softmax_rows(np.where(seen, (q[:, h] @ k[:, h // (H // G)].T) * scale, -np.inf)) @ v[:, h // (H // G)] for h in range(H)], axis=1)
        R.chunk_attention = moved
        try:
            return R.forward(cfg, m.w, tok)
        finally:
            R.chunk_attention = real
    assert np.abs(shifted(outside) - m.ref(outside))[[r for r in rows_out if r in starts]].max(1).min() > 0.1
    dec = m.open(cai, 384, 1, dt)
    for tok in (inside, outside):
        for cuts in ([T], [60, 1], [2, 100, 3], [65, 63, 20, 1, 1, 40]):
            dec.reset()
            check(feed(dec, tok.tolist(), cuts), m.ref(tok), dt)
    dec.close()


@DT
def test_a_block_wider_than_the_pool(cai, tmp_path, dt):
    m = Model(tmp_path, B.kconfig([B.klayer(B.rotary(heads=3, kv_heads=1, dim=40, vdim=72, block=1 << 29, rot=40, base=1e4))]), seed=6)
    tok = m.tokens(384, 2)
    dec = m.open(cai, 384, 1, dt)
    for cuts in ([384], [300, 1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    with pytest.raises(cai.CaiError):
        dec.step_batch([(0, tok[:1], [0])])       # nothing of an unfinished block can be given back
    dec.close()


@DT
def test_far_positions_turn_right(cai, tmp_path, dt):
    """blocks at positions in the thousands: angles of many turns, and a pool of two blocks that carries the whole sequence"""
    m = Model(tmp_path, B.kconfig([B.klayer(B.rotary(block=64, dim=32, rot=32, base=3.0))], width=48, vocab=60), seed=8)
    tok = m.tokens(2500, 3)
    want = m.ref(tok)
    dec = m.open(cai, 256, 1, dt)
    check(feed(dec, tok, [100, 64, 90, 128, 30])[2300:], want[2300:], dt)
    dec.close()


@DT
def test_a_far_token_is_kept_by_the_state(cai, tmp_path, dt):
    """slow decay: what the first tokens wrote is read hundreds of tokens later"""
    cfg = B.kconfig([B.klayer(B.ssd(heads=2, vdim=24, state=48, groups=2, conv=1, norm_groups=1))], width=96, vocab=97)

    def edit(w):
        w["l0.mix.A_log"] = np.full(2, -7.0); w["l0.mix.dt_bias"] = np.full(2, 0.5); w["l0.mix.D"] *= 0
        emb = np.zeros((97, 96)); emb[:, :96] = np.sign(np.random.default_rng(4).standard_normal((97, 96)))
        w["embed"] = emb
        c = w["l0.mix.in"]
        c[192:288] = c[96:192]           # C reads what B writes: a token finds itself again
        w["l0.mix.conv.b"] *= 0
        w["l0.mix.conv"] = np.full((48 + 192, 1), 1.2)
    m = Model(tmp_path, cfg, seed=2, edit=edit)
    tok = np.random.default_rng(9).integers(10, 97, 500)
    tok[2] = 5; tok[450:] = np.where(tok[450:] == 5, 11, tok[450:]); tok[490] = 5
    want = m.ref(tok)
    lost = tok.copy(); lost[2] = 6
    assert err(R.forward(cfg, m.w, lost)[490:491], want[490:491]) > 5 * TOL["f32"]
    dec = m.open(cai, 64, 1, dt)
    for cuts in ([500], [470, 1], [33, 2]):
        dec.reset()
        check(feed(dec, tok.tolist(), cuts)[480:], want[480:], dt)
    dec.close()


# ---------------------------------------------------------------- long decoding, generation, sessions
@DT
def test_long_decoding_in_a_small_pool(cai, models, dt):
    """a pool of three pages carries 420 tokens: pages of finished blocks come back while the sequence runs on"""
    m = models[dt]
    tok = m.tokens(420, 8)
    dec = m.open(cai, 192, 1, dt)
    check(feed(dec, tok, [1]), m.ref(tok), dt)
    assert dec.cache_rows() <= 192
    dec.close()


def test_greedy_generation_through_every_entry_point(cai, models):
    m = models["f32"]
    prompts = [m.tokens(n, 70 + n) for n in (30, 3, 77, 12, 64)]
    dec = m.open(cai, 384, 2)
    want = []
    for p in prompts:
        want.append(greedy(dec, p, 40)); dec.reset()
        margin(m, p, want[-1])
    am, _ = dec.prefill(prompts[2])               # the captured device-side loop, across page and block borders
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


def test_snapshot_restore_and_fork(cai, models):
    m = models["f32"]
    tok = m.tokens(120, 31)
    dec = m.open(cai, 448, 2)
    feed(dec, tok[:80], [80])
    snap = dec.snapshot()
    dec.fork(0, 1)
    a = feed(dec, tok[80:], [7], 0)
    b = feed(dec, tok[80:], [1], 1)
    check(a, m.ref(tok)[80:], "f32"); check(b, m.ref(tok)[80:], "f32")
    dec.reset(1)
    dec.restore(snap, 1)
    check(feed(dec, tok[80:], [40], 1), m.ref(tok)[80:], "f32")
    h = dec.hidden_state(39)
    check((R.linear(m.w["head"], h.astype(np.float64)))[None], m.ref(tok)[-1:], "f32")
    cai.load().cai_kv_snap_destroy(snap)
    dec.close()


def test_layers_of_one_kind_only(cai, tmp_path):
    """no attention: a pool without pages; no state: a cache alone"""
    for i, mixer in enumerate((B.ssd(), B.rotary())):
        m = Model(tmp_path / str(i), B.kconfig([B.klayer(mixer, 30), B.klayer(mixer)], loop=dict(start=1, stop=2, times=2)), seed=i)
        tok = m.tokens(90, i)
        dec = m.open(cai, 128, 2)
        check(feed(dec, tok, [50, 3, 1], 1), m.ref(tok), "f32")
        dec.close()


@pytest.mark.parametrize("name, change", [
    ("heads", lambda c, w: c["layers"][0]["mixer"].update(heads=3, kv_heads=2)), ("type", lambda c, w: c["layers"][0].update(type="delta")),
    ("rot", lambda c, w: c["layers"][0]["mixer"]["rot"].update(dims=3)), ("rot.dims", lambda c, w: c["layers"][0]["mixer"]["rot"].update(dims=26)),
    ("mask.size", lambda c, w: c["layers"][0]["mixer"].pop("mask")), ("norm_groups", lambda c, w: c["layers"][1]["mixer"].update(norm_groups=7)),
    ("groups", lambda c, w: c["layers"][1]["mixer"].update(groups=3)), ("mix.in", lambda c, w: c["layers"][1]["mixer"].update(state=21)),
    ("router.top", lambda c, w: c["layers"][1]["mlp"]["router"].update(top=7)), ("e5", lambda c, w: w.pop("l1.mlp.e5.up")), ("e6", lambda c, w: c["layers"][1]["mlp"]["router"].update(experts=7, top=1) or
     w.update({"l1.mlp.router": np.zeros((7, 72)), "l1.mlp.correction": np.zeros(7)})), ("kind", lambda c, w: c["layers"][0]["mlp"].update(kind="other")),
    ("loop.in", lambda c, w: w.pop("loop.in")), ("residual_mult", lambda c, w: c.pop("residual_mult")), ("limit", lambda c, w: c["layers"][1]["mlp"]["shared"].pop("limit")),
    ("o.b", lambda c, w: w.pop("l0.mix.o.b")), ("conv", lambda c, w: c["layers"][1]["mixer"].update(conv=4))])
def test_loader_names_what_is_wrong(cai, tmp_path, name, change):
    cfg = B.kconfig([B.klayer(B.rotary(), 40), B.klayer(B.ssd(), B.moe())], loop=dict(start=0, stop=1, times=2))
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
