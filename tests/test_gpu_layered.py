"""The layered decoder on the device against the float64 oracle: every mechanism alone, prompts, decoding, portions, mixed
batches, reused pages and slots, window edges, long decoding, greedy and sampled generation through the scheduler."""
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


@pytest.fixture(scope="module")
def cai():
    return dev()


BIG = dict(layers=[B.layer(B.delta(heads=6, kv_heads=3, dim=20, vdim=36, conv=3)), B.layer(B.delta(heads=1, dim=70, vdim=130, conv=1), ff=None),
                   B.layer((B.attn(heads=6, kv_heads=2, dim=20, vdim=44, window=11), B.delta(heads=4, kv_heads=2, dim=9, vdim=17, conv=5))),
                   B.layer(B.delta(heads=3, dim=33, vdim=5, conv=2), ff=17)], width=100, vocab=211, loop=dict(start=1, stop=3, times=3))


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    return Model(tmp_path_factory.mktemp("layered"), B.config(**BIG), seed=11)


# ---------------------------------------------------------------- products over bfloat16 weights
@pytest.mark.parametrize("rows, cols", [(37, 50), (64, 64), (131, 520), (700, 1100), (9000, 96)])
def test_bf16_products(cai, rows, cols):
    rng = np.random.default_rng(rows)
    bits, w = B.to_bf16(rng.standard_normal((rows, cols)))
    w = w.reshape(rows, cols); bias = rng.standard_normal(rows).astype(np.float32)
    q = cai.QWeight(cai.BF16, rows, cols, bits, bias)
    assert np.array_equal(q.dequant_rows(3, 5), w[3:8].astype(np.float32))
    for n in (1, 2, 3, 5, 8, 9, 33, 70, 130):
        x = rng.standard_normal((n, cols)).astype(np.float32)
        want = x.astype(np.float64) @ w.T + bias
        if n <= 8:
            assert err(q.gemv(x), want) < 3e-6
            assert err(q.gemv(x, cai.ACT_RELU), np.maximum(want, 0)) < 3e-6
        assert err(q.gemm(x), want) < 3e-6


def test_bf16_matrices_stay_out_of_the_other_decoders(cai):
    bits, _ = B.to_bf16(np.zeros((64, 64)))
    q = cai.QWeight(cai.BF16, 64, 64, bits)
    with pytest.raises(cai.CaiError):
        q.ffn_gateup(np.zeros((1, 64), np.float32))


# ---------------------------------------------------------------- each mechanism alone
def only(part):
    def edit(w):
        for n in w:
            if part == "attention" and n.endswith("right.out"):
                w[n] = w[n] * 0
            if part == "channel delta" and n.endswith("left.out"):
                w[n] = w[n] * 0
            if part == "feed-forward" and n.endswith("norm1b"):
                w[n] = w[n] * 0
            if part == "squash" and n.endswith(".alpha"):
                w[n] = w[n] * 3
    return edit


MECHANISMS = {
    "delta": [("delta", B.delta(h, g, d, dv, t)) for h, g, d, dv, t in ((1, 1, 8, 8, 1), (4, 2, 64, 64, 4), (2, 2, 33, 70, 2), (3, 1, 129, 20, 6), (2, 1, 128, 128, 4), (1, 1, 256, 256, 3))],
    "channel delta": [("parallel", (B.attn(), B.delta(h, g, d, dv, t))) for h, g, d, dv, t in ((1, 1, 8, 8, 1), (4, 2, 32, 64, 4), (3, 3, 45, 131, 3), (2, 1, 200, 34, 5))],
    "attention": [("parallel", (B.attn(h, g, d, dv, w), B.delta())) for h, g, d, dv, w in
                  ((1, 1, 8, 8, 1), (4, 4, 24, 40, 2), (6, 2, 48, 96, 64), (8, 1, 130, 70, 65), (10, 2, 256, 256, 33), (2, 1, 64, 20, 1000), (3, 1, 17, 9, 63))],
    "feed-forward": [("delta", B.delta())], "squash": [("parallel", (B.attn(), B.delta()))],
}
CASES = [(m, i) for m, v in MECHANISMS.items() for i in range(len(v))]


@pytest.mark.parametrize("dt", ["f32", "bf16"])
@pytest.mark.parametrize("mech, i", CASES, ids=["%s-%d" % c for c in CASES])
def test_mechanism_alone(cai, tmp_path, mech, i, dt):
    kind, mixer = MECHANISMS[mech][i]
    m = Model(tmp_path, B.config([B.layer(mixer, ff=48 if mech == "feed-forward" else None)], width=40 + 8 * i, vocab=67), seed=i, edit=only(mech), rank_a=3 + 9 * i, rank_g=20)
    tok = m.tokens(90, i)
    dec = m.open(cai, 128, 1, dt)
    check(feed(dec, tok, [90]), m.ref(tok), dt)
    dec.reset()
    check(feed(dec, tok, [70, 1]), m.ref(tok), dt)
    dec.close()


# ---------------------------------------------------------------- whole models
@pytest.mark.parametrize("dt", ["f32", "bf16"])
@pytest.mark.parametrize("cuts", [[300], [1], [2], [3, 2, 65, 1, 1, 16, 17, 2], [64], [130, 1], [5, 9, 7]], ids=str)
def test_portions_and_decoding_agree_with_the_whole(cai, model, cuts, dt):
    tok = model.tokens(150, 3)
    dec = model.open(cai, 192, 1, dt)
    check(feed(dec, tok, cuts), model.ref(tok), dt)
    assert dec.len() == 150 and dec.cache_rows() <= 128
    dec.close()


@pytest.mark.parametrize("loop", [None, (0, 3, 2), (2, 3, 3), (0, 1, 4), (1, 1, 5), (1, 2, 1), (0, 2, 2)], ids=str)
def test_repeated_layers(cai, tmp_path, loop):
    """stretches at the start, in the middle, at the end, of one layer, empty and run once: each pass has cache and state of its own"""
    cfg = B.config([B.layer(B.delta()), B.layer((B.attn(window=5), B.delta(dim=12)), ff=None), B.layer((B.attn(heads=2, window=70), B.delta()))],
                   loop=loop and dict(start=loop[0], stop=loop[1], times=loop[2]))
    if loop is None:
        del cfg["loop"]
    m = Model(tmp_path, cfg, seed=4)
    tok = m.tokens(100, 1)
    dec = m.open(cai, 128)
    for cuts in ([100], [40, 1], [33, 2, 5]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), "f32")
    dec.close()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_a_window_wider_than_the_pool(cai, tmp_path, dt):
    m = Model(tmp_path, B.config([B.layer((B.attn(heads=3, kv_heads=1, dim=40, vdim=72, window=1 << 29), B.delta()))]), seed=6)
    tok = m.tokens(384, 2)
    dec = m.open(cai, 384, 1, dt)
    for cuts in ([384], [300, 1]):
        dec.reset()
        check(feed(dec, tok, cuts), m.ref(tok), dt)
    dec.close()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_first_tokens(cai, model, dt):
    dec = model.open(cai, 64, 1, dt)
    for n in range(1, 7):
        tok = model.tokens(n, 40 + n)
        dec.reset()
        check(feed(dec, tok, [n]), model.ref(tok), dt)
        dec.reset()
        check(feed(dec, tok, [1]), model.ref(tok), dt)
    dec.close()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_mixed_batches_with_reused_slots_and_pages(cai, model, dt):
    """eight requests over three slots; portions of some beside single tokens of others; a pool that the live ones nearly fill"""
    rng = np.random.default_rng(5)
    lens = [70, 9, 131, 1, 64, 33, 90, 200]
    reqs = [model.tokens(n, 100 + i) for i, n in enumerate(lens)]
    dec = model.open(cai, 320, 3, dt)
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
        check(np.concatenate(got[i]), model.ref(reqs[i]), dt)
    assert dec.room(0) == 320                     # every page came back
    dec.close()


def test_batches_agree_with_each_request_alone_to_rounding(cai, model):
    reqs = [model.tokens(n, 60 + n) for n in (21, 90, 2, 1)]
    dec = model.open(cai, 512, 4)
    alone = []
    for r in reqs:
        alone.append(feed(dec, r, [len(r)])); dec.reset()
    lg = dec.step_batch([(3 - i, r, range(len(r))) for i, r in enumerate(reqs)])[1]
    assert err(lg.astype(np.float64), np.concatenate(alone).astype(np.float64)) < 4e-6
    dec.close()


# ---------------------------------------------------------------- window edges
def pointed(window, heads=2):
    """token 400 + t asks for token t: keys carry a sign vector in the first half of the width, askers the same one in the second,
    W_k reads the first half and W_q the second, so that one score stands far above all others"""
    cfg = B.config([B.layer((B.attn(heads=heads, kv_heads=1, dim=64, vdim=24, window=window, scale=0.15), B.delta()), ff=None)], width=128, vocab=800)

    def edit(w):
        sign = np.sign(np.random.default_rng(77).standard_normal((400, 64)))
        w["embed"] = np.zeros((800, 128)); w["embed"][:400, :64] = sign; w["embed"][400:, 64:] = sign
        w["l0.norm1"] = np.ones(128); w["l0.norm1.b"] = np.zeros(128)
        w["l0.mix.left.k"] = np.eye(64, 128); w["l0.mix.left.q"] = np.concatenate([np.eye(64, 128, 64)] * heads)
        w["l0.mix.left.q.norm"] = np.full(64, 1.0); w["l0.mix.left.k.norm"] = np.full(64, 1.5)
        w["l0.mix.right.out"] = w["l0.mix.right.out"] * 0
    return cfg, edit


@pytest.mark.parametrize("dt", ["f32", "bf16"])
@pytest.mark.parametrize("window", [2, 3, 63, 64, 65, 128, 200, 257])
def test_window_edges(cai, tmp_path, window, dt):
    """a key that outweighs all others, just inside and just outside the window of the token that asks for it: in a prompt, in
    portions and decoded, at page borders and elsewhere"""
    cfg, edit = pointed(window)
    m = Model(tmp_path, cfg, seed=window, edit=edit)
    T = 330
    keys = np.random.default_rng(window).permutation(400)[:T]
    places = [p for p in (0, 5, 59, 63, 64, 70, 127, 128) if p + window < T]
    if window == 2:
        places = places[:-1]
    inside, outside = keys.copy(), keys.copy()
    for p in places:
        inside[p + window - 1] = 400 + keys[p]; outside[p + window] = 400 + keys[p]
    # the oracle tells the edge apart: seen from the last place of the window, not from the next one
    wider = json.loads(json.dumps(cfg)); wider["layers"][0]["mixer"]["left"]["mask"]["size"] = window + 1
    rows = [p + window for p in places if not (outside[p] >= 400)]
    apart = np.abs(R.forward(wider, m.w, outside) - m.ref(outside))[rows].max(1)
    assert apart.min() > 0.1
    dec = m.open(cai, 384, 1, dt)
    for tok in (inside, outside):
        for cuts in ([T], [60, 1], [2, 100, 3], [65, 63, 20, 1, 1, 40]):
            dec.reset()
            check(feed(dec, tok.tolist(), cuts), m.ref(tok), dt)
    dec.close()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_a_far_token_is_kept_by_the_state(cai, tmp_path, dt):
    """slow decay and full-strength writes: what the first tokens wrote is read hundreds of tokens later"""
    cfg = B.config([B.layer(B.delta(heads=2, kv_heads=2, dim=48, vdim=24, conv=1), ff=None)], width=96, vocab=97)

    def edit(w):
        w["l0.mix.dt_bias"] = np.full(2, -9.0); w["l0.mix.k"] = w["l0.mix.q"]; w["l0.mix.b"] = w["l0.mix.b"] * 0.05
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


# ---------------------------------------------------------------- long decoding, generation, scheduler
@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_long_decoding_in_a_small_pool(cai, model, dt):
    """a pool of two pages carries 420 tokens: pages behind the window come back while the sequence runs on"""
    tok = model.tokens(420, 8)
    dec = model.open(cai, 128, 1, dt)
    check(feed(dec, tok, [1]), model.ref(tok), dt)
    assert dec.cache_rows() <= 128
    dec.close()


def dec_tail(model, tokens, n):
    out = []
    for _ in range(n):
        out.append(int(model.ref(tokens + out)[-1].argmax()))
    return out


def test_sampled_requests_do_not_depend_on_their_company(cai, model):
    prompts = [model.tokens(n, 20 + n) for n in (8, 40, 21)]
    dec = model.open(cai, 256, 3)
    sched = cai.Scheduler(dec)
    alone = []
    for k, p in enumerate(prompts):
        i = sched.submit(p, 25, temperature=1.3, top_k=12, seed=k + 1); sched.run(); alone.append(sched.result(i)[0])
    ids = [sched.submit(p, 25, temperature=1.3, top_k=12, seed=k + 1) for k, p in enumerate(prompts)]
    sched.run()
    assert [sched.result(i)[0] for i in ids] == alone
    assert len(set(map(tuple, alone))) == 3 and any(a != greedy_of(dec, p) for a, p in zip(alone, prompts))
    # a drawn token is one of the most probable ones
    lg = model.ref(prompts[0] + alone[0][:-1])[len(prompts[0]) - 1:]
    for row, t in zip(lg, alone[0]):
        assert t in np.argsort(row)[-14:]
    sched.close(); dec.close()


def greedy_of(dec, p):
    dec.reset()
    return greedy(dec, p, 25)


def test_the_scheduler_serves_the_uniform_decoders_too(cai):
    from helpers.fixtures_io import ref_path
    dec = cai.Decoder.load(ref_path("tiny_llama_f32.gguf"), 32, 2, cai.DTYPE_F32)
    prompts = [[1, 5, 2, 7], [3, 0, 6], [4, 4, 1, 2, 3, 5, 6, 7, 0, 1, 2]]
    want = []
    for p in prompts:
        dec.reset()
        out = [dec.prefill(p)[0]]
        while len(out) < 6:
            out.append(int(dec.step([out[-1]], [len(p) + len(out) - 1])[0][0]))
        want.append(out)
    sched = cai.Scheduler(dec, portion=5)
    ids = [sched.submit(p, 6) for p in prompts]
    sched.run()
    assert [sched.result(i)[0] for i in ids] == want
    # inner rows of a long entry
    dec.reset()
    lg = dec.step_batch([(0, prompts[2], [0, 5, 10])])[1]
    dec.reset()
    one = np.array([dec.step([t], [p])[1][0] for p, t in enumerate(prompts[2])])
    assert err(lg, one[[0, 5, 10]]) < 1e-5
    sched.close(); dec.close()


# ---------------------------------------------------------------- sessions
def test_snapshot_restore_fork_and_hidden_state(cai, model):
    tok = model.tokens(120, 31)
    dec = model.open(cai, 384, 2)
    feed(dec, tok[:80], [80])
    snap = dec.snapshot()
    dec.fork(0, 1)
    a = feed(dec, tok[80:], [7], 0)
    b = feed(dec, tok[80:], [1], 1)
    check(a, model.ref(tok)[80:], "f32"); check(b, model.ref(tok)[80:], "f32")
    dec.reset(1)
    dec.restore(snap, 1)
    assert dec.len(1) == 80
    check(feed(dec, tok[80:], [40], 1), model.ref(tok)[80:], "f32")
    h = dec.hidden_state(39)
    check((R.linear(model.w["head"], h.astype(np.float64)))[None], model.ref(tok)[-1:], "f32")
    t, p = dec.candidates(5, row=39)
    assert t.tolist() == np.argsort(-model.ref(tok)[-1])[:5].tolist()
    with pytest.raises(cai.CaiError):
        dec.truncate(100, 1)                      # recurrent state cannot be taken back
    dec.truncate(0, 1)
    assert dec.len(1) == 0
    cai.load().cai_kv_snap_destroy(snap)
    dec.close()


def test_a_full_pool_refuses_a_step_and_changes_nothing(cai, tmp_path):
    m = Model(tmp_path, B.config([B.layer((B.attn(window=500), B.delta()))]), seed=3)
    tok = m.tokens(140, 4)
    dec = m.open(cai, 128, 2)
    a = feed(dec, tok[:60], [60], 0)
    feed(dec, tok[:50], [50], 1)
    with pytest.raises(cai.CaiError):
        dec.step_batch([(0, tok[60:70], [9]), (1, tok[50:60], [9])])
    assert dec.len(0) == 60 and dec.len(1) == 50 and dec.room(0) == 4
    b = feed(dec, tok[60:64], [2], 0)
    dec.reset(1)
    c = feed(dec, tok[64:128], [64], 0)
    check(np.concatenate([a, b, c]), m.ref(tok[:128]), "f32")
    with pytest.raises(cai.CaiError):
        dec.step_batch([(0, tok[128:129], [0])])
    for bad in ([(0, [999], [0])], [(2, [1], [0])], [(0, [1], []), (0, [1], [])]):
        with pytest.raises(cai.CaiError):
            dec.step_batch(bad)
    for f in (lambda: dec.set_eviction(1, 2), lambda: dec.set_rope_scaling(1, 2.0), lambda: dec.profile(1)):
        with pytest.raises(cai.CaiError):
            f()
    sched = cai.Scheduler(dec)
    with pytest.raises(cai.CaiError):
        sched.submit(tok, 10)
    sched.close(); dec.close()


@pytest.mark.parametrize("name, change", [
    ("heads", lambda c, w: c["layers"][0]["mixer"].update(heads=3, kv_heads=2)), ("type", lambda c, w: c["layers"][0].update(type="other")),
    ("mlp.gate", lambda c, w: c["layers"][0]["mlp"].update(ff=57)), ("kind", lambda c, w: c["layers"][0]["mlp"].update(kind="other")),
    ("head", lambda c, w: w.pop("head")), ("dim", lambda c, w: c["layers"][0]["mixer"].pop("dim")), ("loop.stop", lambda c, w: c["loop"].update(stop=9)),
    ("alpha", lambda c, w: w.pop("l0.norm2.alpha")), ("eps", lambda c, w: c["norm"].clear())])
def test_loader_names_what_is_wrong(cai, tmp_path, name, change):
    cfg = B.config([B.layer(B.delta())])
    w = B.weights(cfg)
    change(cfg, w)
    B.write(str(tmp_path), cfg, w)
    with pytest.raises(cai.CaiError) as e:
        cai.Decoder.load(str(tmp_path), 64)
    assert name in str(e.value)


# ---------------------------------------------------------------- programs
def test_command_line_generation(cai, model):
    prompts = [model.tokens(9, 1), model.tokens(20, 2)]
    dec = model.open(cai, 128)
    want = []
    for p in prompts:
        want.append(greedy(dec, p, 7)); dec.reset()
    dec.close()
    exe = os.path.join(ROOT, "neural-api_amd", "host", "caihip_run")
    one = subprocess.run([exe, model.folder, "7", "--dtype", "float32"] + [str(t) for t in prompts[0]], capture_output=True, text=True, timeout=100)
    assert one.returncode == 0 and [int(t) for t in one.stdout.splitlines()[0].split()] == want[0], one.stdout + one.stderr
    both = subprocess.run([exe, model.folder, "7", "--dtype", "float32", "--portion", "4"] + [str(t) for t in prompts[0]] + ["--"] + [str(t) for t in prompts[1]],
                          capture_output=True, text=True, timeout=100)
    assert [[int(t) for t in s.split()] for s in both.stdout.splitlines()] == want, both.stdout + both.stderr


@pytest.mark.parametrize("dt, name", [("f32", "float32"), ("bf16", "bfloat16")])
def test_trace_replay(cai, model, tmp_path, dt, name):
    a, b = model.tokens(50, 6), model.tokens(30, 7)
    steps = [dict(step=0, entries=[dict(id="x", tokens=a[:40], want=[39, 0])], end=[]), dict(step=1, entries=[dict(id="y", tokens=b[:2], want=[])], end=[]),
             dict(step=2, entries=[dict(id="y", tokens=b[2:], want=[27]), dict(id="x", tokens=a[40:41], want=[0])], end=["y"]),
             dict(step=3, entries=[dict(id="z", tokens=b, want=[29]), dict(id="x", tokens=a[41:], want=[8, 7])], end=["x", "z"])]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", model.folder, "--dtype", name, "--out", str(tmp_path), "--max-tokens", "128"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done %d" % i for i in range(4)], r.stderr
    got = lambda i: np.fromfile(tmp_path / ("%d.f32" % i), "<f4").reshape(-1, model.cfg["vocab"])
    check(got(0), model.ref(a)[[39, 0]], dt)
    assert not os.path.exists(tmp_path / "1.f32")
    check(got(2), np.stack([model.ref(b)[29], model.ref(a)[40]]), dt)
    check(got(3), np.stack([model.ref(b)[29], model.ref(a)[49], model.ref(a)[48]]), dt)
