"""A layered model on disk beside its float64 oracle, and how the device tests feed and compare it."""
import numpy as np

from helpers import layered_build as B
from helpers import layered_ref as R

TOL = {"f32": 2e-5, "bf16": 4e-2}          # rms of the logit difference over the rms of the logits


class Model:
    def __init__(self, folder, cfg, seed=0, edit=None, **kw):
        w = B.weights(cfg, seed, **kw)
        if edit:
            edit(w)
        self.cfg, self.folder = cfg, str(folder)
        self.w = B.write(self.folder, cfg, w)
        self.cache = {}

    def ref(self, tokens):
        key = tuple(int(t) for t in tokens)
        if key not in self.cache:
            self.cache[key] = R.forward(self.cfg, self.w, np.array(key))
        return self.cache[key]

    def open(self, cai, max_tokens, max_seq=1, dt="f32"):
        return cai.Decoder.load(self.folder, max_tokens, max_seq, cai.DTYPE_F32 if dt == "f32" else cai.DTYPE_BF16)

    def tokens(self, n, seed):
        return np.random.default_rng(seed).integers(0, self.cfg["vocab"], n).tolist()


def err(got, want):
    d = got - want
    return float(np.sqrt((d * d).mean(-1)).max() / np.sqrt((want * want).mean()))


def check(got, want, dt):
    e = err(np.asarray(got, np.float64), want)
    assert e < TOL[dt], "logits differ by %.2e of their size" % e


def feed(dec, tokens, cuts, seq=0):
    """logits of every token of one request brought in portions of the given sizes (the last size repeats)"""
    out, i, k = [], 0, 0
    while i < len(tokens):
        n = min(cuts[min(k, len(cuts) - 1)], len(tokens) - i)
        out.append(dec.step_batch([(seq, tokens[i:i + n], range(n))])[1])
        i += n; k += 1
    return np.concatenate(out)


def greedy(dec, prompt, n, seq=0):
    out = [int(dec.step_batch([(seq, prompt, [len(prompt) - 1])])[0][0])]
    while len(out) < n:
        out.append(int(dec.step_batch([(seq, out[-1:], [0])])[0][0]))
    return out


def margin(model, prompt, out):
    """smallest lead of the chosen token in the oracle's logits along a greedy run"""
    lg = model.ref(list(prompt) + out[:-1])[len(prompt) - 1:]
    top = np.sort(lg, axis=1)
    assert [int(r.argmax()) for r in lg] == out or float((top[:, -1] - top[:, -2]).min()) < 1e-3
    return lg


def test_greedy_generation_through_every_entry_point(cai, model):
    prompts = [model.tokens(n, 70 + n) for n in (30, 3, 77, 12, 64)]
    dec = model.open(cai, 256, 2)
    want = []
    for p in prompts:
        want.append(greedy(dec, p, 40)); dec.reset()
        margin(model, p, want[-1])
    # captured device-side loop, across page borders
    am, _ = dec.prefill(prompts[2])
    assert [am] + dec.generate(am, 77, 39).tolist() == want[2]
    assert [t for t in dec.generate_lookup(prompts[2] + want[2], 3)[0].tolist()] == dec_tail(model, prompts[2] + want[2], 3)
    dec.reset()
    # step, window and prefill forms of the session
    am, lg = dec.step_window(prompts[1], 0)
    check(lg, model.ref(prompts[1]), "f32")
    am, lg = dec.step([want[1][0]], [3])
    check(lg, model.ref(prompts[1] + want[1][:1])[3:], "f32")
    dec.reset()
    # the scheduler, with portions shorter than the prompts and more requests than sequences
    sched = cai.Scheduler(dec, max_rows=24, portion=10)
    ids = [sched.submit(p, 40) for p in prompts]
    live, waiting = sched.step()
    assert live == 2 and waiting == 3
    sched.run()
    assert [sched.result(i) for i in ids] == [(w, True) for w in want]
    # an end token stops a request, a dropped request frees its place
    stop = want[0][5]
    a = sched.submit(prompts[0], 40, eos=stop); b = sched.submit(prompts[1], 40); sched.step(); sched.drop(b); sched.run()
    assert sched.result(a)[0] == want[0][:want[0].index(stop) + 1]
    sched.close(); dec.close()
