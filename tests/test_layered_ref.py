"""The layered decoder's float64 oracle against independent statements of the same mechanisms, and the registry's refusals."""
import json
import os

import numpy as np
import pytest

from helpers import layered_build as B
from helpers import layered_ref as R


def test_delta_rule_without_decay_recalls_what_was_written():
    # orthogonal keys, full write strength: reading with a key returns the value last written under it
    k = np.eye(4)[None][:, [0, 1, 2, 0, 3]].transpose(1, 0, 2)
    v = np.arange(5 * 3, dtype=float).reshape(5, 1, 3)
    q = np.eye(4)[[0, 0, 1, 0, 2]][:, None]
    o = R.delta_rule(q, k, v, np.ones((5, 1, 4)), np.ones((5, 1)))
    assert np.allclose(o[:, 0], [v[0, 0], v[0, 0], v[1, 0], v[3, 0], v[2, 0]])


def test_delta_rule_is_a_product_of_state_transitions():
    rng = np.random.default_rng(1)
    T, d, dv = 6, 5, 4
    q, k, v = rng.standard_normal((T, 1, d)), R.unit(rng.standard_normal((T, 1, d))), rng.standard_normal((T, 1, dv))
    g, b = rng.uniform(0.2, 1.0, (T, 1, d)), rng.uniform(0, 1, (T, 1))
    S, want = np.zeros((d, dv)), []
    for t in range(T):
        kk = k[t, 0][:, None]
        S = (np.eye(d) - b[t, 0] * kk @ kk.T) @ np.diag(g[t, 0]) @ S + b[t, 0] * kk @ v[t]
        want.append(q[t, 0] @ S)
    assert np.allclose(R.delta_rule(q, k, v, g, b)[:, 0], want)


def test_convolution_is_causal_and_its_last_tap_is_the_current_token():
    x = np.random.default_rng(2).standard_normal((7, 3))
    w = np.zeros((3, 4)); w[:, 3] = [1, 0, 0]; w[:, 1] = [0, 1, 0]; w[:, 0] = [0, 0, 1]
    y = R.causal_conv(x, w)
    assert np.allclose(y[:, 0], x[:, 0])
    assert np.allclose(y[2:, 1], x[:-2, 1]) and np.all(y[:2, 1] == 0)
    assert np.allclose(y[3:, 2], x[:-3, 2]) and np.all(y[:3, 2] == 0)


@pytest.mark.parametrize("window", [1, 3, 50])
def test_window_attention_sees_exactly_its_window(window):
    rng = np.random.default_rng(3)
    T = 9
    q, k, v = rng.standard_normal((T, 4, 6)), rng.standard_normal((T, 2, 6)), rng.standard_normal((T, 2, 5))
    o = R.window_attention(q, k, v, 0.3, window)
    for i in range(T):
        lo = max(0, i - window + 1)
        for h in range(4):
            s = np.exp(0.3 * k[lo:i + 1, h // 2] @ q[i, h])
            assert np.allclose(o[i, h], (s / s.sum()) @ v[lo:i + 1, h // 2])


def test_run_order_of_repeated_layers():
    cfg = dict(layers=[None] * 5, loop=dict(start=1, stop=3, times=3))
    assert R.run_order(cfg) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False), (4, False)]
    assert R.run_order(dict(layers=[None] * 2)) == [(0, False), (1, False)]


def test_oracle_is_sensitive_to_what_it_checks():
    """a window off by one, a lost state, a wrong group or a missing repeat moves the logits well beyond the tests' tolerances"""
    cfg = B.config([B.layer(B.delta()), B.layer((B.attn(), B.delta(dim=12)))], loop=dict(start=0, stop=2, times=2))
    w = {n: B.to_bf16(a)[1].reshape(np.shape(a)) for n, a in B.weights(cfg, 5).items()}
    tok = np.random.default_rng(6).integers(0, cfg["vocab"], 40)
    base = R.forward(cfg, w, tok)
    for change in (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=10), lambda c: c["loop"].update(times=1),
                   lambda c: c["layers"][1]["mixer"]["left"].update(scale=0.25), lambda c: c["norm"].update(eps=0.1)):
        other = json.loads(json.dumps(cfg)); change(other)
        assert np.abs(R.forward(other, w, tok) - base).max() > 2e-2
    assert np.abs(R.forward(cfg, w, tok[1:])[-1] - base[-1]).max() > 2e-5      # a token well before every window still counts


# ---------------------------------------------------------------- Kiruvik's mechanisms
def test_rotation_turns_pairs_by_relative_position():
    rng = np.random.default_rng(4)
    x, y = rng.standard_normal((1, 1, 12)), rng.standard_normal((1, 1, 12))
    rot = lambda z, p: R.rotate_half(z, 50.0, 8, p)
    assert np.allclose(rot(x, 0), x) and np.allclose(rot(x, 9)[..., 8:], x[..., 8:])
    assert np.allclose((rot(x, 7) * rot(y, 3)).sum(), (rot(x, 104) * rot(y, 100)).sum())       # scores depend on the distance alone
    z = np.zeros((1, 1, 12)); z[0, 0, 1] = 1.0
    a = 5 * 50.0 ** (-2 / 8)
    assert np.allclose(rot(z, 5)[0, 0, [1, 5]], [np.cos(a), np.sin(a)])                         # dimension i pairs with i + dims / 2
    many = rng.standard_normal((6, 2, 12))
    assert np.allclose(R.rotate_half(many, 50.0, 8)[4], R.rotate_half(many[4:5], 50.0, 8, 4)[0])


@pytest.mark.parametrize("size", [1, 3, 4, 50])
def test_block_attention_sees_its_own_block_up_to_itself(size):
    rng = np.random.default_rng(3)
    T = 9
    q, k, v = rng.standard_normal((T, 4, 6)), rng.standard_normal((T, 2, 6)), rng.standard_normal((T, 2, 5))
    o = R.chunk_attention(q, k, v, 0.3, size)
    for i in range(T):
        lo = i - i % size
        for h in range(4):
            s = np.exp(0.3 * k[lo:i + 1, h // 2] @ q[i, h])
            assert np.allclose(o[i, h], (s / s.sum()) @ v[lo:i + 1, h // 2])


def test_state_space_recurrence_is_a_decayed_sum_over_the_past():
    rng = np.random.default_rng(5)
    T, H, P, G, N = 7, 4, 3, 2, 5
    x, B_, C = rng.standard_normal((T, H, P)), rng.standard_normal((T, G, N)), rng.standard_normal((T, G, N))
    dt, rate, D = rng.uniform(0.1, 1, (T, H)), rng.uniform(0.1, 2, H), rng.standard_normal(H)
    y = R.ssd_recurrence(x, B_, C, dt, rate, D)
    for t in range(T):
        for h in range(H):
            g = h // 2
            want = D[h] * x[t, h] + sum((C[t, g] @ B_[s, g]) * np.exp(-rate[h] * dt[s + 1:t + 1, h].sum()) * dt[s, h] * x[s, h] for s in range(t + 1))
            assert np.allclose(y[t, h], want)


def test_routing_chooses_with_the_correction_and_weighs_without_it():
    z = np.log(np.array([[0.4, 0.3, 0.2, 0.1]]))
    assert np.allclose(R.route(z, np.zeros(4), 2, 3.0), [[3 * 0.4 / 0.7, 3 * 0.3 / 0.7, 0, 0]])
    assert np.allclose(R.route(z, np.array([0, 0, 0, 0.5]), 2, 3.0), [[3 * 0.4 / 0.5, 0, 0, 3 * 0.1 / 0.5]])


def test_clamped_expert_and_gelu():
    one = np.eye(1)
    w = {"gate": one, "up": one, "down": one}
    f = lambda h, limit: R.clamped_expert(w, "", np.array([[h]]), limit)[0, 0]
    act = lambda g, u: g / (1 + np.exp(-1.702 * g)) * (u + 1)
    assert np.isclose(f(0.5, 2.0), act(0.5, 0.5)) and np.isclose(f(3.0, 2.0), act(2.0, 2.0)) and np.isclose(f(-3.0, 2.0), act(-3.0, -2.0))      # the gate has no lower bound
    assert np.isclose(R.gelu_tanh(np.array(1.0)), 0.841192, atol=1e-6) and np.isclose(R.gelu_tanh(np.array(-2.0)), -0.045402, atol=1e-6)
    x = np.arange(1.0, 7.0)[None]
    assert np.allclose(R.group_rms_norm(x, 3, 0.0)[0, :2], x[0, :2] / np.sqrt(2.5))


def test_kiruvik_oracle_is_sensitive_to_what_it_checks():
    """every constant of the configuration, a lost state and a pass without its matrix move the logits well beyond the tests' tolerances"""
    cfg = B.kconfig([B.klayer(B.ssd(), B.moe()), B.klayer(B.rotary(), 40), B.klayer(B.ssd(heads=3, norm_groups=1, groups=1))], loop=dict(start=1, stop=3, times=2))
    w = {n: B.to_bf16(a)[1].reshape(np.shape(a)) for n, a in B.weights(cfg, 5).items()}
    tok = np.random.default_rng(6).integers(0, cfg["vocab"], 40)
    base = R.forward(cfg, w, tok)
    at = lambda c, i: c["layers"][i]
    for change in (lambda c: at(c, 1)["mixer"]["mask"].update(size=10), lambda c: c["loop"].update(times=1), lambda c: c["loop"].update(start=0), lambda c: c.update(residual_mult=0.85),
                   lambda c: at(c, 1)["mixer"].update(scale=0.25), lambda c: at(c, 1)["mixer"]["rot"].update(base=600.0), lambda c: at(c, 1)["mixer"]["rot"].update(dims=12),
                   lambda c: c["norm"].update(eps=0.1), lambda c: at(c, 0)["mixer"].update(norm_groups=1), lambda c: at(c, 0)["mlp"]["router"].update(top=3),
                   lambda c: at(c, 0)["mlp"]["router"].update(scale=2.0), lambda c: at(c, 0)["mlp"]["expert"].update(limit=1.0), lambda c: at(c, 0)["mlp"]["shared"].update(limit=1.1)):
        other = json.loads(json.dumps(cfg)); change(other)
        assert np.abs(R.forward(other, w, tok) - base).max() > 1e-2
    for name in ("l0.mix.conv.b", "l0.mix.D", "l0.mix.dt_bias", "l1.mix.q.b", "l1.mix.k.b", "l1.mix.v.b", "l1.mix.o.b", "l0.mlp.correction", "loop.in"):
        other = dict(w); other[name] = w[name] * 0.5
        assert np.abs(R.forward(cfg, other, tok) - base).max() > 1e-2, name


# ---------------------------------------------------------------- Gamanex's mechanisms
def test_sigmoid_attention_weighs_each_key_for_itself():
    rng = np.random.default_rng(11)
    T, r1, r2, b = 7, np.array([0.5, 0.0, 1.3, 0.2]), np.array([0.3, 1.0, 2.0, 0.7]), np.array([-1.0, 0.5, 0.0, -2.0])
    q, k, v = rng.standard_normal((T, 4, 6)), rng.standard_normal((T, 2, 6)), rng.standard_normal((T, 2, 5))
    o = R.sigmoid_attention(q, k, v, 0.3, r1, r2, b)
    for i in range(T):
        for h in range(4):
            want = sum(v[j, h // 2] / (1 + np.exp(-(0.3 * k[j, h // 2] @ q[i, h] + b[h])) * (1 + r2[h] * (i - j)) ** r1[h]) for j in range(i + 1))
            assert np.allclose(o[i, h], want)
    # nothing is shared between the keys: another key more changes the sum by its own part alone
    far = R.sigmoid_attention(q[:, :, :], np.concatenate([k[:-1], k[-1:] * 9]), v, 0.3, r1, r2, b)
    assert np.allclose(far[:-1], o[:-1]) and not np.allclose(far[-1], o[-1])


def test_query_temperature_steps_with_the_position():
    t = R.query_temperature(np.arange(12), 0.5, 4)
    assert np.allclose(t[:3], 1.0) and np.allclose(t[3:7], 1 + 0.5 * np.log(2)) and np.allclose(t[7:11], 1 + 0.5 * np.log(3)) and np.isclose(t[11], 1 + 0.5 * np.log(4))
    assert np.allclose(R.query_temperature(np.arange(3), 1.0, 1), 1 + np.log([2, 3, 4]))


def test_routing_among_the_chosen():
    z = np.array([[1.0, 3.0, -2.0, 2.0]])
    e = np.exp([3.0, 2.0])
    assert np.allclose(R.route_among_chosen(z, 2), [[0, e[0] / e.sum(), 0, e[1] / e.sum()]])
    assert np.allclose(R.route_among_chosen(z, 1), [[0, 1, 0, 0]]) and np.allclose(R.route_among_chosen(z, 4), R.softmax_rows(z))


def test_gamanex_oracle_is_sensitive_to_what_it_checks():
    """every constant and every small tensor, a far token, another layer's keys: each moves the logits well beyond the tests' tolerances"""
    cfg = B.gconfig([B.glayer(B.sig(), 40), B.glayer(B.sig(heads=6, kv_heads=3, dim=10), B.gmoe()), B.glayer(B.sig(kv_from=0, every=5, coef=0.7), B.gmoe(top=3)), B.glayer(B.sig())])
    w = {n: B.to_bf16(a)[1].reshape(np.shape(a)) for n, a in B.weights(cfg, 5).items()}
    tok = np.random.default_rng(6).integers(0, cfg["vocab"], 40)
    base = R.forward(cfg, w, tok)
    at = lambda c, i: c["layers"][i]
    for change in (lambda c: at(c, 0)["mixer"].update(scale=0.25), lambda c: at(c, 2)["mixer"]["q_temp"].update(coef=0.8), lambda c: at(c, 0)["mixer"]["q_temp"].update(every=8),
                   lambda c: c["norm"].update(eps=0.1), lambda c: c.update(logit_scale=0.75), lambda c: at(c, 1)["mlp"]["router"].update(top=3)):
        other = json.loads(json.dumps(cfg)); change(other)
        assert np.abs(R.forward(other, w, tok) - base).max() > 1e-2
    for name in w:
        if not name.startswith("l1.mlp.e") and not name.startswith("l2.mlp.e"):
            other = dict(w); other[name] = w[name] * 0.5
            assert np.abs(R.forward(cfg, other, tok) - base).max() > 1e-2 or name in ("l0.mix.k", "l1.mix.k", "l3.mix.k", "l0.mix.q", "l1.mix.q", "l2.mix.q", "l3.mix.q"), name   # (a norm takes these back)
    other = dict(w); other["embed"] = w["embed"].copy(); other["embed"][tok[0]] += 1.0
    first_only = tok.copy(); first_only[1:][first_only[1:] == tok[0]] = (tok[0] + 1) % cfg["vocab"]
    assert np.abs(R.forward(cfg, other, first_only)[-1] - R.forward(cfg, w, first_only)[-1]).max() > 1e-2
    own = json.loads(json.dumps(cfg)); del own["layers"][2]["mixer"]["kv_from"]
    ow = dict(w, **{"l2.mix." + n: w["l3.mix." + n] for n in ("k", "v", "k.norm")})
    assert np.abs(R.forward(own, ow, tok) - base).max() > 1e-2


# ---------------------------------------------------------------- Zenorax's mechanisms
def test_turn_rates_slow_down_the_slow_pairs():
    f, amp = R.turn_rates(16, 100.0)
    assert np.allclose(f, 100.0 ** (-np.arange(8) / 8)) and amp == 1.0
    assert np.allclose(R.turn_rates(16, 100.0, linear=2.5)[0], f / 2.5)
    g, amp = R.turn_rates(16, 100.0, yarn=dict(factor=4.0, original=200, fast=10.0, slow=2.0))
    turns = 200 * f / (2 * np.pi)                       # over the original length
    assert np.allclose(g[turns > 14], f[turns > 14]) and np.allclose(g[turns < 1.5], f[turns < 1.5] / 4) and np.isclose(amp, 1 + 0.1 * np.log(4))
    between = (g < f * 0.999) & (g > f / 4 * 1.001)
    assert between.any() and not between[0] and not between[-1] and np.all(np.diff(g / f) <= 1e-12)


def test_rotation_of_neighbours_and_halves():
    rng = np.random.default_rng(4)
    x, y, rates = rng.standard_normal((1, 1, 12)), rng.standard_normal((1, 1, 12)), np.array([1.0, 0.3, 0.05])
    for near in (False, True):
        rot = lambda z, p: R.rotate_pairs(z, rates, 1.5, near, p)
        assert np.allclose(rot(x, 0)[..., :6], 1.5 * x[..., :6]) and np.allclose(rot(x, 9)[..., 6:], x[..., 6:])
        assert np.isclose((rot(x, 7) * rot(y, 3)).sum(), (rot(x, 104) * rot(y, 100)).sum())
        z = np.zeros((1, 1, 12)); z[0, 0, 2 if near else 1] = 1.0
        assert np.allclose(rot(z, 5)[0, 0, [2, 3] if near else [1, 4]], 1.5 * np.array([np.cos(1.5), np.sin(1.5)]))
    assert np.allclose(R.rotate_pairs(x, R.turn_rates(8, 50.0)[0], pos0=7), R.rotate_half(x, 50.0, 8, 7))


def test_sink_takes_its_share_of_the_weights():
    rng = np.random.default_rng(8)
    T, sink = 6, np.array([2.0, -3.0, 40.0, -60.0])
    q, k, v = rng.standard_normal((T, 4, 6)), rng.standard_normal((T, 2, 6)), rng.standard_normal((T, 2, 5))
    o, bare = R.causal_attention(q, k, v, 0.3, sink), R.causal_attention(q, k, v, 0.3)
    for i in range(T):
        for h in range(4):
            s = np.exp(0.3 * k[:i + 1, h // 2] @ q[i, h])
            assert np.allclose(o[i, h], s @ v[:i + 1, h // 2] / (s.sum() + np.exp(sink[h]))) and np.allclose(bare[i, h], s @ v[:i + 1, h // 2] / s.sum())


def test_forget_gates_write_what_they_forget():
    rng = np.random.default_rng(9)
    T, d, dv = 6, 4, 3
    q, f, v = rng.standard_normal((T, 1, d)), rng.uniform(0, 1, (T, 1, d)), rng.standard_normal((T, 1, dv))
    o = R.forget_gate_recurrence(q, f, v)
    for t in range(T):
        want = sum(q[t, 0, c] * f[s + 1:t + 1, 0, c].prod() * (1 - f[s, 0, c]) * v[s, 0] for s in range(t + 1) for c in range(d))
        assert np.allclose(o[t, 0], want)
    one = np.repeat(v[:1], T, axis=0)                   # a constant input: every row of the state tends to it
    assert np.allclose(R.forget_gate_recurrence(q, 0 * f, one), q.sum(-1, keepdims=True) * one)


def test_routing_within_the_best_groups():
    z = np.array([[2.0, -1.0, 1.5, 1.4, 0.0, 0.1]])
    s = 1 / (1 + np.exp(-z[0]))
    pick = lambda *e: [[s[i] if i in e else 0.0 for i in range(6)]]
    none = np.zeros(6)
    assert np.allclose(R.route_groups(z, none, 2, 3, 1), pick(2, 3))           # two good ones beat the best with a bad neighbour
    assert np.allclose(R.route_groups(z, none, 2, 3, 3), pick(0, 2)) and np.allclose(R.route_groups(z, none, 2, 1, 1), pick(0, 2))
    assert np.allclose(R.route_groups(z, none, 3, 3, 2), pick(0, 2, 3))
    assert np.allclose(R.route_groups(z, np.array([0, 0, -1.0, -1.0, 0, 0]), 1, 3, 1), pick(0))
    low = np.full(6, -5.0); low[4] = -4.0; low[5] = -4.9                       # negative choice scores: left out is less than any of them
    assert np.allclose(R.route_groups(z, low, 2, 3, 1), pick(4, 5))
    assert np.allclose(R.route_groups(z, none, 2, 6, 2), pick(0, 2))           # groups of one
    assert np.allclose(R.soft_cap(np.array([0.01, 1e3, -1e3]), 5.0), [0.01, 5.0, -5.0], atol=1e-6)


def test_zenorax_oracle_is_sensitive_to_what_it_checks():
    """every constant and every small tensor, a far token: each moves the logits well beyond the tests' tolerances"""
    cfg = B.zconfig([B.zlayer(B.lat(), B.zmoe()), B.zlayer(B.keyval(), B.zmoe(keep=3)), B.zlayer(B.forget(), B.zmoe(top=2)), B.zlayer(B.lat(heads=2, yarn=None))])
    w = {n: B.to_bf16(a)[1].reshape(np.shape(a)) for n, a in B.weights(cfg, 5).items()}
    tok = np.random.default_rng(6).integers(0, cfg["vocab"], 40)
    base = R.forward(cfg, w, tok)
    at = lambda c, i: c["layers"][i]
    mix = lambda i, **kw: lambda c: at(c, i)["mixer"].update(**kw)
    rot = lambda i, **kw: lambda c: at(c, i)["mixer"]["rot"].update(**kw)
    yarn = lambda **kw: lambda c: at(c, 0)["mixer"]["rot"]["scaling"].update(**kw)
    for change in (mix(0, scale=0.25), mix(1, scale=0.4), rot(0, base=100.0), rot(1, base=20.0), rot(1, dims=8), yarn(factor=8.0), yarn(original=1200), yarn(fast=20.0), yarn(slow=4.0),
                   lambda c: at(c, 1)["mixer"]["rot"]["scaling"].update(factor=3.0), lambda c: at(c, 1)["mixer"]["rot"].pop("scaling"), lambda c: c["norm"].update(eps=0.1),
                   lambda c: c["embedding"].update(scale=1.0), lambda c: c.update(logit_softcap=7.0), lambda c: at(c, 0)["mlp"]["router"].update(top=2),
                   lambda c: at(c, 0)["mlp"]["router"]["groups"].update(keep=1 + 2), lambda c: at(c, 0)["mlp"]["router"]["groups"].update(count=2, keep=1)):
        other = json.loads(json.dumps(cfg)); change(other)
        assert np.abs(R.forward(other, w, tok) - base).max() > 1e-2
    for name in w:
        if ".mlp.e" not in name:
            other = dict(w, **{name: w[name].copy()}); other[name][::2] *= 0.3          # (every second row: a norm takes a common factor back)
            assert np.abs(R.forward(cfg, other, tok) - base).max() > 1e-2, name
    assert np.abs(R.forward(cfg, w, tok[1:])[-1] - base[-1]).max() > 1e-2


@pytest.mark.parametrize("text, reason", [("{", "malformed"), ("[]", ""), ('{"architecture": "Nobody"}', "Samanex"), ("{}", "Samanex"),
                                          ('{"architecture": "Samanex"} x', "after"), ('{"architecture": "\\ud800"}', "malformed")])
def test_registry_refuses_what_it_does_not_know(tmp_path, text, reason):
    from helpers.device import cai
    (tmp_path / "config.json").write_text(text)
    with pytest.raises(cai.CaiError) as e:
        cai.Decoder.load(str(tmp_path), 64)
    assert reason in str(e.value)


def test_registry_refuses_bad_arguments(tmp_path):
    from helpers.device import cai
    for args in ((0, 1, 0), (64, 0, 0), (64, 1, 7)):
        with pytest.raises(cai.CaiError):
            cai.Decoder.load(str(tmp_path), *args)
    with pytest.raises(cai.CaiError):
        cai.Decoder.load(str(tmp_path / "absent"), 64)


def test_trace_runner_is_executable():
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    assert os.access(os.path.join(root, "bin", "trace_run"), os.X_OK)
