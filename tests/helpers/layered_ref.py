"""Plain, slow float64 implementation of the layered decoder designs, one function per mechanism.

This is the oracle of the layered decoder (tests/test_layered_ref.py, tests/test_gpu_layered.py): numpy only, token by token where the mechanism is a
recurrence, a full score matrix where it is an attention, and no code shared with the product library.
"""
import numpy as np


# ---------------------------------------------------------------- mechanisms
def linear(w, x):
    """rows of x through a matrix stored [out, in]"""
    return x @ w.T


def dynamic_tanh(x, alpha, w, b):
    """y = w * tanh(alpha x) + b: a squashing in place of a normalisation, no statistics"""
    return np.tanh(alpha * x) * w + b


def rms_norm(x, eps):
    """x over its root mean square along the last axis, eps inside the root"""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def causal_conv(x, taps_w):
    """depthwise convolution over time, zeros before the start; taps_w[c, -1] weighs the current token"""
    n_taps = taps_w.shape[1]
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        for k in range(n_taps):
            s = t - (n_taps - 1) + k
            if s >= 0:
                y[t] += taps_w[:, k] * x[s]
    return y


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def softmax_rows(s):
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def window_attention(q, k, v, scale, window):
    """q [T, H, d], k [T, G, d], v [T, G, dv]; query i sees the `window` tokens that end at itself"""
    T, H, _ = q.shape
    G = k.shape[1]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = (j <= i) & (i - j < window)
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(seen, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        out[:, h] = softmax_rows(s) @ v[:, g]
    return out


def delta_rule(q, k, v, decay, beta):
    """Gated delta rule, token by token.  q, k [T, H, d]; v [T, H, dv]; decay [T, H, d] (one per key channel, a per-head
    decay repeated); beta [T, H].  S [H, d, dv] starts at zero: decay the rows, write the correction, read."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    out = np.zeros(v.shape)
    for t in range(T):
        S *= decay[t][:, :, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t]))
        S += k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hkv,hk->hv", S, q[t])
    return out


# ---------------------------------------------------------------- mixers
def delta_mixer(w, pre, c, h, eps, channel_decay):
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    act = [silu(causal_conv(linear(w[pre + n], h), w[pre + n + ".conv"])) for n in "qkv"]
    q = unit(act[0].reshape(T, G, d)) * d ** -0.5
    k = unit(act[1].reshape(T, G, d))
    v = act[2].reshape(T, H, dv)
    q, k = (np.repeat(z, H // G, axis=1) for z in (q, k))
    beta = sigmoid(linear(w[pre + "b"], h))
    rate = np.exp(w[pre + "A_log"])
    if channel_decay:
        z = linear(w[pre + "a2"], linear(w[pre + "a1"], h)) + w[pre + "dt_bias"].reshape(-1)
        decay = np.exp(-rate[None, :, None] * softplus(z).reshape(T, H, d))
        gate = sigmoid(linear(w[pre + "g2"], linear(w[pre + "g1"], h)))
    else:
        z = linear(w[pre + "a"], h) + w[pre + "dt_bias"]
        decay = np.repeat(np.exp(-rate * softplus(z))[:, :, None], d, axis=2)
        gate = silu(linear(w[pre + "g"], h))
    o = delta_rule(q, k, v, decay, beta)
    o = rms_norm(o, eps) * w[pre + "norm"] * gate.reshape(T, H, dv)
    return linear(w[pre + "o"], o.reshape(T, H * dv))


def attention_mixer(w, pre, c, h, eps):
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = rms_norm(linear(w[pre + "q"], h).reshape(T, H, d), eps) * w[pre + "q.norm"]
    k = rms_norm(linear(w[pre + "k"], h).reshape(T, G, d), eps) * w[pre + "k.norm"]
    v = linear(w[pre + "v"], h).reshape(T, G, dv)
    o = window_attention(q, k, v, c["scale"], c["mask"]["size"])
    return linear(w[pre + "o"], o.reshape(T, H * dv))


def parallel_mixer(w, pre, c, h, eps):
    a = attention_mixer(w, pre + "left.", c["left"], h, eps)
    b = delta_mixer(w, pre + "right.", c["right"], h, eps, True)
    return 0.5 * (rms_norm(a, eps) * w[pre + "left.out"] + rms_norm(b, eps) * w[pre + "right.out"])


def relu_glu(w, pre, h):
    return linear(w[pre + "down"], np.maximum(linear(w[pre + "gate"], h), 0.0) * linear(w[pre + "up"], h))


# ---------------------------------------------------------------- mechanisms of Kiruvik
def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rotate_half(x, base, dims, pos0=0):
    """x [T, heads, d]: dimension i of the first `dims` turns with dimension i + dims / 2 by position * base^(-2i/dims)"""
    half = dims // 2
    out = x.copy()
    for i in range(half):
        a = ((pos0 + np.arange(x.shape[0])) * base ** (-2.0 * i / dims))[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * np.cos(a) - v * np.sin(a)
        out[:, :, i + half] = v * np.cos(a) + u * np.sin(a)
    return out


def chunk_attention(q, k, v, scale, size):
    """as window_attention, but query i sees the keys up to itself of its own block of `size` positions"""
    T, H, _ = q.shape
    G = k.shape[1]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = (j <= i) & (i // size == j // size)
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(seen, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        out[:, h] = softmax_rows(s) @ v[:, g]
    return out


def ssd_recurrence(x, B, C, dt, rate, D):
    """State-space duality, token by token.  x [T, H, P]; B, C [T, G, N]; dt [T, H]; rate, D [H].  S [H, N, P] starts at zero:
    decay by exp(-rate dt), add dt B x^T, read with C; the input passes by with weight D."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = np.zeros((H, N, P))
    y = np.zeros_like(x)
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            S[h] = np.exp(-rate[h] * dt[t, h]) * S[h] + dt[t, h] * np.outer(B[t, g], x[t, h])
            y[t, h] = S[h].T @ C[t, g] + D[h] * x[t, h]
    return y


def group_rms_norm(x, groups, eps):
    T, n = x.shape
    return rms_norm(x.reshape(T, groups, n // groups), eps).reshape(T, n)


def clamped_expert(w, pre, h, limit):
    g = np.minimum(linear(w[pre + "gate"], h), limit)
    u = np.clip(linear(w[pre + "up"], h), -limit, limit)
    return linear(w[pre + "down"], g * sigmoid(1.702 * g) * (u + 1.0))


def route(z, correction, top, scale):
    """[T, experts] weights of one token's experts, zero where not chosen: soft-max scores, chosen with the correction added, weighted
    without it"""
    s = softmax_rows(z)
    out = np.zeros_like(s)
    for t in range(s.shape[0]):
        chosen = np.argsort(-(s[t] + correction), kind="stable")[:top]
        out[t, chosen] = s[t, chosen] / (s[t, chosen].sum() + 1e-20) * scale
    return out


def rotary_attention_mixer(w, pre, c, h):
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (linear(w[pre + n], h) + w[pre + n + ".b"] for n in "qkv")
    q = rotate_half(q.reshape(T, H, d), c["rot"]["base"], c["rot"]["dims"])
    k = rotate_half(k.reshape(T, G, d), c["rot"]["base"], c["rot"]["dims"])
    o = chunk_attention(q, k, v.reshape(T, G, dv), c["scale"], c["mask"]["size"]).reshape(T, H * dv)
    o = o * sigmoid(linear(w[pre + "g"], h))
    return linear(w[pre + "o"], o) + w[pre + "o.b"]


def ssd_mixer(w, pre, c, h, eps):
    T = h.shape[0]
    H, P, N, G = c["heads"], c["vdim"], c["state"], c["groups"]
    inner = H * P
    z, x, B, C, dt = np.split(linear(w[pre + "in"], h), np.cumsum([inner, inner, G * N, G * N]), axis=1)
    xbc = silu(causal_conv(np.concatenate([x, B, C], axis=1), w[pre + "conv"]) + w[pre + "conv.b"])
    x, B, C = np.split(xbc, np.cumsum([inner, G * N]), axis=1)
    dt = softplus(dt + w[pre + "dt_bias"])
    y = ssd_recurrence(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), dt, np.exp(w[pre + "A_log"]), w[pre + "D"])
    y = group_rms_norm(y.reshape(T, inner) * silu(z), c["norm_groups"], eps) * w[pre + "norm"]
    return linear(w[pre + "o"], y)


def gelu_glu(w, pre, h):
    return linear(w[pre + "down"], gelu_tanh(linear(w[pre + "gate"], h)) * linear(w[pre + "up"], h))


def expert_mixture(w, pre, c, h):
    r = c["router"]
    wt = route(linear(w[pre + "router"], h), w[pre + "correction"], r["top"], r["scale"])
    y = clamped_expert(w, pre + "shared.", h, c["shared"]["limit"])
    for e in range(r["experts"]):
        y = y + wt[:, e:e + 1] * clamped_expert(w, pre + "e%d." % e, h, c["expert"]["limit"])
    return y


# ---------------------------------------------------------------- mechanisms of Gamanex
def sigmoid_attention(q, k, v, scale, r1, r2, bias):
    """q [T, H, d], k [T, G, d], v [T, G, dv].  Query i weighs every key j <= i by the sigmoid of its score, nothing is normalised over
    the keys.  The score loses r1 ln(1 + r2 (i - j)) with the distance and gains a number per head."""
    T, H, _ = q.shape
    G = k.shape[1]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    far = np.maximum(i - j, 0)
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale - r1[h] * np.log(1.0 + r2[h] * far) + bias[h]
        out[:, h] = np.where(j <= i, sigmoid(s), 0.0) @ v[:, g]
    return out


def query_temperature(positions, coef, every):
    """factor of a query at a position: grows with the logarithm of how many times `every` positions have passed"""
    return 1.0 + coef * np.log(np.floor((positions + 1) / every) + 1.0)


def sigmoid_attention_mixer(w, pre, c, h, eps, kept, layer):
    """kept: keys and values of earlier layers by layer number; a layer with 'kv_from' reads them there"""
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = rms_norm(linear(w[pre + "q"], h), eps) * w[pre + "q.norm"]
    q = q * query_temperature(np.arange(T), c["q_temp"]["coef"], c["q_temp"]["every"])[:, None]
    if c.get("kv_from") is not None:
        k, v = kept[c["kv_from"]]
    else:
        k = (rms_norm(linear(w[pre + "k"], h), eps) * w[pre + "k.norm"]).reshape(T, G, d)
        v = linear(w[pre + "v"], h).reshape(T, G, dv)
        kept[layer] = k, v
    o = sigmoid_attention(q.reshape(T, H, d), k, v, c["scale"], w[pre + "r1"], w[pre + "r2"], w[pre + "pb"])
    return linear(w[pre + "o"], o.reshape(T, H * dv))


def squared_relu_mlp(w, pre, h):
    return linear(w[pre + "down"], np.maximum(linear(w[pre + "up"], h), 0.0) ** 2)


def silu_expert(w, pre, h):
    return linear(w[pre + "down"], silu(linear(w[pre + "gate"], h)) * linear(w[pre + "up"], h))


def route_among_chosen(z, top):
    """[T, experts] weights: the `top` largest logits, soft-max over these alone"""
    out = np.zeros_like(z)
    for t in range(z.shape[0]):
        chosen = np.argsort(-z[t], kind="stable")[:top]
        out[t, chosen] = softmax_rows(z[t, chosen][None])[0]
    return out


def silu_expert_mixture(w, pre, c, h):
    wt = route_among_chosen(linear(w[pre + "router"], h) + w[pre + "router.b"], c["router"]["top"])
    return sum(wt[:, e:e + 1] * silu_expert(w, pre + "e%d." % e, h) for e in range(c["router"]["experts"]))


def sublayer_gate(w, name, h):
    """what a sublayer's result is multiplied by before it joins the stream, from the sublayer's own input"""
    return sigmoid(linear(w[name], h) + w[name + ".b"])


# ---------------------------------------------------------------- mechanisms of Zenorax
def turn_rates(dims, base, linear=1.0, yarn=None):
    """radians a position of every pair of a rotation over `dims` dimensions, and what cosine and sine are multiplied by.  linear: all
    slowed down alike.  yarn: the slow pairs are slowed down by its factor, the fast ones not, a ramp in between."""
    i = np.arange(dims // 2)
    f = base ** (-2.0 * i / dims) / linear
    if not yarn:
        return f, 1.0
    pair = lambda turns: dims * np.log(yarn["original"] / (2 * np.pi * turns)) / (2 * np.log(base))
    lo, hi = max(np.floor(pair(yarn["fast"])), 0), min(np.ceil(pair(yarn["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0, 1)
    return f / yarn["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(yarn["factor"]) + 1


def rotate_pairs(x, rates, amp=1.0, neighbours=False, pos0=0):
    """x [T, heads, d]: pair i turns by position * rates[i] and grows by amp; a pair is dimensions 2i and 2i + 1 (neighbours) or i and
    i + len(rates); dimensions past 2 len(rates) stay"""
    n = len(rates)
    out = x.copy()
    for i in range(n):
        a = ((pos0 + np.arange(x.shape[0])) * rates[i])[:, None]
        p, q = (2 * i, 2 * i + 1) if neighbours else (i, i + n)
        u, v = x[:, :, p], x[:, :, q]
        out[:, :, p] = amp * (u * np.cos(a) - v * np.sin(a))
        out[:, :, q] = amp * (v * np.cos(a) + u * np.sin(a))
    return out


def causal_attention(q, k, v, scale, sink=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv]; soft-max over every key up to the query.  sink [H]: the denominator holds one more term,
    the exponential of a number per head that has no key"""
    T, H, _ = q.shape
    G = k.shape[1]
    seen = np.arange(T)[None, :] <= np.arange(T)[:, None]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(seen, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        m = s.max(-1, keepdims=True) if sink is None else np.maximum(s.max(-1, keepdims=True), sink[h])
        e = np.exp(s - m)
        den = e.sum(-1, keepdims=True) + (0.0 if sink is None else np.exp(sink[h] - m))
        out[:, h] = (e / den) @ v[:, g]
    return out


def latent_attention_mixer(w, pre, c, h, eps):
    """queries through a latent of their own; keys (the part that does not turn) and values made from one shared latent; one key part that
    turns, shared by all heads; a sigmoid gate on the heads"""
    T, H, d, dr, dv, r = h.shape[0], c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    rates, amp = turn_rates(c["rot"]["dims"], c["rot"]["base"], yarn=c["rot"].get("scaling"))
    q = linear(w[pre + "uq"], rms_norm(linear(w[pre + "dq"], h), eps) * w[pre + "dq.norm"]).reshape(T, H, d + dr)
    kv = linear(w[pre + "dkv"], h)
    lat = rms_norm(kv[:, :r], eps) * w[pre + "dkv.norm"]
    turned = rotate_pairs(kv[:, None, r:], rates, amp, True)
    q = np.concatenate([q[:, :, :d], rotate_pairs(q[:, :, d:], rates, amp, True)], axis=2)
    k = np.concatenate([linear(w[pre + "uk"], lat).reshape(T, H, d), np.repeat(turned, H, axis=1)], axis=2)
    o = causal_attention(q, k, linear(w[pre + "uv"], lat).reshape(T, H, dv), c["scale"]).reshape(T, H * dv)
    return linear(w[pre + "o"], o * sigmoid(linear(w[pre + "g"], h)))


def key_value_attention_mixer(w, pre, c, h, eps):
    """the values are the keys as projected; queries and keys turn, then are normed per head without a gain"""
    T, H, G, d = h.shape[0], c["heads"], c["kv_heads"], c["dim"]
    scaling = c["rot"].get("scaling")
    rates, _ = turn_rates(c["rot"]["dims"], c["rot"]["base"], linear=scaling["factor"] if scaling else 1.0)
    q, k = linear(w[pre + "q"], h).reshape(T, H, d), linear(w[pre + "k"], h).reshape(T, G, d)
    o = causal_attention(rms_norm(rotate_pairs(q, rates), eps), rms_norm(rotate_pairs(k, rates), eps), k, c["scale"], w[pre + "sink"])
    return linear(w[pre + "o"], o.reshape(T, H * d))


def forget_gate_recurrence(q, f, v):
    """q, f [T, H, d]; v [T, H, dv].  S [H, d, dv] starts at zero: its rows are forgotten by f, what f forgets is written, q reads"""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    out = np.zeros(v.shape)
    for t in range(T):
        for i in range(H):
            S[i] = f[t, i][:, None] * S[i] + np.outer(1.0 - f[t, i], v[t, i])
            out[t, i] = S[i].T @ q[t, i]
    return out


def forget_gate_mixer(w, pre, c, h, eps):
    T, H, d, dv = h.shape[0], c["heads"], c["dim"], c["vdim"]
    q, v = silu(linear(w[pre + "q"], h)).reshape(T, H, d), linear(w[pre + "v"], h).reshape(T, H, dv)
    low = w[pre + "lower"]
    f = (low + (1.0 - low) * sigmoid(linear(w[pre + "f"], h) + w[pre + "f.b"])).reshape(T, H, d)
    o = rms_norm(forget_gate_recurrence(q, f, v), eps) * w[pre + "norm"]
    return linear(w[pre + "o"], o.reshape(T, H * dv))


def route_groups(z, correction, top, count, keep):
    """[T, experts] weights, zero where not chosen: sigmoid scores; with the correction added, the `keep` groups whose two best add up to
    most, then the `top` best of these groups; weighted by the scores alone"""
    s = sigmoid(z)
    n = z.shape[1]
    out = np.zeros_like(s)
    for t in range(z.shape[0]):
        c = (s[t] + correction).reshape(count, n // count)
        best = np.argsort(-np.sort(c, axis=1)[:, -2:].sum(1), kind="stable")[:keep]
        masked = np.full(c.shape, -np.inf)
        masked[best] = c[best]
        chosen = np.argsort(-masked.reshape(-1), kind="stable")[:top]
        out[t, chosen] = s[t, chosen]
    return out


def grouped_expert_mixture(w, pre, c, h):
    r = c["router"]
    wt = route_groups(linear(w[pre + "router"], h), w[pre + "correction"], r["top"], r["groups"]["count"], r["groups"]["keep"])
    return sum(wt[:, e:e + 1] * squared_relu_mlp(w, pre + "e%d." % e, h) for e in range(r["experts"]))


def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


# ---------------------------------------------------------------- the models
def run_order(cfg):
    """(layer, first layer of a repeated pass) for every layer run"""
    n = len(cfg["layers"])
    lp = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    runs = [(i, False) for i in range(lp["start"])]
    for p in range(lp["times"]):
        runs += [(i, p > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, False) for i in range(max(lp["stop"], lp["start"]), n)]


def forward(cfg, w, tokens, layers_out=None):
    """logits [T, vocab] of a whole prompt"""
    if cfg["architecture"] == "Kiruvik":
        return kiruvik_forward(cfg, w, tokens, layers_out)
    if cfg["architecture"] == "Gamanex":
        return gamanex_forward(cfg, w, tokens, layers_out)
    if cfg["architecture"] == "Zenorax":
        return zenorax_forward(cfg, w, tokens, layers_out)
    eps = cfg["norm"]["eps"]
    norm = lambda name, x: dynamic_tanh(x, w[name + ".alpha"], w[name], w[name + ".b"])
    x = w["embed"][np.asarray(tokens)]
    x0 = x
    for i, again in run_order(cfg):
        L = cfg["layers"][i]
        p = "l%d." % i
        if again:
            x = x + x0
        h = norm(p + "norm1", x)
        y = delta_mixer(w, p + "mix.", L["mixer"], h, eps, False) if L["type"] == "delta" else parallel_mixer(w, p + "mix.", L["mixer"], h, eps)
        x = x + norm(p + "norm1b", y)
        if L.get("mlp"):
            x = x + norm(p + "norm2b", relu_glu(w, p + "mlp.", norm(p + "norm2", x)))
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(w["head"], norm("final.norm", x))


def kiruvik_forward(cfg, w, tokens, layers_out=None):
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    norm = lambda name, x: dynamic_tanh(x, w[name + ".alpha"], w[name], w[name + ".b"])
    x = w["embed"][np.asarray(tokens)]
    x0 = x
    lp = cfg.get("loop")
    n = len(cfg["layers"])
    order = list(range(n)) if not lp else list(range(lp["start"])) + list(range(lp["start"], lp["stop"])) * lp["times"] + list(range(lp["stop"], n))
    for r, i in enumerate(order):
        L = cfg["layers"][i]
        p = "l%d." % i
        if lp and lp["start"] <= r < lp["start"] + (lp["stop"] - lp["start"]) * lp["times"] and i == lp["start"]:
            x = linear(w["loop.in"], np.concatenate([x, x0], axis=1))
        h = norm(p + "norm1", x)
        y = rotary_attention_mixer(w, p + "mix.", L["mixer"], h) if L["type"] == "attention" else ssd_mixer(w, p + "mix.", L["mixer"], h, eps)
        x = x + m * norm(p + "norm1b", y)
        if L.get("mlp"):
            h = norm(p + "norm2", x)
            y = gelu_glu(w, p + "mlp.", h) if L["mlp"]["kind"] == "dense" else expert_mixture(w, p + "mlp.", L["mlp"], h)
            x = x + m * norm(p + "norm2b", y)
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(w["head"], norm("final.norm", x))


def gamanex_forward(cfg, w, tokens, layers_out=None):
    eps, kept = cfg["norm"]["eps"], {}
    x = w["embed"][np.asarray(tokens)]
    for i, L in enumerate(cfg["layers"]):
        p = "l%d." % i
        h = rms_norm(x, eps) * w[p + "norm1"]
        y = sigmoid_attention_mixer(w, p + "mix.", L["mixer"], h, eps, kept, i) * w[p + "ls1"] * sublayer_gate(w, p + "rg1", h)
        if L.get("mlp"):
            h = rms_norm(x, eps) * w[p + "norm2"]
            f = squared_relu_mlp(w, p + "mlp.", h) if L["mlp"]["kind"] == "dense" else silu_expert_mixture(w, p + "mlp.", L["mlp"], h)
            y = y + f * w[p + "ls2"] * sublayer_gate(w, p + "rg2", h)
        x = x + y
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(w["head"], rms_norm(x, eps) * w["final.norm"]) * cfg["logit_scale"]


ZENORAX_MIXERS = dict(latent_attention=latent_attention_mixer, attention=key_value_attention_mixer, hgrn2=forget_gate_mixer)


def zenorax_forward(cfg, w, tokens, layers_out=None):
    eps = cfg["norm"]["eps"]
    norm = lambda name, z: rms_norm(z, eps) * w[name]
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    kept = [x]
    for i, L in enumerate(cfg["layers"]):
        p = "l%d." % i
        h = norm(p + "norm1", x)
        h = h + causal_conv(h, w[p + "canon1"])
        x = x + norm(p + "norm1b", ZENORAX_MIXERS[L["type"]](w, p + "mix.", L["mixer"], h, eps))
        if L.get("mlp"):
            x = x + norm(p + "norm2b", grouped_expert_mixture(w, p + "mlp.", L["mlp"], norm(p + "norm2", x)))
        kept.append(x)
        x = sum(a * z for a, z in zip(w[p + "dwa"], kept))
        if layers_out is not None:
            layers_out.append(x.copy())
    return soft_cap(linear(w["embed"], norm("final.norm", x)), cfg["logit_softcap"])
