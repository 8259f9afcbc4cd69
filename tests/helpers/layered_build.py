"""Small random models for the layered-decoder tests: a configuration, weights rounded to bfloat16, a model folder."""
import json
import os
import struct

import numpy as np


def to_bf16(a):
    """(bits, the rounded values as float64)"""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    u = ((u + 0x7fff + ((u >> 16) & 1)) >> 16).astype(np.uint16)
    return u, (u.astype(np.uint32) << 16).view(np.float32).astype(np.float64)


def delta(heads=2, kv_heads=1, dim=20, vdim=36, conv=3):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)


def attn(heads=4, kv_heads=2, dim=24, vdim=40, window=9, scale=0.21):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask=dict(size=window))


def layer(mixer, ff=56):
    """a delta layer from a delta mixer, a parallel layer from a (left, right) pair; ff None: no feed-forward"""
    mlp = None if ff is None else dict(kind="dense", ff=ff)
    if isinstance(mixer, tuple):
        return dict(type="parallel", mixer=dict(left=mixer[0], right=mixer[1]), mlp=mlp)
    return dict(type="delta", mixer=mixer, mlp=mlp)


def config(layers, width=72, vocab=131, eps=1e-5, loop=None):
    return dict(architecture="Samanex", width=width, vocab=vocab, layers=layers, norm=dict(eps=eps),
                loop=loop or dict(start=0, stop=len(layers), times=1))


# ---------------------------------------------------------------- Kiruvik
def rotary(heads=4, kv_heads=2, dim=24, vdim=40, block=9, scale=0.21, rot=10, base=500.0):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask=dict(size=block), rot=dict(base=base, dims=rot))


def ssd(heads=4, vdim=18, state=20, groups=2, conv=3, norm_groups=3):
    return dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)


def moe(experts=6, top=2, ff=20, scale=1.7, limit=0.9, shared_ff=28, shared_limit=1.3):
    return dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top, scale=scale), shared=dict(ff=shared_ff, limit=shared_limit))


def klayer(mixer, mlp=None):
    """an attention or a state-space layer; mlp: a width (dense), a mixture, or None"""
    return dict(type="attention" if "rot" in mixer else "mamba2", mixer=mixer, mlp=dict(kind="dense", ff=mlp) if isinstance(mlp, int) else mlp)


def kconfig(layers, width=72, vocab=131, eps=1e-5, loop=None, mult=0.8):
    return dict(architecture="Kiruvik", width=width, vocab=vocab, layers=layers, norm=dict(eps=eps), residual_mult=mult, loop=loop)


def kiruvik_weights(cfg, seed=0):
    rng = np.random.default_rng(seed)
    w, width = {}, cfg["width"]

    def lin(name, rows, cols, gain=1.0):
        w[name] = rng.standard_normal((rows, cols)) * gain / np.sqrt(cols)

    def vec(name, shape, mean=0.0, spread=0.2):
        w[name] = mean + spread * rng.standard_normal(shape)

    def norm(name):
        vec(name, width, 1.0); vec(name + ".b", width, 0.0, 0.1)
        w[name + ".alpha"] = np.asarray(rng.uniform(0.4, 1.2))

    def glu(p, ff):
        lin(p + "gate", ff, width, 1.5); lin(p + "up", ff, width, 1.5); lin(p + "down", width, ff)

    vec("embed", (cfg["vocab"], width), 0.0, 1.0)
    lin("head", cfg["vocab"], width, 2.0)
    norm("final.norm")
    if cfg["loop"] and cfg["loop"]["stop"] > cfg["loop"]["start"]:
        lin("loop.in", width, 2 * width, 1.3)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = "l%d." % i, L["mixer"], L["mlp"]
        norm(p + "norm1"); norm(p + "norm1b")
        if L["type"] == "attention":
            for n, r in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                lin(p + "mix." + n, r, width, 1.5); vec(p + "mix." + n + ".b", r, 0.0, 0.4)
            lin(p + "mix.g", m["heads"] * m["vdim"], width, 2.0)
            lin(p + "mix.o", width, m["heads"] * m["vdim"]); vec(p + "mix.o.b", width, 0.0, 0.3)
        else:
            inner = m["heads"] * m["vdim"]; ch = inner + 2 * m["groups"] * m["state"]
            lin(p + "mix.in", inner + ch + m["heads"], width, 1.5)
            vec(p + "mix.conv", (ch, m["conv"]), 0.3, 0.5); vec(p + "mix.conv.b", ch, 0.0, 0.3)
            vec(p + "mix.dt_bias", m["heads"], -2.0, 1.0); w[p + "mix.A_log"] = rng.uniform(-2.0, 1.0, m["heads"])
            vec(p + "mix.D", m["heads"], 0.7, 0.5); vec(p + "mix.norm", inner, 1.0)
            lin(p + "mix.o", width, inner)
        if f:
            norm(p + "norm2"); norm(p + "norm2b")
            if f["kind"] == "dense":
                glu(p + "mlp.", f["ff"])
            else:
                lin(p + "mlp.router", f["router"]["experts"], width, 2.0); vec(p + "mlp.correction", f["router"]["experts"], 0.0, 0.1)
                for e in range(f["router"]["experts"]):
                    glu(p + "mlp.e%d." % e, f["expert"]["ff"])
                glu(p + "mlp.shared.", f["shared"]["ff"])
    return w


def steady_choice(w):
    """corrections so far apart that they alone decide which experts run: rounding cannot change the choice"""
    for n in w:
        if n.endswith(".correction"):
            w[n] = 4.0 * np.random.default_rng(len(w[n])).permutation(len(w[n]))


# ---------------------------------------------------------------- Gamanex
def sig(heads=4, kv_heads=2, dim=24, vdim=40, scale=0.21, coef=0.4, every=7, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, q_temp=dict(coef=coef, every=every))
    return m if kv_from is None else dict(m, kv_from=kv_from)


def gmoe(experts=6, top=2, ff=20):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))


def glayer(mixer, mlp=None):
    """mlp: a width (dense), a mixture, or None"""
    return dict(type="attention", mixer=mixer, mlp=dict(kind="dense", ff=mlp) if isinstance(mlp, int) else mlp)


def gconfig(layers, width=72, vocab=131, eps=1e-5, logit_scale=0.7):
    return dict(architecture="Gamanex", width=width, vocab=vocab, layers=layers, norm=dict(eps=eps), logit_scale=logit_scale)


def gamanex_weights(cfg, seed=0):
    rng = np.random.default_rng(seed)
    w, width = {}, cfg["width"]

    def lin(name, rows, cols, gain=1.0):
        w[name] = rng.standard_normal((rows, cols)) * gain / np.sqrt(cols)

    def vec(name, shape, mean=0.0, spread=0.2):
        w[name] = mean + spread * rng.standard_normal(shape)

    vec("embed", (cfg["vocab"], width), 0.0, 1.0)
    lin("head", cfg["vocab"], width, 2.0)
    vec("final.norm", width, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = "l%d." % i, L["mixer"], L["mlp"]
        a = p + "mix."
        qw, kw = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
        lin(a + "q", qw, width); vec(a + "q.norm", qw, 1.2, 0.4)
        if m.get("kv_from") is None:
            lin(a + "k", kw, width); lin(a + "v", m["kv_heads"] * m["vdim"], width); vec(a + "k.norm", kw, 1.1, 0.4)
        w[a + "r1"] = rng.uniform(0.1, 1.2, m["heads"]); w[a + "r2"] = rng.uniform(0.05, 2.0, m["heads"])
        vec(a + "pb", m["heads"], -1.5, 1.0)
        lin(a + "o", width, m["heads"] * m["vdim"])
        for k in ("1", "2") if f else ("1",):
            vec(p + "norm" + k, width, 1.0); vec(p + "ls" + k, width, 0.8, 0.4)
            lin(p + "rg" + k, width, width, 1.5); vec(p + "rg" + k + ".b", width, 0.3, 0.5)
        if f and f["kind"] == "dense":
            lin(p + "mlp.up", f["ff"], width); lin(p + "mlp.down", width, f["ff"])
        elif f:
            lin(p + "mlp.router", f["router"]["experts"], width, 2.0); vec(p + "mlp.router.b", f["router"]["experts"], 0.0, 0.5)
            for e in range(f["router"]["experts"]):
                x = p + "mlp.e%d." % e
                lin(x + "gate", f["expert"]["ff"], width, 1.5); lin(x + "up", f["expert"]["ff"], width, 1.5); lin(x + "down", width, f["expert"]["ff"])
    return w


def steady_experts(cfg):
    """edit: logits whose bias alone decides which experts run, so that rounding cannot change the choice"""
    def edit(w):
        for i, L in enumerate(cfg["layers"]):
            if L["mlp"] and L["mlp"]["kind"] == "moe":
                n, top = L["mlp"]["router"]["experts"], L["mlp"]["router"]["top"]
                w["l%d.mlp.router.b" % i][np.random.default_rng(i).permutation(n)[:top]] += 14.0
    return edit


# ---------------------------------------------------------------- Zenorax
def lat(heads=4, dim=20, rot_dim=12, vdim=28, kv_rank=36, q_rank=44, scale=0.2, rot=None, base=300.0, yarn=(4.0, 400, 8.0, 1.0)):
    """yarn: factor, original, fast, slow, or None"""
    r = dict(base=base, dims=rot_dim if rot is None else rot)
    if yarn:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale, rot=r)


def keyval(heads=4, kv_heads=2, dim=24, scale=0.3, rot=16, base=200.0, factor=1.7):
    r = dict(base=base, dims=rot)
    if factor:
        r["scaling"] = dict(factor=factor)
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale, rot=r)


def forget(heads=3, dim=20, vdim=28):
    return dict(heads=heads, dim=dim, vdim=vdim)


def zmoe(experts=8, top=3, ff=20, count=4, keep=2):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top, groups=dict(count=count, keep=keep)))


def zlayer(mixer, mlp=None):
    return dict(type="latent_attention" if "kv_rank" in mixer else "attention" if "rot" in mixer else "hgrn2", mixer=mixer, mlp=mlp)


def zconfig(layers, width=72, vocab=131, eps=1e-5, taps=3, scale=1.9, cap=9.0):
    return dict(architecture="Zenorax", width=width, vocab=vocab, layers=layers, norm=dict(eps=eps), canon=dict(taps=taps), embedding=dict(scale=scale), logit_softcap=cap)


def steady_groups(w):
    """as steady_choice, for a choice of groups in front of it: no two pairs of corrections have the same sum"""
    for n in w:
        if n.endswith(".correction"):
            w[n] = 4.0 * 2.0 ** np.random.default_rng(len(w[n])).permutation(len(w[n]))


def zenorax_weights(cfg, seed=0):
    rng = np.random.default_rng(seed)
    w, width = {}, cfg["width"]

    def lin(name, rows, cols, gain=1.0):
        w[name] = rng.standard_normal((rows, cols)) * gain / np.sqrt(cols)

    def vec(name, shape, mean=0.0, spread=0.2):
        w[name] = mean + spread * rng.standard_normal(shape)

    vec("embed", (cfg["vocab"], width), 0.0, 0.7)
    vec("final.norm", width, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = "l%d." % i, L["mixer"], L["mlp"]
        a = p + "mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            vec(p + n, width, 1.0)
        vec(p + "canon1", (width, cfg["canon"]["taps"]), 0.1, 0.4)
        vec(p + "dwa", i + 2, 0.2, 0.3); w[p + "dwa"][-1] += 0.8
        if L["type"] == "latent_attention":
            H = m["heads"]
            lin(a + "dq", m["q_rank"], width); vec(a + "dq.norm", m["q_rank"], 1.2)
            lin(a + "uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"], 1.3)
            lin(a + "dkv", m["kv_rank"] + m["rot_dim"], width, 1.4); vec(a + "dkv.norm", m["kv_rank"], 1.1)
            lin(a + "uk", H * m["dim"], m["kv_rank"], 1.3); lin(a + "uv", H * m["vdim"], m["kv_rank"])
            lin(a + "g", H * m["vdim"], width, 1.5); lin(a + "o", width, H * m["vdim"])
        elif L["type"] == "attention":
            lin(a + "q", m["heads"] * m["dim"], width); lin(a + "k", m["kv_heads"] * m["dim"], width)
            vec(a + "sink", m["heads"], 1.0, 1.0); lin(a + "o", width, m["heads"] * m["dim"])
        else:
            n = m["heads"] * m["dim"]
            lin(a + "q", n, width, 1.5); lin(a + "f", n, width, 1.5); lin(a + "v", m["heads"] * m["vdim"], width)
            vec(a + "f.b", n, 1.0, 1.0); w[a + "lower"] = rng.uniform(0.0, 0.9, n); vec(a + "norm", m["vdim"], 1.0); lin(a + "o", width, m["heads"] * m["vdim"])
        if f:
            lin(p + "mlp.router", f["router"]["experts"], width, 2.0); vec(p + "mlp.correction", f["router"]["experts"], 0.0, 0.2)
            for e in range(f["router"]["experts"]):
                lin(p + "mlp.e%d.up" % e, f["expert"]["ff"], width, 1.5); lin(p + "mlp.e%d.down" % e, width, f["expert"]["ff"])
    return w


def weights(cfg, seed=0, rank_a=7, rank_g=11):
    """name -> float array before rounding"""
    if cfg["architecture"] == "Kiruvik":
        return kiruvik_weights(cfg, seed)
    if cfg["architecture"] == "Gamanex":
        return gamanex_weights(cfg, seed)
    if cfg["architecture"] == "Zenorax":
        return zenorax_weights(cfg, seed)
    rng = np.random.default_rng(seed)
    w, width = {}, cfg["width"]

    def lin(name, rows, cols, gain=1.0):
        w[name] = rng.standard_normal((rows, cols)) * gain / np.sqrt(cols)

    def vec(name, shape, mean=0.0, spread=0.2):
        w[name] = mean + spread * rng.standard_normal(shape)

    def norm(name):
        vec(name, width, 1.0); vec(name + ".b", width, 0.0, 0.1)
        w[name + ".alpha"] = np.asarray(rng.uniform(0.4, 1.2))

    def put_delta(p, c, channel):
        kw, vw = c["kv_heads"] * c["dim"], c["heads"] * c["vdim"]
        for n, r in (("q", kw), ("k", kw), ("v", vw)):
            lin(p + n, r, width, 1.5); vec(p + n + ".conv", (r, c["conv"]), 0.3, 0.5)
        lin(p + "b", c["heads"], width)
        w[p + "A_log"] = rng.uniform(-2.0, 1.0, c["heads"])
        vec(p + "norm", c["vdim"], 1.0)
        if channel:
            lin(p + "a1", rank_a, width); lin(p + "a2", c["heads"] * c["dim"], rank_a, 2.0)
            lin(p + "g1", rank_g, width); lin(p + "g2", vw, rank_g, 2.0)
            vec(p + "dt_bias", c["heads"] * c["dim"], -2.0, 1.0)
        else:
            lin(p + "a", c["heads"], width); lin(p + "g", vw, width)
            vec(p + "dt_bias", c["heads"], -2.0, 1.0)
        lin(p + "o", width, vw)

    vec("embed", (cfg["vocab"], width), 0.0, 1.0)
    lin("head", cfg["vocab"], width, 2.0)
    norm("final.norm")
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        norm(p + "norm1"); norm(p + "norm1b")
        if L["type"] == "delta":
            put_delta(p + "mix.", m, False)
        else:
            a = m["left"]
            lin(p + "mix.left.q", a["heads"] * a["dim"], width); lin(p + "mix.left.k", a["kv_heads"] * a["dim"], width)
            lin(p + "mix.left.v", a["kv_heads"] * a["vdim"], width); lin(p + "mix.left.o", width, a["heads"] * a["vdim"])
            vec(p + "mix.left.q.norm", a["dim"], 1.3); vec(p + "mix.left.k.norm", a["dim"], 1.2)
            put_delta(p + "mix.right.", m["right"], True)
            vec(p + "mix.left.out", width, 1.1); vec(p + "mix.right.out", width, 0.9)
        if L["mlp"]:
            norm(p + "norm2"); norm(p + "norm2b")
            lin(p + "mlp.gate", L["mlp"]["ff"], width); lin(p + "mlp.up", L["mlp"]["ff"], width); lin(p + "mlp.down", width, L["mlp"]["ff"])
    return w


def write(folder, cfg, w):
    """writes config.json and model.safetensors; returns the rounded weights as float64"""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, parts, at, out = {}, [], 0, {}
    for name, a in w.items():
        bits, out[name] = to_bf16(a)
        out[name] = out[name].reshape(np.shape(a))
        raw = bits.tobytes()
        head[name] = dict(dtype="BF16", shape=list(np.shape(a)), data_offsets=[at, at + len(raw)])
        parts.append(raw); at += len(raw)
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h)
        for raw in parts:
            f.write(raw)
    return out
