"""Synthetic block-quantized weights generated on the GPU (benchmark / full-size test plumbing).

torch is used only to make random bytes quickly: N(0, std) values are drawn on the device and packed into
GGUF blocks by vectorised torch ops; the resulting device pointer is handed to cai_qw_create, which copies.
The packers follow the same definitions as the CPU packers in oracle/oracle.c (Q8_0: reference writer,
neural/neuralgguf.pas:1966-1989; Q4_K: simple affine fit on the layout of neural/neuralgguf.pas:440-514);
they need not be bit-identical to them because parity is always judged on the bytes the device consumed.
"""
import torch

from . import caihip as cai


def _half_bytes(x):
    return x.to(torch.float16).view(torch.uint8)


def pack_q8_0(x):
    """x: [rows, cols] float32 -> uint8 [rows, cols/32, 34]"""
    rows, cols = x.shape
    xb = x.view(rows, cols // 32, 32)
    amax = xb.abs().amax(-1)
    scale = amax / 127.0
    inv = torch.where(scale > 0, 1.0 / scale, torch.zeros_like(scale))
    q = xb * inv[..., None]
    q = torch.where(q >= 0, torch.floor(q + 0.5), torch.ceil(q - 0.5)).clamp_(-127, 127).to(torch.int8)
    out = torch.empty(rows, cols // 32, 34, dtype=torch.uint8, device=x.device)
    out[..., 0:2] = _half_bytes(scale).view(rows, cols // 32, 2)
    out[..., 2:] = q.view(torch.uint8)
    return out


def pack_q4_0(x):
    rows, cols = x.shape
    xb = x.view(rows, cols // 32, 32)
    idx = xb.abs().argmax(-1, keepdim=True)
    mx = xb.gather(-1, idx).squeeze(-1)
    d = mx / -8.0
    inv = torch.where(d != 0, 1.0 / d, torch.zeros_like(d))
    q = (xb * inv[..., None] + 8.5).to(torch.int32).clamp_(0, 15).to(torch.uint8)
    out = torch.empty(rows, cols // 32, 18, dtype=torch.uint8, device=x.device)
    out[..., 0:2] = _half_bytes(d).view(rows, cols // 32, 2)
    out[..., 2:] = q[..., :16] | (q[..., 16:] << 4)
    return out


def pack_q4_k(x):
    """x: [rows, cols] float32 (cols % 256 == 0) -> uint8 [rows, cols/256, 144]"""
    rows, cols = x.shape
    nsb = cols // 256
    xb = x.view(rows, nsb, 8, 32)
    lo = xb.amin(-1).clamp(max=0.0)
    hi = torch.maximum(xb.amax(-1), lo)
    step = (hi - lo) / 15.0
    d16 = (step.amax(-1) / 63.0).to(torch.float16)
    m16 = ((-lo).amax(-1) / 63.0).to(torch.float16)
    d = d16.float()[..., None]; dm = m16.float()[..., None]
    sc = torch.where(d > 0, torch.round(step / d), torch.zeros_like(step)).clamp_(0, 63)
    mn = torch.where(dm > 0, torch.round(-lo / dm), torch.zeros_like(lo)).clamp_(0, 63)
    ds = (d * sc)[..., None]; off = (dm * mn)[..., None]
    q = torch.where(ds > 0, torch.round((xb + off) / ds), torch.zeros_like(xb)).clamp_(0, 15).to(torch.uint8)
    sc = sc.to(torch.uint8); mn = mn.to(torch.uint8)
    out = torch.empty(rows, nsb, 144, dtype=torch.uint8, device=x.device)
    out[..., 0:2] = d16.view(torch.uint8).view(rows, nsb, 2)
    out[..., 2:4] = m16.view(torch.uint8).view(rows, nsb, 2)
    out[..., 4:8] = (sc[..., :4] & 63) | ((sc[..., 4:] >> 4) << 6)
    out[..., 8:12] = (mn[..., :4] & 63) | ((mn[..., 4:] >> 4) << 6)
    out[..., 12:16] = (sc[..., 4:] & 15) | ((mn[..., 4:] & 15) << 4)
    qs = q.view(rows, nsb, 4, 2, 32)
    out[..., 16:] = (qs[..., 0, :] | (qs[..., 1, :] << 4)).reshape(rows, nsb, 128)
    return out


def pack_q5_k(x):
    """x: [rows, cols] float32 (cols % 256 == 0) -> uint8 [rows, cols/256, 176]: the affine fit of pack_q4_k with 32 levels; the
    fifth bit of weight i of sub-block j is bit j of plane byte i (layout of neural/neuralgguf.pas:516-587)"""
    rows, cols = x.shape
    nsb = cols // 256
    xb = x.view(rows, nsb, 8, 32)
    lo = xb.amin(-1).clamp(max=0.0)
    hi = torch.maximum(xb.amax(-1), lo)
    step = (hi - lo) / 31.0
    d16 = (step.amax(-1) / 63.0).to(torch.float16)
    m16 = ((-lo).amax(-1) / 63.0).to(torch.float16)
    d = d16.float()[..., None]; dm = m16.float()[..., None]
    sc = torch.where(d > 0, torch.round(step / d), torch.zeros_like(step)).clamp_(0, 63)
    mn = torch.where(dm > 0, torch.round(-lo / dm), torch.zeros_like(lo)).clamp_(0, 63)
    ds = (d * sc)[..., None]; off = (dm * mn)[..., None]
    q = torch.where(ds > 0, torch.round((xb + off) / ds), torch.zeros_like(xb)).clamp_(0, 31).to(torch.uint8)
    sc = sc.to(torch.uint8); mn = mn.to(torch.uint8)
    out = torch.empty(rows, nsb, 176, dtype=torch.uint8, device=x.device)
    out[..., 0:2] = d16.view(torch.uint8).view(rows, nsb, 2)
    out[..., 2:4] = m16.view(torch.uint8).view(rows, nsb, 2)
    out[..., 4:8] = (sc[..., :4] & 63) | ((sc[..., 4:] >> 4) << 6)
    out[..., 8:12] = (mn[..., :4] & 63) | ((mn[..., 4:] >> 4) << 6)
    out[..., 12:16] = (sc[..., 4:] & 15) | ((mn[..., 4:] & 15) << 4)
    plane = torch.zeros(rows, nsb, 32, dtype=torch.uint8, device=x.device)
    for j in range(8):
        plane |= (q[..., j, :] >> 4) << j
    out[..., 16:48] = plane
    qs = (q & 15).view(rows, nsb, 4, 2, 32)
    out[..., 48:] = (qs[..., 0, :] | (qs[..., 1, :] << 4)).reshape(rows, nsb, 128)
    return out


def pack_q6_k(x):
    """x: [rows, cols] float32 (cols % 256 == 0) -> uint8 [rows, cols/256, 210]: symmetric fit, one signed scale per 16
    weights, codes q in 0..63 standing for q - 32 (layout of neural/neuralgguf.pas:639-717)"""
    rows, cols = x.shape
    nsb = cols // 256
    xg = x.view(rows, nsb, 16, 16)
    step = xg.abs().amax(-1) / 31.0
    d16 = (step.amax(-1) / 127.0).to(torch.float16)
    d = d16.float()[..., None]
    sc = torch.where(d > 0, torch.round(step / d), torch.zeros_like(step)).clamp_(0, 127)
    ds = (d * sc)[..., None]
    q = (torch.where(ds > 0, torch.round(xg / ds), torch.zeros_like(xg)).clamp_(-32, 31) + 32).to(torch.uint8)
    q = q.view(rows, nsb, 2, 4, 32)                       # [half][j][l]: weight 128 half + 32 j + l
    out = torch.empty(rows, nsb, 210, dtype=torch.uint8, device=x.device)
    lo = q & 15; hi = q >> 4
    ql = torch.stack([lo[..., 0, :] | (lo[..., 2, :] << 4), lo[..., 1, :] | (lo[..., 3, :] << 4)], dim=-2)   # [half][2][32]
    out[..., 0:128] = ql.reshape(rows, nsb, 128)
    out[..., 128:192] = (hi[..., 0, :] | (hi[..., 1, :] << 2) | (hi[..., 2, :] << 4) | (hi[..., 3, :] << 6)).reshape(rows, nsb, 64)
    out[..., 192:208] = sc.to(torch.int8).view(torch.uint8)
    out[..., 208:210] = d16.view(torch.uint8).view(rows, nsb, 2)
    return out


PACKERS = {cai.Q8_0: pack_q8_0, cai.Q4_0: pack_q4_0, cai.Q4_K: pack_q4_k, cai.Q5_K: pack_q5_k, cai.Q6_K: pack_q6_k}


def random_qweight(qtype, rows, cols, gen, std=0.02, bias=False, chunk_rows=32768, keep_bytes=False):
    """Resident random matrix of the given block type.  Returns (QWeight, bytes tensor or None)."""
    parts = []
    for r0 in range(0, rows, chunk_rows):
        r = min(chunk_rows, rows - r0)
        x = torch.randn(r, cols, device="cuda", dtype=torch.float32, generator=gen) * std
        parts.append(PACKERS[qtype](x).reshape(-1))
        del x
    raw = parts[0] if len(parts) == 1 else torch.cat(parts)
    b = None
    if bias:
        b = (torch.randn(rows, device="cuda", dtype=torch.float32, generator=gen) * std).cpu().numpy()
    torch.cuda.synchronize()
    w = cai.QWeight(qtype, rows, cols, raw.data_ptr(), b)
    return w, (raw if keep_bytes else None), b


# the block types kept as the stored stream: (elements, bytes, offsets of the f16 fields) per block
RAW_BLOCKS = {cai.Q4_1: (32, 20, (0, 2)), cai.Q5_0: (32, 22, (0,)), cai.Q5_1: (32, 24, (0, 2)),
              cai.Q2_K: (256, 84, (80, 82)), cai.Q3_K: (256, 110, (108,)), cai.Q5_K: (256, 176, (0, 2))}


def random_raw_qweight(qtype, rows, cols, gen):
    """Resident matrix of a stored-stream block type for timing: random code / scale bytes (every pattern is a valid block),
    the f16 fields set to a small positive half so that the values stay finite."""
    be, bb, halfs = RAW_BLOCKS[qtype]
    raw = torch.randint(0, 256, (rows * (cols // be), bb), device="cuda", dtype=torch.uint8, generator=gen)
    for h in halfs:
        raw[:, h] = 0x66; raw[:, h + 1] = 0x10
    torch.cuda.synchronize()
    return cai.QWeight(qtype, rows, cols, raw.data_ptr())


def random_int8_rows(rows, cols, gen, scale=1e-3):
    """Resident random matrix in the reference's per-row int8 format (codes in [-127, 127], one float scale per row)."""
    codes = torch.randint(-127, 128, (rows, cols), device="cuda", dtype=torch.int8, generator=gen)
    scales = torch.full((rows,), scale, device="cuda", dtype=torch.float32)
    torch.cuda.synchronize()
    return cai.QWeight(cai.I8ROW, rows, cols, codes.data_ptr(), None, scales.data_ptr())


def more_bits_layer(i, n):
    """The blocks whose attn_v and ffn_down a Q4_K_M export keeps in Q6_K (the first and last eighth and every third between)."""
    return i < n // 8 or i >= 7 * n // 8 or (i - n // 8) % 3 == 2


def random_decoder_spec(cfg, qtype, head_qtype, seed=424242, qkv_bias=False, std=0.02, keep_bytes=False, embed_qtype=None, q6k_mix=False):
    """Backend-neutral spec whose tensors are already resident (entry "qw"); norm gains are 1.
    q6k_mix: attn_v and ffn_down of the more_bits_layer blocks in Q6_K (the Q4_K_M mix)."""
    import numpy as np
    gen = torch.Generator(device="cuda"); gen.manual_seed(seed)
    d, hq, hkv, hd, I, V, L = cfg["d_model"], cfg["n_q_heads"], cfg["n_kv_heads"], cfg["head_dim"], cfg["ffn"], cfg["vocab"], cfg["n_layers"]
    ne = cfg.get("n_experts", 0)
    T, Vv = {}, {}

    def put(key, qt, rows, cols, bias=False):
        w, raw, b = random_qweight(qt, rows, cols, gen, std, bias, keep_bytes=keep_bytes)
        T[key] = dict(qw=w, type=qt, rows=rows, cols=cols, raw_dev=raw, bias=b)

    put((-1, cai.W_EMBED), embed_qtype if embed_qtype is not None else head_qtype, V, d)
    if not cfg.get("tied", False):
        put((-1, cai.W_HEAD), head_qtype, V, d)
    Vv[(-1, cai.V_FINAL_NORM)] = np.ones(d, np.float32)
    for l in range(L):
        put((l, cai.W_Q), qtype, hq * hd, d, qkv_bias)
        put((l, cai.W_K), qtype, hkv * hd, d, qkv_bias)
        hi = q6k_mix and more_bits_layer(l, L)
        put((l, cai.W_V), cai.Q6_K if hi else qtype, hkv * hd, d, qkv_bias)
        put((l, cai.W_O), qtype, d, hq * hd)
        Vv[(l, cai.V_ATTN_NORM)] = np.ones(d, np.float32)
        Vv[(l, cai.V_MLP_NORM)] = np.ones(d, np.float32)
        if cfg.get("qk_norm_full", 0):
            Vv[(l, cai.V_Q_NORM)] = np.ones(hq * hd, np.float32)
            Vv[(l, cai.V_K_NORM)] = np.ones(hkv * hd, np.float32)
        if ne:
            put((l, cai.W_ROUTER), qtype, ne, d)
            put((l, cai.W_GATEUP), qtype, ne * 2 * I, d)
            put((l, cai.W_DOWN), qtype, ne * d, I)
        else:
            put((l, cai.W_GATEUP), qtype, 2 * I, d)
            put((l, cai.W_DOWN), cai.Q6_K if hi else qtype, d, I)
    c = {k: v for k, v in cfg.items() if k != "tied"}
    return dict(cfg=c, tensors=T, vecs=Vv)


# ---- model folders for the layered decoder ----
def layered_config(width, ff, heads, kv_heads, dim, n_layers, vocab, window, conv=4, every=4, loop=None):
    """A Samanex configuration of real-model proportions: every `every`-th layer is a parallel one, the others are delta layers."""
    rec = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, conv=conv)
    par = dict(left=dict(heads=heads, kv_heads=max(1, kv_heads // 2), dim=dim, vdim=dim, scale=dim ** -0.5, mask=dict(size=window)), right=dict(rec, kv_heads=heads))
    layers = [dict(type="parallel" if i % every == every - 1 else "delta", mixer=par if i % every == every - 1 else rec, mlp=dict(kind="dense", ff=ff)) for i in range(n_layers)]
    return dict(architecture="Samanex", width=width, vocab=vocab, layers=layers, norm=dict(eps=1e-6), loop=loop or dict(start=0, stop=n_layers, times=1))


def kiruvik_config(width, ff, heads, kv_heads, dim, n_layers, vocab, block, conv=4, every=4, experts=32, top=4, state=128, vdim=64, groups=1):
    """A Kiruvik configuration of real-model proportions: every `every`-th layer is an attention, the others are Mamba-2 layers of twice
    the width inside; dense feed-forwards and mixtures (of as many active rows: `top` experts and a shared one of half) in turn."""
    att = dict(heads=heads, kv_heads=max(1, kv_heads // 2), dim=dim, vdim=dim, scale=dim ** -0.5, mask=dict(size=block), rot=dict(base=1e4, dims=dim))
    ssd = dict(heads=2 * width // vdim, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=1)
    moe = dict(kind="moe", expert=dict(ff=ff // (2 * top), limit=7.0), router=dict(experts=experts, top=top, scale=1.5), shared=dict(ff=ff // 2, limit=7.0))
    layers = [dict(type="attention" if i % every == every - 1 else "mamba2", mixer=att if i % every == every - 1 else ssd, mlp=moe if i % 2 else dict(kind="dense", ff=ff))
              for i in range(n_layers)]
    return dict(architecture="Kiruvik", width=width, vocab=vocab, layers=layers, norm=dict(eps=1e-6), residual_mult=0.8, loop=dict(start=0, stop=n_layers, times=1))


def gamanex_config(width, ff, heads, kv_heads, dim, n_layers, vocab, experts=32, top=4):
    """A Gamanex configuration of real-model proportions: every second layer reads the keys and values of the one before it; dense
    feed-forwards (two matrices, three halves of the width a gated one would have) and mixtures (of as many active rows) in turn."""
    att = dict(heads=heads, kv_heads=max(1, kv_heads // 2), dim=dim, vdim=dim, scale=dim ** -0.5, q_temp=dict(coef=0.1, every=256))
    moe = dict(kind="moe", expert=dict(ff=ff // top), router=dict(experts=experts, top=top))
    layers = [dict(type="attention", mixer=dict(att, kv_from=i - 1) if i % 2 else att, mlp=moe if i % 2 else dict(kind="dense", ff=ff * 3 // 2)) for i in range(n_layers)]
    return dict(architecture="Gamanex", width=width, vocab=vocab, layers=layers, norm=dict(eps=1e-6), logit_scale=0.5)


def zenorax_config(width, ff, heads, kv_heads, dim, n_layers, vocab, experts=32, top=8, taps=4):
    """A Zenorax configuration of real-model proportions: latent attention, attention with keys as values and forget-gate layers in turn,
    each with a mixture of `top` of `experts` experts (of as many active weights as a gated feed-forward of width `ff`)."""
    lat = dict(heads=heads, dim=dim, rot_dim=dim // 2, vdim=dim, kv_rank=4 * dim, q_rank=width * 3 // 8, scale=(1.5 * dim) ** -0.5,
               rot=dict(base=1e4, dims=dim // 2, scaling=dict(factor=8.0, original=4096, fast=32.0, slow=1.0)))
    att = dict(heads=heads, kv_heads=max(1, kv_heads // 2), dim=dim, vdim=dim, scale=dim ** -0.5, rot=dict(base=1e4, dims=dim, scaling=dict(factor=2.0)))
    rec = dict(heads=width // dim, dim=dim, vdim=dim)
    moe = dict(kind="moe", expert=dict(ff=ff * 3 // (2 * top)), router=dict(experts=experts, top=top, groups=dict(count=8, keep=4)))
    kinds = (("latent_attention", lat), ("attention", att), ("hgrn2", rec))
    layers = [dict(type=kinds[i % 3][0], mixer=kinds[i % 3][1], mlp=moe) for i in range(n_layers)]
    return dict(architecture="Zenorax", width=width, vocab=vocab, layers=layers, norm=dict(eps=1e-6), canon=dict(taps=taps), embedding=dict(scale=width ** 0.5), logit_softcap=30.0)


def layered_shapes(cfg, rank=128):
    """name -> (shape, standard deviation, mean) of every tensor of a layered model"""
    if cfg["architecture"] == "Kiruvik":
        return kiruvik_shapes(cfg)
    if cfg["architecture"] == "Gamanex":
        return gamanex_shapes(cfg)
    if cfg["architecture"] == "Zenorax":
        return zenorax_shapes(cfg)
    w, out = cfg["width"], {}

    def lin(name, rows, cols):
        out[name] = ((rows, cols), cols ** -0.5, 0.0)

    def norm(name):
        out[name] = ((w,), 0.1, 1.0); out[name + ".b"] = ((w,), 0.05, 0.0); out[name + ".alpha"] = ((), 0.0, 0.7)

    def delta(p, c, channel):
        kw, vw = c["kv_heads"] * c["dim"], c["heads"] * c["vdim"]
        for n, r in (("q", kw), ("k", kw), ("v", vw)):
            lin(p + n, r, w); out[p + n + ".conv"] = ((r, c["conv"]), 0.3, 0.25)
        lin(p + "b", c["heads"], w); out[p + "A_log"] = ((c["heads"],), 0.5, 0.0); out[p + "norm"] = ((c["vdim"],), 0.1, 1.0)
        if channel:
            lin(p + "a1", rank, w); lin(p + "a2", c["heads"] * c["dim"], rank); lin(p + "g1", rank, w); lin(p + "g2", vw, rank)
        else:
            lin(p + "a", c["heads"], w); lin(p + "g", vw, w)
        out[p + "dt_bias"] = ((c["heads"] * c["dim"] if channel else c["heads"],), 1.0, -3.0)
        lin(p + "o", w, vw)

    out["embed"] = ((cfg["vocab"], w), 1.0, 0.0)
    lin("head", cfg["vocab"], w); norm("final.norm")
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        norm(p + "norm1"); norm(p + "norm1b")
        if L["type"] == "delta":
            delta(p + "mix.", m, False)
        else:
            a = m["left"]
            lin(p + "mix.left.q", a["heads"] * a["dim"], w); lin(p + "mix.left.k", a["kv_heads"] * a["dim"], w); lin(p + "mix.left.v", a["kv_heads"] * a["vdim"], w)
            lin(p + "mix.left.o", w, a["heads"] * a["vdim"])
            out[p + "mix.left.q.norm"] = ((a["dim"],), 0.1, 1.0); out[p + "mix.left.k.norm"] = ((a["dim"],), 0.1, 1.0)
            delta(p + "mix.right.", m["right"], True)
            out[p + "mix.left.out"] = ((w,), 0.1, 1.0); out[p + "mix.right.out"] = ((w,), 0.1, 1.0)
        if L["mlp"]:
            norm(p + "norm2"); norm(p + "norm2b")
            lin(p + "mlp.gate", L["mlp"]["ff"], w); lin(p + "mlp.up", L["mlp"]["ff"], w); lin(p + "mlp.down", w, L["mlp"]["ff"])
    return out


def kiruvik_shapes(cfg):
    w, out = cfg["width"], {}

    def lin(name, rows, cols):
        out[name] = ((rows, cols), cols ** -0.5, 0.0)

    def norm(name):
        out[name] = ((w,), 0.1, 1.0); out[name + ".b"] = ((w,), 0.05, 0.0); out[name + ".alpha"] = ((), 0.0, 0.7)

    def glu(p, ff):
        lin(p + "gate", ff, w); lin(p + "up", ff, w); lin(p + "down", w, ff)

    out["embed"] = ((cfg["vocab"], w), 1.0, 0.0)
    lin("head", cfg["vocab"], w); lin("loop.in", w, 2 * w); norm("final.norm")
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        norm(p + "norm1"); norm(p + "norm1b")
        if L["type"] == "attention":
            for n, r in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                lin(p + "mix." + n, r, w); out[p + "mix." + n + ".b"] = ((r,), 0.1, 0.0)
            lin(p + "mix.g", m["heads"] * m["vdim"], w); lin(p + "mix.o", w, m["heads"] * m["vdim"]); out[p + "mix.o.b"] = ((w,), 0.1, 0.0)
        else:
            inner = m["heads"] * m["vdim"]; ch = inner + 2 * m["groups"] * m["state"]
            lin(p + "mix.in", inner + ch + m["heads"], w); lin(p + "mix.o", w, inner)
            out[p + "mix.conv"] = ((ch, m["conv"]), 0.3, 0.25); out[p + "mix.conv.b"] = ((ch,), 0.1, 0.0)
            out[p + "mix.dt_bias"] = ((m["heads"],), 1.0, -3.0); out[p + "mix.A_log"] = ((m["heads"],), 0.5, 0.0)
            out[p + "mix.D"] = ((m["heads"],), 0.1, 1.0); out[p + "mix.norm"] = ((inner,), 0.1, 1.0)
        f = L["mlp"]
        if f:
            norm(p + "norm2"); norm(p + "norm2b")
            if f["kind"] == "dense":
                glu(p + "mlp.", f["ff"])
            else:
                lin(p + "mlp.router", f["router"]["experts"], w); out[p + "mlp.correction"] = ((f["router"]["experts"],), 0.01, 0.0)
                for e in range(f["router"]["experts"]):
                    glu(p + "mlp.e%d." % e, f["expert"]["ff"])
                glu(p + "mlp.shared.", f["shared"]["ff"])
    return out


def gamanex_shapes(cfg):
    w, out = cfg["width"], {}

    def lin(name, rows, cols):
        out[name] = ((rows, cols), cols ** -0.5, 0.0)

    def vec(name, n, std, mean):
        out[name] = ((n,), std, mean)

    out["embed"] = ((cfg["vocab"], w), 1.0, 0.0)
    lin("head", cfg["vocab"], w); vec("final.norm", w, 0.1, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = "l%d." % i, L["mixer"], L["mlp"]
        lin(p + "mix.q", m["heads"] * m["dim"], w); vec(p + "mix.q.norm", m["heads"] * m["dim"], 0.1, 1.0)
        if m.get("kv_from") is None:
            lin(p + "mix.k", m["kv_heads"] * m["dim"], w); lin(p + "mix.v", m["kv_heads"] * m["vdim"], w); vec(p + "mix.k.norm", m["kv_heads"] * m["dim"], 0.1, 1.0)
        vec(p + "mix.r1", m["heads"], 0.1, 0.5); vec(p + "mix.r2", m["heads"], 0.1, 0.5); vec(p + "mix.pb", m["heads"], 0.5, -4.0)
        lin(p + "mix.o", w, m["heads"] * m["vdim"])
        for k in "12" if f else "1":
            vec(p + "norm" + k, w, 0.1, 1.0); vec(p + "ls" + k, w, 0.1, 0.5); lin(p + "rg" + k, w, w); vec(p + "rg" + k + ".b", w, 0.1, 0.0)
        if f and f["kind"] == "dense":
            lin(p + "mlp.up", f["ff"], w); lin(p + "mlp.down", w, f["ff"])
        elif f:
            lin(p + "mlp.router", f["router"]["experts"], w); vec(p + "mlp.router.b", f["router"]["experts"], 0.01, 0.0)
            for e in range(f["router"]["experts"]):
                x = p + "mlp.e%d." % e
                lin(x + "gate", f["expert"]["ff"], w); lin(x + "up", f["expert"]["ff"], w); lin(x + "down", w, f["expert"]["ff"])
    return out


def zenorax_shapes(cfg):
    w, out = cfg["width"], {}

    def lin(name, rows, cols):
        out[name] = ((rows, cols), cols ** -0.5, 0.0)

    def vec(name, n, std, mean):
        out[name] = ((n,), std, mean)

    out["embed"] = ((cfg["vocab"], w), w ** -0.5, 0.0)
    vec("final.norm", w, 0.1, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = "l%d." % i, L["mixer"], L["mlp"]
        a = p + "mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            vec(p + n, w, 0.1, 1.0)
        out[p + "canon1"] = ((w, cfg["canon"]["taps"]), 0.2, 0.1); vec(p + "dwa", i + 2, 0.05, 1.0 / (i + 2))
        if L["type"] == "latent_attention":
            lin(a + "dq", m["q_rank"], w); vec(a + "dq.norm", m["q_rank"], 0.1, 1.0); lin(a + "uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"])
            lin(a + "dkv", m["kv_rank"] + m["rot_dim"], w); vec(a + "dkv.norm", m["kv_rank"], 0.1, 1.0)
            lin(a + "uk", m["heads"] * m["dim"], m["kv_rank"]); lin(a + "uv", m["heads"] * m["vdim"], m["kv_rank"])
            lin(a + "g", m["heads"] * m["vdim"], w); lin(a + "o", w, m["heads"] * m["vdim"])
        elif L["type"] == "attention":
            lin(a + "q", m["heads"] * m["dim"], w); lin(a + "k", m["kv_heads"] * m["dim"], w); vec(a + "sink", m["heads"], 0.5, 0.0); lin(a + "o", w, m["heads"] * m["dim"])
        else:
            n = m["heads"] * m["dim"]
            lin(a + "q", n, w); lin(a + "f", n, w); lin(a + "v", m["heads"] * m["vdim"], w)
            vec(a + "f.b", n, 1.0, 2.0); vec(a + "lower", n, 0.05, 0.5); vec(a + "norm", m["vdim"], 0.1, 1.0); lin(a + "o", w, m["heads"] * m["vdim"])
        if f:
            lin(p + "mlp.router", f["router"]["experts"], w); vec(p + "mlp.correction", f["router"]["experts"], 0.01, 0.0)
            for e in range(f["router"]["experts"]):
                lin(p + "mlp.e%d.up" % e, f["expert"]["ff"], w); lin(p + "mlp.e%d.down" % e, w, f["expert"]["ff"])
    return out


def layered_active_weights(cfg):
    """linear weights one token of a prompt meets, the vocabulary left out"""
    import numpy as np
    total = 0
    for name, (shape, _, _) in layered_shapes(cfg).items():
        if len(shape) != 2 or name in ("embed", "head") or name.endswith(("conv", "canon1")):
            continue
        n = int(np.prod(shape))
        part = name.split(".")
        if len(part) > 2 and part[1] == "mlp" and part[2][0] == "e" and part[2][1:].isdigit():
            r = cfg["layers"][int(part[0][1:])]["mlp"]["router"]
            n = n * r["top"] / r["experts"]
        total += n
    return total


def write_layered_folder(folder, cfg, seed=0, rank=128):
    """config.json and model.safetensors with random bfloat16 weights (one random block, repeated from a random start)"""
    import json
    import os
    import struct

    import numpy as np
    rng = np.random.default_rng(seed)
    block = rng.standard_normal((1 << 22) + 4099, dtype=np.float32)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    shapes, head, at = layered_shapes(cfg, rank), {}, 0
    for name, (shape, _, _) in shapes.items():
        n = 2 * int(np.prod(shape, dtype=np.int64))
        head[name] = dict(dtype="BF16", shape=list(shape), data_offsets=[at, at + n]); at += n
    h = json.dumps(head).encode(); h += b" " * (-len(h) % 8)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h)
        for name, (shape, std, mean) in shapes.items():
            n = int(np.prod(shape, dtype=np.int64))
            bits = ((block * np.float32(std) + np.float32(mean)).view(np.uint32) >> 16).astype(np.uint16)
            k = int(rng.integers(0, 4096))
            while n > 0:
                m = min(n, bits.size - k)
                f.write(bits[k:k + m].tobytes()); n -= m; k = 0
