"""Slow float64 definition of the Kolotar decoder, one function per mechanism, written from the
design's equations: dense attention over whole sequences one query at a time, a token-by-token
recurrence, no paging, no batching, nothing carried between calls.  It shares no code with the
package; the tests compare the engine (CPU tier and HIP kernels) with it.

A model is ``(cfg, st)``: the checkpoint's ``config.json`` as a dict and its tensors by name.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms_norm(x, eps, w=None):
    """x / sqrt(mean(x^2) + eps) over the last axis, times w when there is one."""
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w.to(F64)


def silu(z):
    return z * torch.sigmoid(z)


def project(h, st, name):
    """W h for a weight stored [out, in], plus the bias stored under name + '.b' when there is one
    and it is a vector of that many outputs."""
    y = h @ st[name].to(F64).T
    return y + st[name + ".b"].to(F64) if name + ".b" in st else y


# ---- positions ---------------------------------------------------------------------------------

def frequencies(dims, base, scaling=None):
    """(dims / 2 angular frequencies, factor on cos and sin).  Without scaling base^(-2i/dims) and
    1.  With it (YaRN): pair i turns original * f_i / (2 pi) times inside the original context;
    pairs that turn more than ``fast`` times keep their frequency, pairs below ``slow`` turns have
    it divided by ``factor``, with a linear ramp in the pair's index between the two."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return torch.tensor(f, dtype=F64), 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def index_of(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(index_of(float(scaling["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001)))
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(factor) + 1.0


def rotate_half(x, pos, dims, base, scaling=None):
    """x [T, H, d]: among the first ``dims`` channels channel i pairs with i + dims / 2."""
    if dims == 0:
        return x
    n = dims // 2
    f, mult = frequencies(dims, base, scaling)
    ang = pos.to(F64)[:, None] * f
    c, s = (torch.cos(ang) * mult)[:, None], (torch.sin(ang) * mult)[:, None]
    y = x.clone()
    u, v = x[..., :n], x[..., n:dims]
    y[..., :n] = u * c - v * s
    y[..., n:dims] = v * c + u * s
    return y


def rotate_pairs(x, pos, dims, base):
    """x [T, H, d]: among the first ``dims`` channels channel 2i pairs with 2i + 1."""
    y = x.clone()
    f, _ = frequencies(dims, base)
    for i in range(dims // 2):
        a = pos.to(F64) * f[i]
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        y[..., 2 * i] = x[..., 2 * i] * c - x[..., 2 * i + 1] * s
        y[..., 2 * i + 1] = x[..., 2 * i + 1] * c + x[..., 2 * i] * s
    return y


# ---- softmax attention ---------------------------------------------------------------------------

def window_softmax_attention(q, k, v, scale, window, sink=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv].  Row i attends rows j with 0 <= i - j < window
    (0: every earlier row); with ``sink`` [H] the denominator of head h also holds exp(sink[h])."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        for i in range(T):
            lo = max(0, i - window + 1) if window else 0
            sc = (k[lo:i + 1, h // rep] @ q[i, h]) * scale
            m = sc.max() if sink is None else torch.maximum(sc.max(), sink[h])
            e = torch.exp(sc - m)
            den = e.sum() if sink is None else e.sum() + torch.exp(sink[h] - m)
            out[i, h] = (e @ v[lo:i + 1, h // rep]) / den
    return out


def attention_mixer(h, m, st, p, eps, shared):
    """``shared``: a dict that carries the first mixing layer's values through the stack."""
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = rms_norm(project(h, st, p + "q").view(T, H, d), eps, st[p + "q.norm"])
    k = rms_norm(project(h, st, p + "k").view(T, G, d), eps, st[p + "k.norm"])
    v = rms_norm(project(h, st, p + "v").view(T, G, dv), eps)
    rot = m.get("rot") or {}
    args = (torch.arange(T), int(rot.get("dims", 0)), rot.get("base", 1.0), rot.get("scaling"))
    q, k = rotate_half(q, *args), rotate_half(k, *args)
    if m.get("v_mix"):
        if "v" in shared:
            lam = float(st[p + "vmix"])
            v = (1.0 - lam) * v + lam * shared["v"]
        else:
            shared["v"] = v
    o = window_softmax_attention(q, k, v, float(m["scale"]), int((m.get("mask") or {}).get("size") or 0),
                                 st[p + "sink"].to(F64))
    o = o * torch.sigmoid(h @ st[p + "g"].to(F64).T)[:, :, None]
    return project(o.reshape(T, H * dv), st, p + "o")


def latent_mixer(h, m, st, p, eps):
    """Latent attention in its direct form: keys and values are up-projected for every head."""
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = h.shape[0]
    pos = torch.arange(T)
    rot = m["rot"]
    q = project(h, st, p + "q").view(T, H, d + r)
    down = project(h, st, p + "dkv")
    c = rms_norm(down[:, :rank], eps, st[p + "dkv.norm"])
    kr = rotate_pairs(down[:, None, rank:], pos, int(rot["dims"]), rot["base"])
    qr = rotate_pairs(q[..., d:], pos, int(rot["dims"]), rot["base"])
    k = torch.cat([(c @ st[p + "uk"].to(F64).T).view(T, H, d), kr.expand(T, H, r)], -1)
    v = (c @ st[p + "uv"].to(F64).T).view(T, H, dv)
    o = window_softmax_attention(torch.cat([q[..., :d], qr], -1), k, v, float(m["scale"]),
                                 int((m.get("mask") or {}).get("size") or 0))
    return project(o.reshape(T, H * dv) * torch.sigmoid(h @ st[p + "g"].to(F64).T), st, p + "o")


# ---- sigmoid attention with talking heads ---------------------------------------------------------

def query_temperature(pos, coef, every):
    return 1.0 + coef * torch.log(torch.floor((pos.to(F64) + 1.0) / every) + 1.0)


def talking_sigmoid_attention(q, k, v, scale, softcap, bias, talk):
    """q [T, H, d], k [T, G, d], v [T, G, dv], bias [H], talk [H, H].  Row i gives every row
    j <= i the weight sigmoid(cap tanh(scale q.k / cap) + bias[g]) in head g, unnormalised; head h
    uses sum_g talk[h, g] weight_g on the values of its own key / value head."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    kh, vh = k.repeat_interleave(rep, 1), v.repeat_interleave(rep, 1)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for i in range(T):
        sc = torch.einsum("hd,jhd->hj", q[i], kh[:i + 1]) * scale
        if softcap:
            sc = softcap * torch.tanh(sc / softcap)
        w = torch.sigmoid(sc + bias[:, None])
        out[i] = torch.einsum("hj,jhd->hd", talk @ w, vh[:i + 1])
    return out


def sigmoid_mixer(h, m, st, p, eps):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = rms_norm(project(h, st, p + "q"), eps, st[p + "q.norm"]).view(T, H, d)
    k = rms_norm(project(h, st, p + "k"), eps, st[p + "k.norm"]).view(T, G, d)
    v = project(h, st, p + "v").view(T, G, dv)
    if m.get("q_temp"):
        t = query_temperature(torch.arange(T), float(m["q_temp"]["coef"]), float(m["q_temp"]["every"]))
        q = q * t[:, None, None]
    o = talking_sigmoid_attention(q, k, v, float(m["scale"]), float(m.get("softcap") or 0.0),
                                  st[p + "pb"].to(F64), st[p + "talk"].to(F64))
    return project(o.reshape(T, H * dv), st, p + "o")


# ---- gated delta rule -----------------------------------------------------------------------------

def short_conv(x, w):
    """x [T, C], w [C, taps] (last column: the current token): causal sum over time, then SiLU."""
    taps = w.shape[1]
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            if t - j >= 0:
                y[t] += x[t - j] * w[:, taps - 1 - j].to(F64)
    return silu(y)


def delta_rule(q, k, v, beta, g):
    """q, k [T, H, d], v [T, H, dv], beta, g [T, H] -> o [T, H, dv]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def delta_mixer(h, m, st, p, eps):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]

    def unit(x):
        return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)

    def heads(name, n, width):
        return short_conv(h @ st[p + name].to(F64).T, st[p + name + ".conv"]).view(T, n, width)

    q = unit(heads("q", G, d)) * d ** -0.5
    k = unit(heads("k", G, d))
    v = heads("v", H, dv)
    beta = torch.sigmoid(h @ st[p + "b"].to(F64).T)
    z = h @ st[p + "a"].to(F64).T + st[p + "dt_bias"].to(F64)
    g = torch.exp(-torch.exp(st[p + "A_log"].to(F64)) * torch.nn.functional.softplus(z))
    o = delta_rule(q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1), v, beta, g)
    o = rms_norm(o, eps, st[p + "norm"]) * silu(h @ st[p + "g"].to(F64).T).view(T, H, dv)
    return o.reshape(T, H * dv) @ st[p + "o"].to(F64).T


def parallel_mixer(h, m, st, p, eps):
    return float(m["left_scale"]) * sigmoid_mixer(h, m["left"], st, p + "left.", eps) + \
        float(m["right_scale"]) * delta_mixer(h, m["right"], st, p + "right.", eps)


# ---- routed experts -------------------------------------------------------------------------------

def route(z, top):
    """One token's router logits -> (the ``top`` largest, softmax over just those, the gap to the
    best one left out)."""
    srt = torch.sort(z, descending=True)
    gap = float(srt.values[top - 1] - srt.values[top]) if z.shape[0] > top else 1e9
    return srt.indices[:top], torch.softmax(srt.values[:top], 0), gap


def moe_ff(h, mlp, st, p, gaps=None):
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        z = st[p + "router"].to(F64) @ h[t] + st[p + "router.b"].to(F64)
        idx, w, gap = route(z, int(mlp["router"]["top"]))
        if gaps is not None:
            gaps.append(gap)
        for e, we in zip(idx.tolist(), w):
            q = f"{p}e{e}."
            a = silu(st[q + "gate"].to(F64) @ h[t]) * (st[q + "up"].to(F64) @ h[t])
            out[t] += we * (st[q + "down"].to(F64) @ a)
    return out


# ---- the decoder ----------------------------------------------------------------------------------

def post_norm(x, y, alpha, w, eps):
    return rms_norm(alpha * x + y, eps, w)


def forward(cfg, st, tokens, layers_out=None, gaps=None):
    """Logits [T, vocab] of a whole sequence."""
    eps, alpha = float(cfg["norm"]["eps"]), float(cfg["postln_alpha"])
    x = st["embed"].to(F64)[torch.as_tensor(tokens)]
    shared = {}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        if L["type"] == "attention":
            y = attention_mixer(x, L["mixer"], st, p + "mix.", eps, shared)
        elif L["type"] == "latent_attention":
            y = latent_mixer(x, L["mixer"], st, p + "mix.", eps)
        else:
            y = parallel_mixer(x, L["mixer"], st, p + "mix.", eps)
        x = post_norm(x, y, alpha, st[p + "norm1"], eps)
        if L.get("mlp"):
            x = post_norm(x, moe_ff(x, L["mlp"], st, p + "mlp.", gaps), alpha, st[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, eps, st["final.norm"]) @ st["embed"].to(F64).T
