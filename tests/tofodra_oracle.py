"""Slow float64 definition of the Tofodra decoder, one function per mechanism, written from the
design's equations: dense attention one query at a time, a token-by-token recurrence, direct (not
absorbed) latent attention, no paging, no batching, nothing carried between calls.  It shares no
code with the package; the tests compare the engine (CPU tier and HIP kernels) with it.

A model is ``(cfg, st)``: the checkpoint's ``config.json`` as a dict and its tensors by name.
"""
from __future__ import annotations

import torch

F64 = torch.float64


def rms_norm(x, eps, w=None):
    """x / sqrt(mean(x^2) + eps) over the last axis, times w when there is one."""
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w.to(F64)


def silu(z):
    return z * torch.sigmoid(z)


def project(h, st, name):
    """W h for a weight stored [out, in], plus the bias under name + '.b' when there is one."""
    y = h @ st[name].to(F64).T
    return y + st[name + ".b"].to(F64) if name + ".b" in st else y


# ---- positions ---------------------------------------------------------------------------------

def rotate_half(x, pos, dims, base):
    """x [T, H, d]: among the first ``dims`` channels, i and i + dims / 2 turn together by
    pos * base^(-2 i / dims)."""
    y = x.clone()
    n = dims // 2
    for i in range(n):
        a = pos.to(F64) * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        y[..., i] = x[..., i] * c - x[..., i + n] * s
        y[..., i + n] = x[..., i + n] * c + x[..., i] * s
    return y


def rotate_pairs(x, pos, dims, base):
    """The same with the neighbours 2i and 2i + 1."""
    y = x.clone()
    for i in range(dims // 2):
        a = pos.to(F64) * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        y[..., 2 * i] = x[..., 2 * i] * c - x[..., 2 * i + 1] * s
        y[..., 2 * i + 1] = x[..., 2 * i + 1] * c + x[..., 2 * i] * s
    return y


# ---- retention -----------------------------------------------------------------------------------

def retention(q, k, v, decay):
    """q, k [T, H, d], v [T, H, dv], decay [H] -> S^T q of S = decay S + k v^T, token by token."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    g = torch.as_tensor(decay, dtype=F64)[:, None, None]
    for t in range(T):
        S = g * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def retention_mixer(h, m, st, p, eps):
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    pos = torch.arange(T)
    q = rotate_half(project(h, st, p + "q").view(T, H, d), pos, rot["dims"], rot["base"])
    k = rotate_half(project(h, st, p + "k").view(T, H, d), pos, rot["dims"], rot["base"]) * d ** -0.5
    v = project(h, st, p + "v").view(T, H, dv)
    o = rms_norm(retention(q, k, v, m["decay"]), eps).reshape(T, H * dv)
    return project(o * silu(project(h, st, p + "g")), st, p + "o")


# ---- softmax attention ---------------------------------------------------------------------------

def visible(i, window, keep):
    """Indices of the rows that row i attends: j <= i, and with a window (> 0) either fewer than
    ``window`` rows back or among the first ``keep``."""
    return [j for j in range(i + 1) if not window or i - j < window or j < keep]


def softmax_attention(q, k, v, scale, window=0, keep=0):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for i in range(T):
        js = visible(i, window, keep)
        for h in range(H):
            sc = (k[js, h // rep] @ q[i, h]) * scale
            e = torch.exp(sc - sc.max())
            out[i, h] = (e @ v[js, h // rep]) / e.sum()
    return out


def differential(a1, a2, lam, diff, eps):
    """a1 - lam a2 per head, divided by its root mean square, times 1 - diff."""
    return rms_norm(a1 - lam * a2, eps) * (1.0 - diff)


def diff_lambda(lq1, lk1, lq2, lk2, diff):
    def d(a, b):
        return torch.exp((a.to(F64) * b.to(F64)).sum())
    return d(lq1, lk1) - d(lq2, lk2) + diff


def differential_attention(q, k, v, scale, window, keep, lam, diff, eps):
    """q [T, H, 2, d], k [T, G, 2, d] (map 1, map 2), v [T, G, dv] shared by the maps."""
    a1 = softmax_attention(q[:, :, 0], k[:, :, 0], v, scale, window, keep)
    a2 = softmax_attention(q[:, :, 1], k[:, :, 1], v, scale, window, keep)
    return differential(a1, a2, lam, diff, eps)


def attention_mixer(h, m, st, p, eps):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    mask = m.get("mask") or {}
    q = project(h, st, p + "q").view(T, H, 2, d)
    k = project(h, st, p + "k").view(T, G, 2, d)
    v = project(h, st, p + "v").view(T, G, dv)
    diff = float(m["diff"])
    lam = diff_lambda(*(st[p + n] for n in ("lq1", "lk1", "lq2", "lk2")), diff)
    o = differential_attention(q, k, v, float(m["scale"]), int(mask.get("size") or 0),
                               int(mask.get("keep_first") or 0), lam, diff, eps)
    o = o.reshape(T, H * dv) * torch.sigmoid(h @ st[p + "g"].to(F64).T)
    return project(o, st, p + "o")


def latent_of(h, m, st, p, eps):
    """The cached parts of every token: normed latent [T, rank], rotated shared key [T, r]."""
    rank = m["kv_rank"]
    down = project(h, st, p + "dkv")
    rot = m.get("rot") or {"dims": m["rot_dim"], "base": 10000.0}
    kr = rotate_pairs(down[:, None, rank:], torch.arange(h.shape[0]), rot["dims"], rot["base"])
    return rms_norm(down[:, :rank], eps, st[p + "dkv.norm"]), kr[:, 0]


def latent_mixer(h, m, st, p, eps, shared, layer):
    """``shared``: layer index -> its latent and rotated key, for the layers that read them."""
    H, d, r, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    T = h.shape[0]
    src = m.get("kv_from")
    if src is None:
        shared[layer] = latent_of(h, m, st, p, eps)
    c, kr = shared[layer if src is None else src]
    q = project(h, st, p + "q").view(T, H, d + r)
    rot = m.get("rot") or {"dims": r, "base": 10000.0}
    qr = rotate_pairs(q[..., d:], torch.arange(T), rot["dims"], rot["base"])
    k = torch.cat([(c @ st[p + "uk"].to(F64).T).view(T, H, d), kr[:, None].expand(T, H, r)], -1)
    v = (c @ st[p + "uv"].to(F64).T).view(T, H, dv)
    o = softmax_attention(torch.cat([q[..., :d], qr], -1), k, v, float(m["scale"]))
    return project(o.reshape(T, H * dv), st, p + "o")


# ---- feed-forward --------------------------------------------------------------------------------

def clamped_glu(g, u, limit):
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def dense_ff(h, mlp, st, p):
    a = clamped_glu(project(h, st, p + "gate"), project(h, st, p + "up"), float(mlp["limit"]))
    return project(a, st, p + "down")


def silu_glu(h, st, p):
    return project(silu(project(h, st, p + "gate")) * project(h, st, p + "up"), st, p + "down")


def route(z, top, scale):
    """One token's router logits -> (the ``top`` with the largest sigmoid scores, weights, the gap
    between the logits of the last one chosen and the best one left out)."""
    srt = torch.sort(z, descending=True)     # the sigmoid keeps the order
    gap = float(srt.values[top - 1] - srt.values[top]) if z.shape[0] > top else 1e9
    w = torch.sigmoid(srt.values[:top])
    return srt.indices[:top], w / (w.sum() + 1e-20) * scale, gap


def moe_ff(h, mlp, st, p, gaps=None):
    r = mlp["router"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        idx, w, gap = route(st[p + "router"].to(F64) @ h[t], int(r["top"]), float(r["scale"]))
        if gaps is not None:
            gaps.append(gap)
        for e, we in zip(idx.tolist(), w):
            out[t] += we * silu_glu(h[t:t + 1], st, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        out += silu_glu(h, st, p + "shared.")
    return out


# ---- the decoder ----------------------------------------------------------------------------------

def sublayer(x, y, w, ls, eps):
    """Residual plus a branch that is normed and scaled channel by channel first."""
    return x + rms_norm(y, eps, w) * ls.to(F64)


def forward(cfg, st, tokens, layers_out=None, gaps=None):
    """Logits [T, vocab] of a whole sequence."""
    eps = float(cfg["norm"]["eps"])
    x = st["embed"].to(F64)[torch.as_tensor(tokens)] * float(cfg["embedding"]["scale"])
    shared = {}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rms_norm(x, eps, st[p + "norm1"])
        if L["type"] == "attention":
            y = attention_mixer(h, L["mixer"], st, p + "mix.", eps)
        elif L["type"] == "latent_attention":
            y = latent_mixer(h, L["mixer"], st, p + "mix.", eps, shared, i)
        else:
            y = retention_mixer(h, L["mixer"], st, p + "mix.", eps)
        x = sublayer(x, y, st[p + "norm1b"], st[p + "ls1"], eps)
        if L.get("mlp"):
            h = rms_norm(x, eps, st[p + "norm2"])
            y = (dense_ff(h, L["mlp"], st, p + "mlp.") if L["mlp"]["kind"] == "dense" else
                 moe_ff(h, L["mlp"], st, p + "mlp.", gaps))
            x = sublayer(x, y, st[p + "norm2b"], st[p + "ls2"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, eps, st["final.norm"]) @ st["head"].to(F64).T
