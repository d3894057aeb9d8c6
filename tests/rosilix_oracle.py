"""Plain float64 implementation of the Rosilix decoder in numpy, one function per mechanism, whole sequences only (no cache, no batching, no
portions).  It is what the tests compare the layer-list worker with; it shares no code with the product path.

A model: x_t = s_e E[tok_t]; layers; logits = head(rms(x) w).  A layer, with n(y, w) = y / rms(y) * w:
    x <- x + n(mixer(n(x, norm1)), norm1b);   x <- x + n(ffn(n(x, norm2)), norm2b)        (the second line only if the layer has a feed-forward)
"""
import math

import numpy as np


def f64(a):
    return np.asarray(a, dtype=np.float64)


def logistic(z):
    return 1.0 / (1.0 + np.exp(-z))


def rms_unit(y, eps):
    """y over its root mean square (eps inside the root), along the last axis"""
    return y / np.sqrt((y * y).mean(-1, keepdims=True) + eps)


def norm(y, w, eps):
    return rms_unit(y, eps) * w


def turn_pairs(z, positions, dims, base):
    """z [T, ..., d]: dimensions 2 i and 2 i + 1 (i < dims / 2) turn together by p base^(-2 i / dims); dimensions from `dims` on pass"""
    if not dims:
        return z
    fr = float(base) ** (-2.0 * np.arange(dims // 2) / dims)
    ang = f64(positions).reshape((-1,) + (1,) * (z.ndim - 1)) * fr
    out = z.copy()
    u, v = z[..., 0:dims:2], z[..., 1:dims:2]
    out[..., 0:dims:2] = u * np.cos(ang) - v * np.sin(ang)
    out[..., 1:dims:2] = v * np.cos(ang) + u * np.sin(ang)
    return out


def visible(T, chunk=None, window=None):
    """[i, j]: row i sees key j: never a later one, with `chunk` only keys of its own chunk of positions (counted from 0), with `window` only
    keys less than that far back"""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    see = j <= i
    if chunk:
        see = see & (i // chunk == j // chunk)
    if window:
        see = see & (i - j < window)
    return see


def softmax(s, sink=None):
    """weights along the last axis; sink: a score that joins the denominator only"""
    m = s.max(-1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink)
    e = np.exp(s - m)
    return e / (e.sum(-1, keepdims=True) + (0.0 if sink is None else np.exp(sink - m)))


def mixing_factor(lq1, lk1, lq2, lk2, diff):
    """how much of the second map is taken off the first"""
    return math.exp((lq1 * lk1).sum()) - math.exp((lq2 * lk2).sum()) + diff


def difference(a1, a2, lam, diff, eps):
    """the two maps' outputs of every head [..., vdim] into one"""
    return rms_unit(a1 - lam * a2, eps) * (1.0 - diff)


def two_map_attention(q, k, v, see, scale, lam, diff, gate, eps):
    """q [T, H, 2, d], k [T, G, 2, d], v [T, G, dv], see [T, T], gate [T, H]: every head's combined, normed and gated output [T, H, dv]"""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = np.zeros((T, H, v.shape[-1]))
    for hd in range(H):
        g = hd // (H // G)
        maps = []
        for m in range(2):
            s = (q[:, hd, m] @ k[:, g, m].T) * scale
            maps.append(softmax(np.where(see, s, -np.inf)) @ v[:, g])
        out[:, hd] = difference(maps[0], maps[1], lam, diff, eps) * gate[:, hd:hd + 1]
    return out


def attention(h, W, p, mx, eps):
    """differential attention inside chunks"""
    T, H, G, d, dv = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    rot = mx.get("rot") or {"dims": 0, "base": 1.0}
    pos = np.arange(T)
    q = turn_pairs((h @ W[p + "q"].T).reshape(T, H, 2, d), pos, rot["dims"], rot["base"])
    k = turn_pairs((h @ W[p + "k"].T).reshape(T, G, 2, d), pos, rot["dims"], rot["base"])
    v = (h @ W[p + "v"].T).reshape(T, G, dv)
    lam = mixing_factor(W[p + "lq1"], W[p + "lk1"], W[p + "lq2"], W[p + "lk2"], mx["diff"])
    out = two_map_attention(q, k, v, visible(T, (mx.get("mask") or {}).get("size")), mx["scale"], lam, mx["diff"], logistic(h @ W[p + "g"].T), eps)
    return out.reshape(T, H * dv) @ W[p + "o"].T


def latent_rows(h, W, p, mx, eps):
    """what a layer with a down-projection of its own leaves in its cache: the normed latent and the turned key part"""
    R = mx["kv_rank"]
    kv = h @ W[p + "dkv"].T
    return norm(kv[:, :R], W[p + "dkv.norm"], eps), turn_pairs(kv[:, R:], np.arange(h.shape[0]), mx["rot"]["dims"], mx["rot"]["base"])


def latent_attention(h, rows, W, p, mx):
    """rows: (latent, key part), the layer's own or an earlier layer's"""
    T, H, dn, dr, dv = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    c, kr = rows
    q = (h @ W[p + "q"].T).reshape(T, H, dn + dr)
    qr = turn_pairs(q[..., dn:], np.arange(T), mx["rot"]["dims"], mx["rot"]["base"])
    ku, v = (c @ W[p + "uk"].T).reshape(T, H, dn), (c @ W[p + "uv"].T).reshape(T, H, dv)
    hidden = ~visible(T)
    gate = logistic(h @ W[p + "g"].T)
    out = np.zeros((T, H, dv))
    for hd in range(H):
        s = (q[:, hd, :dn] @ ku[:, hd].T + qr[:, hd] @ kr.T) * mx["scale"]
        s[hidden] = -np.inf
        out[:, hd] = (softmax(s, W[p + "sink"][hd]) @ v[:, hd]) * gate[:, hd:hd + 1]
    return out.reshape(T, H * dv) @ W[p + "o"].T


def feed_forward(h, up, down):
    return np.maximum(h @ up.T, 0.0) ** 2 @ down.T


def forward(cfg, W, tokens, taps=None):
    """logits [T, vocab] of one whole sequence; taps: a list that receives the residual after every layer"""
    eps = cfg["norm"]["eps"]
    x = W["embed"][list(tokens)] * cfg["embedding"]["scale"]
    cache = {}
    for li, L in enumerate(cfg["layers"]):
        p, mx = "l%d." % li, L["mixer"]
        h = norm(x, W[p + "norm1"], eps)
        if L["type"] == "latent_attention":
            if mx.get("kv_from") is None:
                cache[li] = latent_rows(h, W, p + "mix.", mx, eps)
            a = latent_attention(h, cache[li if mx.get("kv_from") is None else mx["kv_from"]], W, p + "mix.", mx)
        else:
            a = attention(h, W, p + "mix.", mx, eps)
        x = x + norm(a, W[p + "norm1b"], eps)
        if L.get("mlp"):
            y = feed_forward(norm(x, W[p + "norm2"], eps), W[p + "mlp.up"], W[p + "mlp.down"])
            x = x + norm(y, W[p + "norm2b"], eps)
        if taps is not None:
            taps.append(x.copy())
    return norm(x, W["final.norm"], eps) @ W["head"].T
