"""Plain float64 implementation of the Kamelorn decoder in numpy, one function per mechanism, whole sequences only (no cache, no state
carried between calls, no batching).  It is what the tests compare the layer-list worker with; it shares no code with the product path.

A model keeps n residual streams X_1 .. X_n per token, all equal to s_e E[tok] at the start; the layers run in their run order (a looped
group several times); logits = head(rms(sum of the streams)).  Each of a layer's sub-layers F (mixer, feed-forward) with its mixing
weights a [n], b [n], M [n, n] (from, to):
    u = sum_s a_s X_s;     X_t <- sum_s M[s, t] X_s + r b_t F(rms(u) w)
"""
import math

import numpy as np


def f64(a):
    return np.asarray(a, dtype=np.float64)


def logistic(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * logistic(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rms(y, w, eps):
    return y / np.sqrt((y * y).mean(-1, keepdims=True) + eps) * w


def rms_parts(y, w, parts, eps):
    """every one of `parts` equal consecutive parts of a row by its own root mean square"""
    z = y.reshape(y.shape[0], parts, -1)
    return (z / np.sqrt((z * z).mean(-1, keepdims=True) + eps)).reshape(y.shape) * w


def turn_halves(z, positions, dims, base):
    """z [T, ..., d]: dimension i < dims / 2 turns together with dimension i + dims / 2 by p base^(-2 i / dims); the rest pass"""
    n = dims // 2
    fr = float(base) ** (-2.0 * np.arange(n) / dims) if n else np.zeros(0)
    ang = f64(positions).reshape((-1,) + (1,) * (z.ndim - 1)) * fr
    lo, hi, rest = z[..., :n], z[..., n:2 * n], z[..., 2 * n:]
    return np.concatenate([lo * np.cos(ang) - hi * np.sin(ang), hi * np.cos(ang) + lo * np.sin(ang), rest], -1)


def latent_attention(h, W, p, mx, eps):
    T, H, dn, dr, dv, R = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    pos = np.arange(T)
    q = (h @ W[p + "q"].T).reshape(T, H, dn + dr)
    kv = h @ W[p + "dkv"].T
    c = rms(kv[:, :R], W[p + "dkv.norm"], eps)
    kr = turn_halves(kv[:, R:], pos, mx["rot"]["dims"], mx["rot"]["base"])
    qr = turn_halves(q[..., dn:], pos, mx["rot"]["dims"], mx["rot"]["base"])
    ku = (c @ W[p + "uk"].T).reshape(T, H, dn)
    v = (c @ W[p + "uv"].T).reshape(T, H, dv)
    out = np.zeros((T, H, dv))
    later = np.triu(np.ones((T, T), bool), 1)
    for hd in range(H):
        sc = (q[:, hd, :dn] @ ku[:, hd].T + qr[:, hd] @ kr.T) * mx["scale"]
        sc[later] = -np.inf
        e = np.exp(sc - sc.max(-1, keepdims=True))
        out[:, hd] = (e / e.sum(-1, keepdims=True)) @ v[:, hd]
    return (out.reshape(T, H * dv) * logistic(h @ W[p + "g"].T)) @ W[p + "o"].T


def causal_conv(x, w, b):
    """per channel, the last column of w meets the current token, zeros before the start"""
    T, taps = x.shape[0], w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(pad[j:j + T] * w[:, j] for j in range(taps)) + b


def ssm_scan(x, B, C, dt, a, D, state=None):
    """one head: x [T, v], B, C [T, n], dt [T], a = exp(A_log).  S_t = exp(-a dt_t) S_(t-1) + dt_t B_t x_t^T;  y_t = S_t^T C_t + D x_t"""
    T, n = B.shape
    S = np.zeros((n, x.shape[1])) if state is None else state.copy()
    y = np.zeros_like(x)
    for t in range(T):
        S = math.exp(-a * dt[t]) * S + dt[t] * np.outer(B[t], x[t])
        y[t] = S.T @ C[t] + D * x[t]
    return y, S


def mamba2(h, W, p, mx, eps):
    T, H, v, n, G = h.shape[0], mx["heads"], mx["vdim"], mx["state"], mx["groups"]
    inner = H * v
    z, xbc, dt = np.split(h @ W[p + "in"].T, [inner, 2 * inner + 2 * G * n], axis=1)
    xbc = silu(causal_conv(xbc, W[p + "conv"], W[p + "conv.b"]))
    x, B, C = np.split(xbc, [inner, inner + G * n], axis=1)
    dt = softplus(dt + W[p + "dt_bias"])
    y = np.zeros((T, inner))
    for hd in range(H):
        g = hd // (H // G)
        y[:, hd * v:(hd + 1) * v] = ssm_scan(x[:, hd * v:(hd + 1) * v], B[:, g * n:(g + 1) * n], C[:, g * n:(g + 1) * n], dt[:, hd],
                                             math.exp(W[p + "A_log"][hd]), W[p + "D"][hd])[0]
    return rms_parts(y * silu(z), W[p + "norm"], mx["norm_groups"], eps) @ W[p + "o"].T


def gated_ffn(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(h, router, top, scale):
    """sigmoid scores; the `top` largest (lowest index on ties); weights = their scores over their sum, times scale"""
    s = logistic(h @ router.T)
    idx = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    w = np.take_along_axis(s, idx, -1)
    return idx, w / (w.sum(-1, keepdims=True) + 1e-20) * scale


def mixture(h, W, p, mlp):
    idx, wgt = route(h, W[p + "router"], mlp["router"]["top"], mlp["router"]["scale"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(idx[t], wgt[t]):
            q = p + "e%d." % e
            out[t] += w * gated_ffn(h[t:t + 1], W[q + "gate"], W[q + "up"], W[q + "down"])[0]
    return out


def feed_forward(h, W, p, mlp):
    if mlp["kind"] == "dense":
        return gated_ffn(h, W[p + "gate"], W[p + "up"], W[p + "down"])
    return mixture(h, W, p, mlp)


def sublayer(X, W, p, norm_w, eps, mult, f):
    """X [n, T, width]: one sub-layer on the streams; all new streams from the old ones"""
    u = np.tensordot(W[p + "in"], X, 1)
    y = f(rms(u, norm_w, eps))
    return np.tensordot(W[p + "mix"].T, X, 1) + mult * W[p + "out"][:, None, None] * y


def run_order(cfg):
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return list(range(n))
    return list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n))


def layer(cfg, W, li, X):
    L, eps, p, mult = cfg["layers"][li], cfg["norm"]["eps"], "l%d." % li, cfg["residual_mult"]
    mixer = {"latent_attention": latent_attention, "mamba2": mamba2}[L["type"]]
    X = sublayer(X, W, p + "hc1.", W[p + "norm1"], eps, mult, lambda h: mixer(h, W, p + "mix.", L["mixer"], eps))
    if L.get("mlp"):
        X = sublayer(X, W, p + "hc2.", W[p + "norm2"], eps, mult, lambda h: feed_forward(h, W, p + "mlp.", L["mlp"]))
    return X


def forward(cfg, W, tokens, taps=None):
    """logits [T, vocab] of one whole sequence; taps: a list that receives the sum of the streams after every layer run"""
    x = W["embed"][list(tokens)] * cfg["embedding"]["scale"]
    X = np.stack([x] * cfg["streams"])
    for li in run_order(cfg):
        X = layer(cfg, W, li, X)
        if taps is not None:
            taps.append(X.sum(0))
    return rms(X.sum(0), W["final.norm"], cfg["norm"]["eps"]) @ W["head"].T
