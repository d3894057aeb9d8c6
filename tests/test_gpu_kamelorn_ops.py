"""Each mechanism that the Kamelorn layers add to the layer-list worker alone, through its C-ABI op, against the float64 functions of
tests/kamelorn_oracle.py: the residual streams' step (embedding, update, read-out, norm, sum), the convolution over a
ring, the state space in its three forms (single tokens, chunks, token by token; continued states, several sequences, reused slots), the gate in
front of the norm in parts, latent attention rotated in halves with a gate per column in both forms, the renormalized router, also inside the
experts' first launch."""
import ctypes as C

import numpy as np
import pytest
import torch

import inferflow_amd as ia
from tests import kamelorn_oracle as orc
from tests.gelarax_oracle import bf16_round
from tests.gpu_util import capi, p, sync
from tests.test_gpu_layered_ops import Slots, dev32, devbf, devi, seq_tables

pytestmark = pytest.mark.gpu


def host_seqs(seqs):
    h, r = [], 0
    for n, pos0, slot in seqs:
        h += [r, n, pos0, slot]; r += n
    return (C.c_int * len(h))(*h)


def near(got, want, tol=2e-6):
    return np.abs(got - want).max() < tol * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("rows,S,cols", [(1, 1, 64), (5, 2, 96), (33, 4, 40), (3, 3, 14), (2, 2, 5000), (1, 4, 2048), (2, 8, 260), (3, 16, 132), (2, 7, 9), (1, 5, 20004)])
def test_streams_step(rows, S, cols):
    rng = np.random.default_rng(rows + cols + S)
    X = rng.standard_normal((rows, S, cols)).astype(np.float32)
    y = rng.standard_normal((rows, cols + 4)).astype(np.float32)
    W = {"p.in": bf16_round(rng.standard_normal(S)), "p.out": bf16_round(rng.standard_normal(S)), "p.mix": bf16_round(rng.standard_normal((S, S)))}
    nin, nw = bf16_round(rng.standard_normal(S)), bf16_round(1 + 0.3 * rng.standard_normal(cols))
    mult, eps = 0.37, 1e-3
    L = capi()
    Xs = orc.f64(X).transpose(1, 0, 2)
    new = orc.sublayer(Xs, {k: orc.f64(v) for k, v in W.items()}, "p.", np.ones(cols), eps, mult, lambda h: orc.f64(y[:, :cols]))
    u = np.tensordot(orc.f64(nin), new, 1)
    xd, h, s = dev32(X), torch.full((rows, cols + 4), 7.0, dtype=torch.float32, device="cuda"), torch.full((rows, cols + 1), 7.0, dtype=torch.float32, device="cuda")
    ia.check(L.ifa_streams_step_f32(p(xd), rows, S, cols, None, None, 0, 1.0, p(dev32(y)), cols + 4, p(devbf(W["p.mix"])), p(devbf(W["p.out"])), mult, p(devbf(nin)), p(devbf(nw)),
                                    eps, p(h), cols + 4, p(s), cols + 1, None)); sync()
    assert near(xd.cpu().numpy().transpose(1, 0, 2), new) and near(s.cpu().numpy()[:, :cols], u) and np.all(s.cpu().numpy()[:, cols:] == 7.0)
    assert near(h.cpu().numpy()[:, :cols], orc.rms(u, orc.f64(nw), eps), 5e-6) and np.all(h.cpu().numpy()[:, cols:] == 7.0)
    # nothing to add: the streams stay as they are; the plain sum without read-out weights
    xd = dev32(X)
    ia.check(L.ifa_streams_step_f32(p(xd), rows, S, cols, None, None, 0, 1.0, None, 0, None, None, 1.0, None, p(devbf(nw)), eps, p(h), cols + 4, None, 0, None)); sync()
    assert np.array_equal(xd.cpu().numpy(), X) and near(h.cpu().numpy()[:, :cols], orc.rms(Xs.sum(0), orc.f64(nw), eps), 5e-6)
    # the start of the stack: every stream the scaled embedding; mix / out absent: identity / ones
    E, toks = bf16_round(rng.standard_normal((11, cols))), [int(t) for t in rng.integers(0, 11, rows)]
    xd = dev32(X)
    ia.check(L.ifa_streams_step_f32(p(xd), rows, S, cols, p(devbf(E)), p(devi(toks)), 11, 2.5, None, 0, None, None, 1.0, p(devbf(nin)), p(devbf(nw)), eps, p(h), cols + 4, None, 0,
                                    None)); sync()
    e = orc.f64(E)[toks] * 2.5
    assert near(xd.cpu().numpy(), np.stack([e] * S, 1)) and near(h.cpu().numpy()[:, :cols], orc.rms(e * orc.f64(nin).sum(), orc.f64(nw), eps), 2e-5)
    ia.check(L.ifa_streams_step_f32(p(xd), rows, S, cols, None, None, 0, 1.0, p(dev32(y)), cols + 4, None, None, mult, None, None, eps, None, 0, None, 0, None)); sync()
    assert near(xd.cpu().numpy(), np.stack([e + mult * y[:, :cols]] * S, 1))


@pytest.mark.parametrize("rows,W,F,E,top,kind", [(1, 64, 24, 6, 2, 1), (3, 256, 40, 32, 6, 1), (8, 40, 10, 16, 1, 1), (2, 64, 16, 5, 5, 1), (2, 72, 9, 70, 8, 0), (1, 14, 6, 256, 3, 1),
                                                  (2, 16, 8, 3, 2, 0), (1, 8, 1, 1, 1, 1)])
def test_experts_with_the_choice_inside_their_first_launch(rows, W, F, E, top, kind):
    rng = np.random.default_rng(rows + W + E)
    h = rng.standard_normal((rows, W)).astype(np.float32)
    router = bf16_round(rng.standard_normal((E, W)) * 2 / np.sqrt(W))
    corr = bf16_round(0.2 * rng.standard_normal(E)) if kind == 0 else None
    if E >= 5:
        router[3] = router[1]          # a tie: the lower index wins
        if corr is not None:
            corr[3] = corr[1]
    gate, up, down = (bf16_round(rng.standard_normal(s) * 0.3) for s in ((E, F, W), (E, F, W), (E, W, F)))
    logits = (orc.f64(h) @ orc.f64(router).T).astype(np.float32)
    if kind == 1:
        idx_w, wgt_w = orc.route(orc.f64(h), orc.f64(router), top, 1.7)
    else:
        z = orc.f64(logits); sc = np.exp(z - z.max(-1, keepdims=True)); sc /= sc.sum(-1, keepdims=True)
        idx_w = np.argsort(-(sc + orc.f64(corr)), axis=-1, kind="stable")[:, :top]
        wgt_w = np.take_along_axis(sc, idx_w, -1); wgt_w = wgt_w / wgt_w.sum(-1, keepdims=True) * 1.7
    want = np.zeros((rows, W))
    for t in range(rows):
        for e, wv in zip(idx_w[t], wgt_w[t]):
            want[t] += wv * orc.gated_ffn(orc.f64(h[t:t + 1]), orc.f64(gate[e]), orc.f64(up[e]), orc.f64(down[e]))[0]
    L = capi()
    nb = L.ifa_moe_workspace_bytes(rows, top, W, 3 * F, E)
    ws = torch.empty((nb,), dtype=torch.uint8, device="cuda")
    idx, wgt = torch.full((rows, top), -1, dtype=torch.int32, device="cuda"), torch.zeros((rows, top), dtype=torch.float32, device="cuda")
    y = torch.zeros((rows, W), dtype=torch.float32, device="cuda")
    gu, dd, dh, dl = devbf(np.concatenate([gate, up], 1).reshape(E * 2 * F, W)), devbf(down.reshape(E * W, F)), dev32(h), dev32(logits)
    dc = devbf(corr) if corr is not None else None
    ia.check(L.ifa_moe_experts_routed_rows_f32(kind, 1, 1e-20, 1.7, p(dl), E, p(dc) if dc is not None else None, 0, 0.0, p(dh), W, rows, W, F, E, top, p(gu), p(dd), p(idx), p(wgt), p(ws),
                                               nb, p(y), W, 0, None)); sync()
    assert np.array_equal(idx.cpu().numpy(), idx_w) and near(wgt.cpu().numpy(), wgt_w, 5e-6) and near(y.cpu().numpy(), want, 2e-5)
    # without renormalization: the plain scores
    ia.check(L.ifa_moe_experts_routed_rows_f32(kind, 0, 0.0, 1.0, p(dl), E, p(dc) if dc is not None else None, 0, 0.0, p(dh), W, rows, W, F, E, top, p(gu), p(dd), p(idx), p(wgt), p(ws),
                                               nb, p(y), W, 0, None)); sync()
    plain = wgt.cpu().numpy()
    assert near(plain / plain.sum(-1, keepdims=True) * 1.7, wgt_w, 5e-6)
    if kind == 1:
        assert near(plain, orc.logistic(np.take_along_axis(orc.f64(logits), idx_w, -1)), 5e-6)


@pytest.mark.parametrize("T,n_all,top,scale", [(9, 6, 2, 2.5), (70, 16, 1, 0.3), (5, 5, 5, 1.0), (12, 70, 8, 3.0)])
def test_renormalized_router_in_both_forms(T, n_all, top, scale):
    rng = np.random.default_rng(n_all + top)
    W = 40
    h, router = rng.standard_normal((T, W)).astype(np.float32), bf16_round(rng.standard_normal((n_all, W)) * 0.4)
    if n_all >= 5:
        router[3] = router[1]          # a tie: the lower index wins
    idx_w, wgt_w = orc.route(orc.f64(h), orc.f64(router), top, scale)
    L = capi()
    logits = (orc.f64(h) @ orc.f64(router).T).astype(np.float32)
    for form in ("logits", "rows"):
        if form == "rows" and T > 64:
            continue
        idx, wgt = torch.full((T, top), -1, dtype=torch.int32, device="cuda"), torch.zeros((T, top), dtype=torch.float32, device="cuda")
        if form == "logits":
            ia.check(L.ifa_moe_route_renorm_f32(1, 1, 1e-20, scale, p(dev32(logits)), n_all, T, n_all, top, None, p(idx), p(wgt), None))
        else:
            ia.check(L.ifa_moe_route_rows_renorm_f32(1, 1, 1e-20, scale, p(dev32(h)), W, T, W, p(devbf(router)), n_all, top, None, p(idx), p(wgt), None))
        sync()
        assert np.array_equal(idx.cpu().numpy(), idx_w), form
        assert near(wgt.cpu().numpy(), wgt_w, 5e-6), form


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("channels", [5, 300])
def test_convolution_over_a_ring_in_portions_and_on_reused_slots(taps, channels):
    rng = np.random.default_rng(taps * 10 + channels)
    T = 75
    w, b = bf16_round(rng.standard_normal((channels, taps))), bf16_round(rng.standard_normal(channels))
    seqs = [rng.standard_normal((T, channels)).astype(np.float32) for _ in range(3)]
    want = [orc.silu(orc.causal_conv(orc.f64(x), orc.f64(w), orc.f64(b))) for x in seqs]
    L = capi()
    slots = Slots(2, 4 + taps * channels)
    at = [0, 0, 0]
    wd, bd = devbf(w), devbf(b)
    gate = torch.zeros((256, 1), dtype=torch.float32, device="cuda")
    one = devbf(np.zeros(1, np.float32))
    plan = [[(0, 1, 0), (1, 2, 1)], [(0, 1, 0)], [(0, 2, 0), (1, 73, 1)], [(2, 3, 1), (0, 1, 0)], [(0, 40, 0), (2, 1, 1)], [(0, 30, 0), (2, 71, 1)]]
    for step in plan:
        d, rs, rows = seq_tables([(n, at[q], slot) for q, n, slot in step])
        x = np.concatenate([seqs[q][at[q]:at[q] + n] for q, n, _ in step])
        xd = dev32(np.concatenate([x, np.full((rows, 2), 9.0, np.float32)], 1))
        y = torch.full((rows, channels + 1), 7.0, dtype=torch.float32, device="cuda")
        ia.check(L.ifa_conv_ring_silu_f32(p(xd), channels + 2, channels, taps, p(wd), p(bd), p(d), p(rs), rows, p(slots.table), 4, p(y), channels + 1, None))
        ia.check(L.ifa_ssm_gates_ring_f32(p(gate), 1, 1, rows, p(one), p(one), p(torch.empty_like(gate)), p(torch.empty_like(gate)), p(xd), channels + 2, channels, taps, p(d), len(step),
                                          p(slots.table), 4, None))
        sync()
        got, r0 = y.cpu().numpy(), 0
        assert np.all(got[:, channels:] == 7.0)
        for q, n, _ in step:
            assert near(got[r0:r0 + n, :channels], want[q][at[q]:at[q] + n], 5e-6), (q, at[q], n)
            r0 += n; at[q] += n
    assert at == [T, T, T]


class SsmCase:
    def __init__(self, H, P, N, G, taps, T, n_seqs, seed):
        rng = np.random.default_rng(seed)
        self.H, self.P, self.N, self.G, self.taps = H, P, N, G, taps
        self.inner, self.C = H * P, H * P + 2 * G * N
        self.w, self.b = bf16_round(0.6 * rng.standard_normal((self.C, taps))), bf16_round(0.3 * rng.standard_normal(self.C))
        self.A_log, self.dt_bias, self.D = bf16_round(rng.uniform(-3, 1.5, H)), bf16_round(rng.uniform(-3, 1, H)), bf16_round(rng.standard_normal(H))
        self.A_log[0] = -6.0; self.dt_bias[0] = -3.0          # the first head remembers the first tokens
        if H > 1:
            self.A_log[1] = 3.0; self.dt_bias[1] = 8.0        # the second forgets at once: summed log decays of tens of thousands
        self.raw = [rng.standard_normal((T, self.C + H)).astype(np.float32) for _ in range(n_seqs)]

    def want(self, q):
        xbc = orc.silu(orc.causal_conv(orc.f64(self.raw[q][:, :self.C]), orc.f64(self.w), orc.f64(self.b)))
        dt = orc.softplus(orc.f64(self.raw[q][:, self.C:]) + orc.f64(self.dt_bias))
        y = np.zeros((len(xbc), self.inner))
        for h in range(self.H):
            g = h // (self.H // self.G)
            B, Cc = (xbc[:, o + g * self.N:o + (g + 1) * self.N] for o in (self.inner, self.inner + self.G * self.N))
            y[:, h * self.P:(h + 1) * self.P] = orc.ssm_scan(xbc[:, h * self.P:(h + 1) * self.P], B, Cc, dt[:, h], np.exp(orc.f64(self.A_log[h])), orc.f64(self.D[h]))[0]
        return y


@pytest.mark.parametrize("H,P,N,G,taps", [(4, 24, 48, 2, 4), (6, 8, 12, 3, 3), (2, 64, 128, 1, 4), (3, 5, 7, 3, 2), (1, 1, 1, 1, 1), (2, 70, 200, 2, 5), (4, 64, 64, 1, 4), (2, 40, 256, 1, 4),
                                          (3, 48, 96, 1, 2), (2, 130, 16, 2, 4), (2, 33, 33, 1, 3), (8, 16, 32, 4, 4)])
def test_state_space_in_all_forms_with_continued_states_and_reused_slots(H, P, N, G, taps):
    """the same sequences through: single tokens, chunks and token-by-token steps in turn; three sequences on two slots"""
    T = 205
    c = SsmCase(H, P, N, G, taps, T, 3, H * 1000 + P + N)
    want = [c.want(q) for q in range(3)]
    L = capi()
    ring, st = 4, 4 + ((taps * c.C + 3) // 4) * 4
    w, b, A, db, D = devbf(c.w), devbf(c.b), devbf(c.A_log), devbf(c.dt_bias), devbf(c.D)
    # (sequence, tokens, slot) per step; form "one" needs one token each
    plan = [("scan", [(0, 2, 0)]), ("one", [(0, 1, 0), (1, 1, 1)]), ("chunk", [(0, 65, 0), (1, 130, 1)]), ("one", [(0, 1, 0), (1, 1, 1)]), ("scan", [(0, 3, 0), (1, 2, 1)]),
            ("chunk", [(0, 64, 0), (1, 71, 1)]), ("chunk", [(2, 1, 1), (0, 2, 0)]), ("one", [(2, 1, 1), (0, 1, 0)]), ("chunk", [(2, 200, 1), (0, 63, 0)]),
            ("scan", [(0, 3, 0), (2, 2, 1)]), ("one", [(2, 1, 1)])]
    at = [0, 0, 0]
    slots = Slots(2, st + H * N * P)
    for form, step in plan:
        seqs = [(n, at[q], slot) for q, n, slot in step]
        d, rs, rows = seq_tables(seqs)
        raw = dev32(np.concatenate([c.raw[q][at[q]:at[q] + n] for q, n, _ in step]))
        ld = c.C + H
        dtp = C.c_void_p(raw.data_ptr() + 4 * c.C)
        out = torch.full((rows, c.inner + 1), 7.0, dtype=torch.float32, device="cuda")
        if form == "one":
            ia.check(L.ifa_ssm_step_f32(p(raw), ld, dtp, ld, H, G, N, P, taps, p(w), p(b), p(A), p(db), p(D), p(d), p(rs), rows, p(slots.table), ring, st, p(out), c.inner + 1, None))
        else:
            y = torch.empty((rows, c.C), dtype=torch.float32, device="cuda")
            dt, dec = (torch.empty((rows, H), dtype=torch.float32, device="cuda") for _ in range(2))
            ia.check(L.ifa_conv_ring_silu_f32(p(raw), ld, c.C, taps, p(w), p(b), p(d), p(rs), rows, p(slots.table), ring, p(y), c.C, None))
            ia.check(L.ifa_ssm_gates_ring_f32(dtp, ld, H, rows, p(A), p(db), p(dt), p(dec), p(raw), ld, c.C, taps, p(d), len(step), p(slots.table), ring, None))
            yb, yc = C.c_void_p(y.data_ptr() + 4 * c.inner), C.c_void_p(y.data_ptr() + 4 * (c.inner + G * N))
            if form == "scan":
                ia.check(L.ifa_state_scan_ssm_f32(p(y), c.C, yb, c.C, yc, c.C, H, G, N, P, p(dt), p(dec), p(D), p(d), len(step), p(slots.table), st, p(out), c.inner + 1, None))
            else:
                chunks = sum((n + 63) // 64 for n, _, _ in seqs)
                nb = L.ifa_ssm_chunked_workspace_bytes(chunks, H, G, N, P)
                ws = torch.full((nb // 4,), float("nan"), dtype=torch.float32, device="cuda")
                ia.check(L.ifa_ssm_chunked_f32(p(y), c.C, yb, c.C, yc, c.C, H, G, N, P, p(dt), p(A), p(D), p(d), host_seqs(seqs), len(step), p(slots.table), st, p(ws), nb, p(out),
                                               c.inner + 1, None))
        sync()
        got, r0 = out.cpu().numpy(), 0
        assert np.all(got[:, c.inner:] == 7.0)
        for q, n, _ in step:
            ref = want[q][at[q]:at[q] + n]
            for h in range(H):          # (head by head: their sizes differ by orders of magnitude)
                a, bb = got[r0:r0 + n, h * P:(h + 1) * P], ref[:, h * P:(h + 1) * P]
                assert np.abs(a - bb).max() < 2e-5 * max(0.5, np.abs(want[q][:, h * P:(h + 1) * P]).max()), (form, q, at[q], n, h)
            r0 += n; at[q] += n
    assert at == [205, 205, 205]


@pytest.mark.parametrize("rows,channels,groups", [(1, 64, 1), (5, 96, 8), (3, 4096, 8), (7, 30, 5), (2, 14, 14), (1, 12000, 3)])
def test_gate_in_front_of_the_norm_in_parts(rows, channels, groups):
    rng = np.random.default_rng(channels)
    o, z = rng.standard_normal((rows, channels)).astype(np.float32), rng.standard_normal((rows, channels + 3)).astype(np.float32)
    w = bf16_round(1 + 0.3 * rng.standard_normal(channels))
    want = orc.rms_parts(orc.f64(o) * orc.silu(orc.f64(z[:, :channels])), orc.f64(w), groups, 1e-5)
    L = capi()
    od = dev32(o)
    ia.check(L.ifa_gate_groupnorm_f32(p(od), channels, rows, channels, groups, p(devbf(w)), p(dev32(z)), channels + 3, 1e-5, p(od), channels, None)); sync()          # in place
    assert near(od.cpu().numpy(), want, 5e-6)


@pytest.mark.parametrize("H,dn,dr,dv,R", [(2, 16, 8, 24, 32), (4, 56, 24, 40, 96), (1, 5, 6, 7, 9), (2, 128, 64, 128, 224), (9, 8, 4, 8, 144), (1, 1, 2, 1, 1)])
def test_latent_attention_rotated_in_halves_with_a_gate_per_column(H, dn, dr, dv, R):
    """writer, absorbed form and tiled form, in portions, with one far key that stands out"""
    rng = np.random.default_rng(H * 100 + dn + R)
    T, eps, scale, base = 150, 1e-5, 1.2 * (dn + dr) ** -0.5, 300.0
    q, kv = rng.standard_normal((T, H * (dn + dr))).astype(np.float32), rng.standard_normal((T, R + dr)).astype(np.float32)
    g = rng.standard_normal((T, H * dv)).astype(np.float32)
    cw = bf16_round(1 + 0.3 * rng.standard_normal(R))
    uk, uv = bf16_round(rng.standard_normal((H * dn, R)) / np.sqrt(R)), bf16_round(rng.standard_normal((H * dv, R)) / np.sqrt(R))
    c = orc.rms(orc.f64(kv[:, :R]), orc.f64(cw), eps)
    k5 = (c[5] @ orc.f64(uk).T).reshape(H, dn)
    q[T - 1].reshape(H, dn + dr)[:, :dn] = 6.0 * k5 / np.sqrt((k5 * k5).mean())          # the last row looks at key 5
    W = {"q": np.eye(H * (dn + dr)), "dkv.norm": orc.f64(cw), "uk": orc.f64(uk), "uv": orc.f64(uv), "o": np.eye(H * dv)}
    mx = {"heads": H, "dim": dn, "rot_dim": dr, "vdim": dv, "kv_rank": R, "scale": scale, "rot": {"base": base, "dims": dr}}
    # the oracle's mixer over h = [q | kv | g] with selecting matrices
    D = H * (dn + dr) + R + dr + H * dv
    sel = np.eye(D)
    W.update({"q": sel[:H * (dn + dr)], "dkv": sel[H * (dn + dr):H * (dn + dr) + R + dr], "g": sel[H * (dn + dr) + R + dr:]})
    want = orc.latent_attention(np.concatenate([orc.f64(q), orc.f64(kv), orc.f64(g)], 1), W, "", mx, eps)
    fr = torch.from_numpy(base ** (-2.0 * np.arange(dr // 2) / dr)).cuda()
    L = capi()
    CR, QD, OV, ctx = R + dr, H * (dn + dr), H * dv, 160
    ukd, uvd, cwd = devbf(uk), devbf(uv), devbf(cw)
    for tiled in (0, 1):
        slots = Slots(2, ctx * CR)
        at = 0
        for n in (1, 2, 60, 1, 85, 1):
            seqs = [(n, at, 1)]
            d, rs, rows = seq_tables(seqs)
            qd, kd, gd = dev32(q[at:at + n]), dev32(kv[at:at + n]), dev32(g[at:at + n])
            ia.check(L.ifa_latent_prepare_pairs_f32(1, p(kd), CR, R, dr, dr, p(cwd), eps, p(qd), QD, H, dn, p(fr), 1.0, p(d), p(rs), rows, p(slots.table), 0, None))
            out = torch.full((rows, OV), 7.0, dtype=torch.float32, device="cuda")
            if tiled:
                tot = at + n
                kx, vx = torch.zeros((tot, H * dn), dtype=torch.float32, device="cuda"), torch.zeros((tot, OV), dtype=torch.float32, device="cuda")
                lat = C.c_void_p(slots.mem[1].data_ptr())
                ia.check(L.ifa_linear_bf16w(p(ukd), H * dn, R, lat, CR, tot, None, None, 1.0, 0, 1, p(kx), H * dn, 0, 0, None))
                ia.check(L.ifa_linear_bf16w(p(uvd), OV, R, lat, CR, tot, None, None, 1.0, 0, 1, p(vx), OV, 0, 0, None))
                ia.check(L.ifa_attention_latent_tile_gated_f32(1, p(qd), QD, H, dn, dr, dv, R, scale, p(kx), H * dn, p(vx), OV, p(devi([0])), p(gd), OV, p(d), host_seqs(seqs), 1,
                                                               p(slots.table), 0, p(out), OV, None))
            else:
                qa, ol = torch.zeros((rows, H * CR), dtype=torch.float32, device="cuda"), torch.zeros((rows, H * R), dtype=torch.float32, device="cuda")
                ws = torch.zeros(rows * H * 4 * (R + 2), dtype=torch.float32, device="cuda")
                ia.check(L.ifa_latent_absorb_q_f32(p(qd), QD, H, dn, dr, R, p(ukd), rows, p(qa), H * CR, None))
                ia.check(L.ifa_attention_latent_rows_f32(p(qa), H * CR, H, R, dr, scale, p(d), p(rs), rows, p(slots.table), 0, ctx, p(ws), ws.numel() * 4, p(ol), H * R, None))
                ia.check(L.ifa_latent_expand_out_gated_f32(1, p(ol), H * R, R, H, dv, R, p(uvd), p(gd), OV, rows, p(out), OV, None))
            sync()
            assert near(out.cpu().numpy(), want[at:at + n], 3e-5), (tiled, at, n)
            at += n
        assert at == T
