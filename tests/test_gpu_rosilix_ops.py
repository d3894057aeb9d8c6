"""Each mechanism that the Rosilix layers add to the layer-list worker alone, through its C-ABI op, against the float64 functions of
tests/rosilix_oracle.py: rotation in pairs with the cache writer, differential attention in both forms (chunks, windows, grouped queries, portions,
several sequences, reused slots, keys just inside and just outside), learned sinks and shared rows of latent attention in both forms, the squared
relu in a product's epilogue, the norms with plain weights, the scaled embedding."""
import ctypes as C

import numpy as np
import pytest
import torch

import inferflow_amd as ia
from tests import rosilix_oracle as orc
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


def freqs(base, dims):
    return torch.from_numpy(float(base) ** (-2.0 * np.arange(max(dims // 2, 1)) / max(dims, 1))).cuda()


@pytest.mark.parametrize("pairing", [0, 1])
@pytest.mark.parametrize("H,KH,VH,dim,dv,rot", [(8, 4, 2, 24, 10, 24), (6, 2, 1, 64, 128, 32), (3, 3, 3, 7, 5, 6), (2, 2, 1, 150, 33, 150), (4, 2, 2, 300, 8, 2), (2, 1, 1, 9, 4, 0)])
def test_rotation_in_pairs_and_the_cache_writer(pairing, H, KH, VH, dim, dv, rot):
    rng = np.random.default_rng(H + dim)
    base, ctx = 700.0, 60
    seqs = [(3, 0, 1), (1, 40, 0), (5, 17, 2)]
    d, rs, rows = seq_tables(seqs)
    pos = np.concatenate([np.arange(p0, p0 + n) for n, p0, _ in seqs])
    q, k, v = (rng.standard_normal((rows, n + 4)).astype(np.float32) for n in (H * dim, KH * dim, VH * dv))
    slots = Slots(3, 8 + ctx * (KH * dim + VH * dv))
    k_off, v_off = 8, 8 + ctx * KH * dim
    qd = dev32(q)
    ia.check(capi().ifa_qk_rope_store_pairs_f32(pairing, p(qd), H * dim + 4, H, p(dev32(k)), KH * dim + 4, p(dev32(v)), VH * dv + 4, KH, VH, dim, dv, None, None, 1e-5, rot,
                                                p(freqs(base, rot)), p(d), p(rs), rows, p(slots.table), k_off, v_off, None)); sync()

    def turned(z, heads):
        z = orc.f64(z[:, :heads * dim]).reshape(rows, heads, dim)
        if pairing == 0 and rot:          # halves: the pairs of an interleaved copy
            at = np.r_[np.arange(rot).reshape(2, -1).T.reshape(-1), rot:dim]
            back = np.argsort(at)
            return orc.turn_pairs(z[..., at], pos, rot, base)[..., back].reshape(rows, -1)
        return orc.turn_pairs(z, pos, rot, base).reshape(rows, -1)
    assert near(qd.cpu().numpy()[:, :H * dim], turned(q, H)) and np.array_equal(qd.cpu().numpy()[:, H * dim:], q[:, H * dim:])
    kt, r = turned(k, KH), 0
    for n, p0, slot in seqs:
        mem = slots.mem[slot].cpu().numpy()
        K, V = mem[k_off:v_off].reshape(ctx, -1), mem[v_off:].reshape(ctx, -1)
        assert near(K[p0:p0 + n], kt[r:r + n]) and np.array_equal(V[p0:p0 + n], v[r:r + n, :VH * dv])
        untouched = np.r_[0:p0, p0 + n:ctx]
        assert np.all(K[untouched] == 1e9) and np.all(V[untouched] == 1e9)
        r += n


class DiffCase:
    """three sequences of projected, already turned rows; the last head size decides which form serves it"""

    def __init__(self, H, G, d, dv, chunk, window, T, seed):
        rng = np.random.default_rng(seed)
        self.__dict__.update(H=H, G=G, d=d, dv=dv, chunk=chunk, window=window, T=T)
        self.q = [rng.standard_normal((T, H, 2, d)).astype(np.float32) for _ in range(3)]
        self.k = [rng.standard_normal((T, G, 2, d)).astype(np.float32) for _ in range(3)]
        self.v = [rng.standard_normal((T, G, dv)).astype(np.float32) for _ in range(3)]
        self.g = [rng.standard_normal((T, H)).astype(np.float32) for _ in range(3)]
        self.scale, self.lam, self.diff, self.eps = 1.3 * d ** -0.5, 0.71, 0.35, 1e-5
        # rows whose query stands out towards the oldest key they see, and towards the newest one they do not
        for s in range(3):
            for i in range(3, T, 5):
                lo = 0
                if chunk:
                    lo = i - i % chunk
                if window:
                    lo = max(lo, i - window + 1)
                j = lo if i % 2 else max(lo - 1, 0)
                for h in range(H):
                    kk = self.k[s][j, h // (H // G), i % 2 if d > 1 else 0]
                    self.q[s][i, h, i % 2 if d > 1 else 0] = 5.0 * kk / np.sqrt((kk * kk).mean()) / np.sqrt(d) / self.scale * 1.3

    def want(self, s):
        return orc.two_map_attention(orc.f64(self.q[s]), orc.f64(self.k[s]), orc.f64(self.v[s]), orc.visible(self.T, self.chunk, self.window), self.scale, self.lam, self.diff,
                                     orc.logistic(orc.f64(self.g[s])), self.eps).reshape(self.T, -1)


DIFF_SHAPES = [(4, 2, 24, 40, 37, 0), (6, 1, 64, 96, 64, 0), (2, 2, 128, 128, 100, 0), (8, 2, 32, 64, 0, 0), (3, 3, 7, 9, 33, 0), (1, 1, 1, 1, 10, 0), (4, 1, 64, 128, 0, 50),
               (5, 1, 48, 200, 65, 0), (2, 1, 40, 33, 32, 20), (2, 1, 160, 48, 70, 0), (4, 2, 20, 300, 90, 0), (3, 1, 12, 16, 1, 0), (6, 2, 96, 72, 128, 129), (2, 1, 100, 64, 31, 0),
               (2, 2, 36, 224, 96, 0), (12, 2, 16, 160, 48, 0), (16, 2, 64, 256, 150, 0), (1, 1, 130, 1024, 40, 0), (8, 1, 1024, 256, 60, 0)]


@pytest.mark.parametrize("H,G,d,dv,chunk,window", DIFF_SHAPES)
def test_differential_attention_in_both_forms(H, G, d, dv, chunk, window):
    """three sequences on two slots filled with garbage, in portions of 1 to 130 rows, each portion through the row form and the tiled form"""
    T = 205
    c = DiffCase(H, G, d, dv, chunk, window, T, H * 100 + d + dv)
    want = [c.want(s) for s in range(3)]
    L = capi()
    ctx, kw, vw = T + 3, G * 2 * d, G * dv
    k_off, v_off = 4, 4 + ((ctx * kw + 3) // 4) * 4
    plan = [[(0, 1, 0)], [(0, 2, 0), (1, 31, 1)], [(0, 130, 0), (1, 1, 1)], [(0, 1, 0), (1, 1, 1)], [(1, 64, 1), (0, 40, 0)], [(1, 108, 1), (0, 31, 0)], [(2, 33, 1)], [(2, 171, 1)], [(2, 1, 1)]]
    for tile_min in (1, 1 << 30, 16):
        slots = Slots(2, v_off + ctx * vw)
        at = [0, 0, 0]
        for step in plan:
            seqs = [(n, at[s], slot) for s, n, slot in step]
            d_, rs, rows = seq_tables(seqs)
            for s, n, slot in step:          # (what the cache writer leaves)
                mem = slots.mem[slot]
                mem[k_off + at[s] * kw:k_off + (at[s] + n) * kw] = dev32(c.k[s][at[s]:at[s] + n]).reshape(-1)
                mem[v_off + at[s] * vw:v_off + (at[s] + n) * vw] = dev32(c.v[s][at[s]:at[s] + n]).reshape(-1)
            q = dev32(np.concatenate([c.q[s][at[s]:at[s] + n].reshape(n, -1) for s, n, _ in step]))
            g = dev32(np.concatenate([c.g[s][at[s]:at[s] + n] for s, n, _ in step]))
            ws = torch.full((rows * H * 6 * 2 * (dv + 2),), float("nan"), dtype=torch.float32, device="cuda")
            ldo = H * dv + (4 if rows % 2 else 3)
            out = torch.full((rows, ldo), 7.0, dtype=torch.float32, device="cuda")
            ia.check(L.ifa_attention_diff_f32(p(q), H * 2 * d, H, G, d, dv, c.scale, window, chunk, c.lam, 1.0 - c.diff, c.eps, p(g), H, p(d_), p(rs), rows, p(slots.table), k_off,
                                              v_off, p(out), None, ldo, host_seqs(seqs), len(seqs), tile_min, ctx, p(ws), ws.numel() * 4, None)); sync()
            got, r = out.cpu().numpy(), 0
            assert np.all(got[:, H * dv:] == 7.0)
            if tile_min == 1 and L.ifa_attention_diff_tile_fits(d, dv):          # the same in bfloat16
                half = torch.zeros((rows, ldo), dtype=torch.int16, device="cuda")
                ia.check(L.ifa_attention_diff_f32(p(q), H * 2 * d, H, G, d, dv, c.scale, window, chunk, c.lam, 1.0 - c.diff, c.eps, p(g), H, p(d_), p(rs), rows, p(slots.table), k_off,
                                                  v_off, None, p(half), ldo, host_seqs(seqs), len(seqs), tile_min, ctx, p(ws), ws.numel() * 4, None)); sync()
                assert np.array_equal((half.cpu().numpy().view(np.uint16).astype(np.uint32) << 16).view(np.float32)[:, :H * dv], bf16_round(got[:, :H * dv]))
            for s, n, _ in step:
                # (a head whose two maps nearly cancel is small before its norm: rounding relative to the norm's gain)
                assert near(got[r:r + n, :H * dv], want[s][at[s]:at[s] + n], 1e-4), (tile_min, s, at[s], n)
                assert np.median(np.abs(got[r:r + n, :H * dv] - want[s][at[s]:at[s] + n])) < 2e-6, (tile_min, s, at[s], n)
                r += n; at[s] += n
        assert at == [T, T, T]


def test_differential_attention_without_a_gate_and_decode_shares():
    """single rows over 1500 keys: every number of key shares, no gate; a step of forty single rows stays with the row form"""
    rng = np.random.default_rng(3)
    H, G, d, dv, T = 4, 2, 32, 48, 1500
    c = DiffCase(H, G, d, dv, 0, 0, T, 5)
    see = orc.visible(T)
    L = capi()
    kw, vw = G * 2 * d, G * dv
    n_slots = 40
    slots = Slots(n_slots, T * (kw + vw))
    for sl in range(n_slots):
        slots.mem[sl][:T * kw] = dev32(c.k[sl % 3]).reshape(-1)
        slots.mem[sl][T * kw:] = dev32(c.v[sl % 3]).reshape(-1)
    ends = [0, 15, 16, 63, 64, 65, 700, 1499] + [int(x) for x in rng.integers(0, T, 32)]
    want = []
    for sl, i in enumerate(ends):
        s = sl % 3
        o = orc.two_map_attention(orc.f64(c.q[s][:i + 1]), orc.f64(c.k[s][:i + 1]), orc.f64(c.v[s][:i + 1]), see[:i + 1, :i + 1], c.scale, c.lam, 0.0, np.ones((i + 1, H)), c.eps) \
            if i < 70 else None
        if o is None:          # only the last row
            o = np.zeros((1, H, dv))
            for h in range(H):
                maps = [orc.softmax((orc.f64(c.q[s][i, h, m]) @ orc.f64(c.k[s][:i + 1, h // 2, m]).T)[None] * c.scale) @ orc.f64(c.v[s][:i + 1, h // 2]) for m in range(2)]
                o[0, h] = orc.difference(maps[0], maps[1], c.lam, 0.0, c.eps)[0]
        want.append(o[-1].reshape(-1))
    for shares in (1, 2, 7, 24, 64):
        for batch in ([[i] for i in range(8)] + [list(range(n_slots))]):
            seqs = [(1, ends[i], i) for i in batch]
            d_, rs, rows = seq_tables(seqs)
            q = dev32(np.stack([c.q[i % 3][ends[i]].reshape(-1) for i in batch]))
            ws = torch.full((rows * H * shares * 2 * (dv + 2),), float("nan"), dtype=torch.float32, device="cuda")
            out = torch.zeros((rows, H * dv), dtype=torch.float32, device="cuda")
            ia.check(L.ifa_attention_diff_f32(p(q), H * 2 * d, H, G, d, dv, c.scale, 0, 0, c.lam, 1.0, c.eps, None, 0, p(d_), p(rs), rows, p(slots.table), 0, T * kw, p(out), None, H * dv,
                                              host_seqs(seqs), rows, 16, 64 * shares, p(ws), ws.numel() * 4, None)); sync()
            assert near(out.cpu().numpy(), np.stack([want[i] for i in batch]), 3e-5), (shares, len(batch))


def test_differential_attention_declines_bad_arguments():
    L = capi()
    z = torch.zeros(4096, dtype=torch.float32, device="cuda")
    slots = Slots(1, 4096)
    d_, rs, rows = seq_tables([(1, 0, 0)])

    def rc(H=2, G=1, d=8, dv=8, ws_bytes=4096, ldq=32):
        return L.ifa_attention_diff_f32(p(z), ldq, H, G, d, dv, 1.0, 0, 0, 0.5, 0.5, 1e-5, None, 0, p(d_), p(rs), 1, p(slots.table), 0, 1024, p(z), None, H * dv, host_seqs([(1, 0, 0)]), 1, 16, 4,
                                        p(z), ws_bytes, None)
    assert rc() == 0
    for bad in (dict(H=3, G=2), dict(d=0), dict(d=1025, ldq=9000), dict(dv=0), dict(ws_bytes=16), dict(ldq=31)):
        assert rc(**bad) != 0, bad
    sync()


@pytest.mark.parametrize("H,dn,dr,dv,R", [(2, 16, 8, 24, 32), (4, 56, 24, 40, 96), (1, 5, 6, 7, 9), (2, 128, 64, 128, 224), (9, 8, 4, 8, 144), (1, 1, 2, 1, 1), (3, 130, 70, 136, 40)])
def test_latent_attention_with_sinks_over_own_and_shared_rows(H, dn, dr, dv, R):
    """one layer writes the rows, a second one (queries only) reads them; absorbed and tiled form; sinks far below, near and far above the scores; a far key
    that stands out"""
    rng = np.random.default_rng(H * 100 + dn + R)
    T, eps, scale, base = 150, 1e-5, 1.2 * (dn + dr) ** -0.5, 300.0
    q, kv = rng.standard_normal((T, H * (dn + dr))).astype(np.float32), rng.standard_normal((T, R + dr)).astype(np.float32)
    g = rng.standard_normal((T, H)).astype(np.float32)
    cw, sink = bf16_round(1 + 0.3 * rng.standard_normal(R)), bf16_round(np.array([3.0, -40.0, 60.0, 0.0] * 3)[:H])
    uk, uv = bf16_round(rng.standard_normal((H * dn, R)) / np.sqrt(R)), bf16_round(rng.standard_normal((H * dv, R)) / np.sqrt(R))
    c5 = orc.norm(orc.f64(kv[5:6, :R]), orc.f64(cw), eps)
    k5 = (c5 @ orc.f64(uk).T).reshape(H, dn)
    q[T - 1].reshape(H, dn + dr)[:, :dn] = 6.0 * k5 / np.sqrt((k5 * k5).mean())          # the last row looks at key 5
    # the oracle's mixer over h = [q | kv | g] with selecting matrices
    QD, CR, OV = H * (dn + dr), R + dr, H * dv
    sel = np.eye(QD + CR + H)
    W = {"q": sel[:QD], "dkv": sel[QD:QD + CR], "g": sel[QD + CR:], "dkv.norm": orc.f64(cw), "uk": orc.f64(uk), "uv": orc.f64(uv), "o": np.eye(OV), "sink": orc.f64(sink)}
    mx = {"heads": H, "dim": dn, "rot_dim": dr, "vdim": dv, "kv_rank": R, "scale": scale, "rot": {"base": base, "dims": dr}}
    h = np.concatenate([orc.f64(q), orc.f64(kv), orc.f64(g)], 1)
    rows_w = orc.latent_rows(h, W, "", mx, eps)
    want = orc.latent_attention(h, rows_w, W, "", mx)
    fr = freqs(base, dr)
    L = capi()
    ctx = 160
    ukd, uvd, cwd, sd = devbf(uk), devbf(uv), devbf(cw), devbf(sink)
    fits = L.ifa_attention_latent_tile_fits(dn, dr, dv)
    for tiled in ((0, 1) if fits else (0,)):
        slots = Slots(2, ctx * CR)
        at = 0
        for n in (1, 2, 60, 1, 85, 1):
            seqs = [(n, at, 1)]
            d, rs, rows = seq_tables(seqs)
            kd, gd = dev32(kv[at:at + n]), dev32(g[at:at + n])
            for own in (1, 0):          # (own: writes the rows; not own: turns its queries and finds the rows there)
                qd = dev32(q[at:at + n])
                if own:
                    ia.check(L.ifa_latent_prepare_pairs_f32(0, p(kd), CR, R, dr, dr, p(cwd), eps, p(qd), QD, H, dn, p(fr), 1.0, p(d), p(rs), rows, p(slots.table), 0, None))
                    written = slots.mem[1].clone()
                else:
                    ia.check(L.ifa_latent_rotate_q_f32(0, dr, dr, p(qd), QD, H, dn, p(fr), 1.0, p(d), p(rs), rows, None))
                    sync()
                    assert torch.equal(slots.mem[1], written)
                out = torch.full((rows, OV), 7.0, dtype=torch.float32, device="cuda")
                if tiled:
                    tot = at + n
                    kx, vx = torch.zeros((tot, H * dn), dtype=torch.float32, device="cuda"), torch.zeros((tot, OV), dtype=torch.float32, device="cuda")
                    lat = C.c_void_p(slots.mem[1].data_ptr())
                    ia.check(L.ifa_linear_bf16w(p(ukd), H * dn, R, lat, CR, tot, None, None, 1.0, 0, 1, p(kx), H * dn, 0, 0, None))
                    ia.check(L.ifa_linear_bf16w(p(uvd), OV, R, lat, CR, tot, None, None, 1.0, 0, 1, p(vx), OV, 0, 0, None))
                    ia.check(L.ifa_attention_latent_tile_sinks_f32(0, p(qd), QD, H, dn, dr, dv, R, scale, p(sd), p(kx), H * dn, p(vx), OV, p(devi([0])), p(gd), H, p(d), host_seqs(seqs), 1,
                                                                   p(slots.table), 0, p(out), None, OV, None))
                else:
                    qa, ol = torch.zeros((rows, H * CR), dtype=torch.float32, device="cuda"), torch.zeros((rows, H * R), dtype=torch.float32, device="cuda")
                    ws = torch.zeros(rows * H * 4 * (R + 2), dtype=torch.float32, device="cuda")
                    ia.check(L.ifa_latent_absorb_q_f32(p(qd), QD, H, dn, dr, R, p(ukd), rows, p(qa), H * CR, None))
                    ia.check(L.ifa_attention_latent_rows_sinks_f32(p(qa), H * CR, H, R, dr, scale, p(sd), p(d), p(rs), rows, p(slots.table), 0, ctx, p(ws), ws.numel() * 4, p(ol), H * R, None))
                    ia.check(L.ifa_latent_expand_out_gated_f32(0, p(ol), H * R, R, H, dv, R, p(uvd), p(gd), H, rows, p(out), OV, None))
                sync()
                assert near(out.cpu().numpy(), want[at:at + n], 3e-5), (tiled, own, at, n)
                if tiled:          # the same in bfloat16
                    half = torch.zeros((rows, OV), dtype=torch.int16, device="cuda")
                    ia.check(L.ifa_attention_latent_tile_sinks_f32(0, p(qd), QD, H, dn, dr, dv, R, scale, p(sd), p(kx), H * dn, p(vx), OV, p(devi([0])), p(gd), H, p(d), host_seqs(seqs), 1,
                                                                   p(slots.table), 0, None, p(half), OV, None)); sync()
                    assert np.array_equal((half.cpu().numpy().view(np.uint16).astype(np.uint32) << 16).view(np.float32), bf16_round(out.cpu().numpy()))
            at += n
        assert at == T


@pytest.mark.parametrize("T", [1, 2, 8, 9, 64, 131])
@pytest.mark.parametrize("N,K", [(64, 64), (5, 36), (130, 200), (48, 7)])
def test_squared_relu_in_the_epilogue(T, N, K):
    rng = np.random.default_rng(T + N + K)
    Wm, A, b = bf16_round(rng.standard_normal((N, K))), rng.standard_normal((T, K + 4)).astype(np.float32), bf16_round(rng.standard_normal(N))
    for ops32 in (1, 0):
        a = A if ops32 or T <= 8 else bf16_round(A)
        for bias in (None, b):
            want = np.maximum(orc.f64(a[:, :K]) @ orc.f64(Wm).T + (0 if bias is None else orc.f64(b)), 0) ** 2
            out = torch.full((T, N + 2), 7.0, dtype=torch.float32, device="cuda")
            ia.check(capi().ifa_linear_bf16w_act(p(devbf(Wm)), N, K, p(dev32(A)), K + 4, T, p(devbf(b)) if bias is not None else None, 2, ops32, p(out), N + 2, None)); sync()
            assert near(out.cpu().numpy()[:, :N], want, 1e-5) and np.all(out.cpu().numpy()[:, N:] == 7.0)
    assert capi().ifa_linear_bf16w_act(p(devbf(Wm)), N, K, p(dev32(A)), K + 4, T, None, 3, 1, p(out), N + 2, None) != 0


@pytest.mark.parametrize("T,N,K", [(1, 1, 64), (17, 64, 64), (200, 70, 80), (65, 130, 136), (1100, 1930, 200), (1025, 2049, 72), (2500, 2600, 72), (2561, 2432, 328), (300, 520, 2048)])
def test_products_of_prompts_in_every_tile(T, N, K):
    """row and column counts on both sides of the tiles' borders, inner sizes that are no multiple of a step; every epilogue; the same numbers as the product that
    rounds its activations itself"""
    rng = np.random.default_rng(T + N + K)
    Wm, A, b = bf16_round(rng.standard_normal((N, K))), rng.standard_normal((T, K + 4)).astype(np.float32), bf16_round(rng.standard_normal(N))
    mul, C0 = bf16_round(rng.standard_normal(N)), rng.standard_normal((T, N + 2)).astype(np.float32)
    prod = orc.f64(bf16_round(A)[:, :K]) @ orc.f64(Wm).T
    wd, ad, bd, md, L = devbf(Wm), dev32(A), devbf(b), devbf(mul), capi()
    ld = (K + 63) // 64 * 64
    a16 = torch.full((T, ld), -1, dtype=torch.int16, device="cuda")
    ia.check(L.ifa_rows_to_bf16(p(ad), K + 4, T, K, p(a16), ld, None)); sync()
    bits = a16.cpu().numpy().view(np.uint16)
    assert np.array_equal((bits.astype(np.uint32) << 16).view(np.float32)[:, :K], bf16_round(A)[:, :K]) and np.all(bits[:, K:] == 0)
    # bias, SiLU on a column range, scale per column, accumulation
    c = dev32(C0)
    ia.check(L.ifa_linear_bf16_both(p(wd), N, K, p(a16), ld, T, p(bd), p(md), 0.7, 1, 0, p(c), None, N + 2, 3, min(N, 41), None)); sync()
    want = prod + orc.f64(b)
    want[:, 3:min(N, 41)] *= orc.logistic(want[:, 3:min(N, 41)])
    assert near(c.cpu().numpy()[:, :N], C0[:, :N] + want * orc.f64(mul) * 0.7, 1e-5) and np.array_equal(c.cpu().numpy()[:, N:], C0[:, N:])
    # plain, against the other product too (from 9 rows on it rounds its activations)
    out, other = (torch.full((T, N), 7.0, dtype=torch.float32, device="cuda") for _ in range(2))
    ia.check(L.ifa_linear_bf16_both(p(wd), N, K, p(a16), ld, T, None, None, 1.0, 0, 0, p(out), None, N, 0, 0, None))
    ia.check(L.ifa_linear_bf16w(p(wd), N, K, p(ad), K + 4, T, None, None, 1.0, 0, 0, p(other), N, 0, 0, None)); sync()
    assert near(out.cpu().numpy(), prod, 1e-5) and (T <= 8 or torch.equal(out, other))
    # residual update; the squared relu in both output formats; erf-GELU
    ia.check(L.ifa_linear_bf16_both(p(wd), N, K, p(a16), ld, T, p(bd), None, 1.0, 1, 0, p(out), None, N, 0, 0, None)); sync()
    assert near(out.cpu().numpy(), 2 * prod + orc.f64(b), 1e-5)
    h = torch.zeros((T, N), dtype=torch.int16, device="cuda")
    ia.check(L.ifa_linear_bf16_both(p(wd), N, K, p(a16), ld, T, None, None, 1.0, 0, 2, p(out), None, N, 0, 0, None))
    ia.check(L.ifa_linear_bf16_both(p(wd), N, K, p(a16), ld, T, None, None, 1.0, 0, 2, None, p(h), N, 0, 0, None)); sync()
    assert near(out.cpu().numpy(), np.maximum(prod, 0) ** 2, 1e-5)
    assert np.array_equal((h.cpu().numpy().view(np.uint16).astype(np.uint32) << 16).view(np.float32), bf16_round(out.cpu().numpy()))
    ia.check(L.ifa_linear_bf16_both(p(wd), N, K, p(a16), ld, T, p(bd), None, 1.0, 0, 1, p(out), None, N, 0, 0, None)); sync()
    z = torch.from_numpy(prod + orc.f64(b))
    assert near(out.cpu().numpy(), torch.nn.functional.gelu(z).numpy(), 1e-5)


def test_products_of_prompts_decline_bad_arguments():
    L = capi()
    z = torch.zeros(1 << 16, dtype=torch.float32, device="cuda")

    def rc(N=8, K=64, ld=64, T=4, acc=0, act=0, c=True, h=False, ldc=8):
        return L.ifa_linear_bf16_both(p(z), N, K, p(z), ld, T, None, None, 1.0, acc, act, p(z) if c else None, p(z) if h else None, ldc, 0, 0, None)
    assert rc() == 0
    for bad in (dict(K=56), dict(K=68), dict(ld=72), dict(ld=128), dict(T=0), dict(act=3), dict(c=False), dict(h=True), dict(h=True, act=2, acc=1), dict(ldc=7)):
        assert rc(**bad) != 0, bad
    sync()


@pytest.mark.parametrize("rows,cols", [(1, 64), (5, 97), (3, 4096), (2, 4100), (3, 8192), (2, 9000), (9, 12)])
def test_norms_on_both_sides_with_plain_weights(rows, cols):
    rng = np.random.default_rng(cols)
    x, m = (rng.standard_normal((rows, cols)).astype(np.float32) for _ in range(2))
    wa, wb = (bf16_round(1 + 0.3 * rng.standard_normal(cols)) for _ in range(2))
    eps = 1e-4
    new = orc.f64(x) + orc.norm(orc.f64(m), orc.f64(wa), eps)
    L = capi()
    xd, h = dev32(x), torch.zeros((rows, cols), dtype=torch.float32, device="cuda")
    ia.check(L.ifa_norm_add_norm_f32(p(xd), cols, rows, cols, p(dev32(m)), cols, p(devbf(wa)), p(devbf(wb)), 0.0, eps, p(h), cols, None)); sync()
    assert near(xd.cpu().numpy(), new) and near(h.cpu().numpy(), orc.norm(new, orc.f64(wb), eps), 5e-6)
    ia.check(L.ifa_rmsnorm_offset_f32(p(xd), cols, rows, cols, p(devbf(wb)), 0.0, eps, 0, p(h), cols, None)); sync()
    assert near(h.cpu().numpy(), orc.norm(new, orc.f64(wb), eps), 5e-6)
    # h in bfloat16, with and without the update in front
    half = torch.zeros((rows, cols), dtype=torch.int16, device="cuda")
    for upd in (0, 1):
        xd = dev32(new if not upd else x)
        rc = L.ifa_norm_add_norm_to_bf16(p(xd), cols, rows, cols, p(dev32(m)) if upd else None, cols, p(devbf(wa)) if upd else None, p(devbf(wb)), 0.0, eps, p(half), cols, None); sync()
        if cols % 4 or cols > 8192:
            assert rc != 0
            continue
        ia.check(rc)
        got = (half.cpu().numpy().view(np.uint16).astype(np.uint32) << 16).view(np.float32)
        assert near(xd.cpu().numpy(), new) and np.abs(got - orc.norm(new, orc.f64(wb), eps)).max() < 2 ** -7 * max(1.0, np.abs(got).max())


def test_scaled_embedding():
    rng = np.random.default_rng(9)
    V, W = 31, 50
    E, toks = bf16_round(rng.standard_normal((V, W))), [3, 30, 0, 3, 17]
    d, rs, rows = seq_tables([(2, 4, 1), (3, 0, 0)])
    slots = Slots(2, 8)
    x = torch.zeros((rows, W), dtype=torch.float32, device="cuda")
    ia.check(capi().ifa_embed_pair_scaled_f32(p(devbf(E)), V, W, 11.25, None, 0, 0, 0, p(devi(toks)), p(d), p(rs), rows, p(slots.table), 0, p(x), None, None)); sync()
    assert near(x.cpu().numpy(), orc.f64(E)[toks] * 11.25)
