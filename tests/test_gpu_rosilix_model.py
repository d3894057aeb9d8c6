"""The layer-list worker serving Rosilix models through the InferenceEngine (registry, slots, scheduler, sampling entry points) against the float64
oracle of tests/rosilix_oracle.py: whole prompts, the residual after every layer, token-by-token decoding, portions down to two tokens, mixed batches
with slots reused, marked keys just inside and just outside every chunk and far back under latent attention (own and shared rows), the first tokens of a
sequence, long decoding, other sizes, greedy generation, the trace tool."""
import json
import os
import subprocess

import numpy as np
import pytest

from tests import rosilix_fixtures as fx
from tests import rosilix_oracle as orc
from tests.gelarax_oracle import bf16_round

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL32 = 3e-5        # fp32 operands: rounding of fp32 sums only
TOL16 = 6e-2        # operands of the matrix products rounded to bfloat16


def engine_for(tmp_path, cfg, weights, dtype="float32", ctx=512, queries=6):
    from inferflow_amd.engine import InferenceEngine
    d = fx.write_model_dir(str(tmp_path / ("m%d" % len(os.listdir(tmp_path)))), cfg, weights)
    return InferenceEngine.from_model_dir(d, dtype, ctx, queries, True)


def tokens_for(cfg, n, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def oracle_logits(cfg, weights, tokens, taps=None):
    return orc.forward(cfg, fx.oracle_weights(weights), tokens, taps)


def run_whole(eng, tokens):
    q = eng.add_query(tokens)
    assert q > 0
    out = eng.infer()
    assert [i for i, _ in out] == [q]
    lg = eng.last_logits_f32(q)
    eng.remove_query(q)
    return lg, out[0][1]


def run_portions(eng, tokens, sizes):
    """the prompt in portions of the given sizes (the last size repeats); logits of every token"""
    q = eng.add_query(tokens[:sizes[0]])
    rows, at, k = [], sizes[0], 0
    eng.infer(); rows.append(eng.last_logits_f32(q))
    while at < len(tokens):
        k = min(k + 1, len(sizes) - 1)
        n = min(sizes[k], len(tokens) - at)
        for t in tokens[at:at + n]:
            assert eng.commit({q: t})
        eng.infer(); rows.append(eng.last_logits_f32(q))
        at += n
    eng.remove_query(q)
    return np.concatenate(rows, 0)


# both mixers, with and without a feed-forward; two groups of shared latent rows whose readers have heads of other sizes than the source, one of them
# behind a layer of the other kind; chunks of two sizes; three, two and one query heads per key / value head
MIXED = fx.config([fx.latent_layer(heads=3, dim=20, rot_dim=8, vdim=12, kv_rank=28),
                   fx.attention_layer(heads=4, kv_heads=2, dim=12, vdim=20, chunk=37, rot_dims=8),
                   fx.latent_layer(heads=2, dim=12, rot_dim=8, vdim=24, kv_rank=28, kv_from=0, mlp=None),
                   fx.attention_layer(heads=3, kv_heads=1, dim=16, vdim=8, chunk=50, rot_dims=16, base=70.0, diff=0.6, mlp=None),
                   fx.latent_layer(heads=4, dim=16, rot_dim=4, vdim=16, kv_rank=36, base=500.0, mlp=fx.dense(33)),
                   fx.latent_layer(heads=5, dim=8, rot_dim=4, vdim=8, kv_rank=36, base=500.0, kv_from=4),
                   fx.attention_layer(heads=2, kv_heads=2, dim=24, vdim=32, chunk=64, rot_dims=24, diff=0.1, mlp=fx.dense(100))], width=72, vocab=89)


@pytest.mark.parametrize("dtype,tol", [("float32", TOL32), ("bfloat16", TOL16)])
def test_whole_prompt_matches_the_oracle(tmp_path, dtype, tol):
    w = fx.random_weights(MIXED, 1)
    toks = tokens_for(MIXED, 141, 2)
    eng = engine_for(tmp_path, MIXED, w, dtype)
    lg, nxt = run_whole(eng, toks)
    want = oracle_logits(MIXED, w, toks)
    assert lg.shape == want.shape
    err = fx.rel_err(lg, want)
    assert err.max() < tol and np.median(err) < 0.5 * tol, (err.max(), np.median(err))
    if dtype == "float32":
        assert nxt == int(want[-1].argmax())
    assert fx.rel_err(run_portions(eng, toks, [40, 9, 1]), want).max() < tol
    eng.close()


def test_residual_after_every_layer_matches_the_oracle(tmp_path):
    import ctypes as C
    import inferflow_amd as ia
    w = fx.random_weights(MIXED, 3)
    eng = engine_for(tmp_path, MIXED, w)
    L = ia.lib()
    ia.check(L.ifa_model_set_option(eng.worker(), b"tap_layers", 1))
    for n in (130, 40, 5, 1):
        toks = tokens_for(MIXED, n, 4)
        run_whole(eng, toks)
        res = []
        oracle_logits(MIXED, w, toks, res)
        for li, want in enumerate(res):
            p, b = C.c_void_p(), C.c_size_t()
            ia.check(L.ifa_model_get_buffer(eng.worker(), b"layer_taps", li, C.byref(p), C.byref(b)))
            got = np.zeros((len(toks), MIXED["width"]), np.float32)
            ia.check(L.ifa_memcpy_d2h(got.ctypes.data_as(C.c_void_p), p, got.nbytes, None)); ia.check(L.ifa_stream_sync(None))
            assert np.abs(got - want).max() < 1e-4 * max(1.0, np.abs(want).max()), (n, li)
    eng.close()


@pytest.mark.parametrize("sizes", [[1], [2], [5, 3], [30, 1], [7, 2, 1], [36, 1, 2], [37, 13], [17, 16, 2], [50, 33], [64, 4], [2, 65, 1], [63, 1, 64]])
def test_portions_and_token_by_token_equal_the_whole_prompt(tmp_path, sizes):
    w = fx.random_weights(MIXED, 5)
    toks = tokens_for(MIXED, 133, 6)
    eng = engine_for(tmp_path, MIXED, w)
    whole, _ = run_whole(eng, toks)
    parts = run_portions(eng, toks, sizes)
    assert parts.shape == whole.shape
    assert fx.rel_err(parts, whole).max() < TOL32
    assert fx.rel_err(parts, oracle_logits(MIXED, w, toks)).max() < TOL32
    eng.close()


def test_folded_launches_and_separate_ops_agree(tmp_path):
    """the norms between two sub-layers in one launch against launches of their own"""
    import inferflow_amd as ia
    w = fx.random_weights(MIXED, 25)
    toks = tokens_for(MIXED, 60, 26)
    want = oracle_logits(MIXED, w, toks)
    eng = engine_for(tmp_path, MIXED, w)
    for fuse in (1, 0, 1):
        ia.check(ia.lib().ifa_model_set_option(eng.worker(), b"fuse_post", fuse))
        for sizes in ([33, 1], [3, 2], [8, 7, 1]):
            assert fx.rel_err(run_portions(eng, toks, sizes), want).max() < TOL32, (fuse, sizes)
    eng.close()


@pytest.mark.parametrize("n", [1, 2, 3])
def test_first_tokens_of_a_sequence(tmp_path, n):
    """the shortest prompts, whole and token by token, on a slot that held a longer sequence before"""
    w = fx.random_weights(MIXED, 21)
    eng = engine_for(tmp_path, MIXED, w, queries=1)
    run_whole(eng, tokens_for(MIXED, 150, 22))
    toks = tokens_for(MIXED, n, 23 + n)
    want = oracle_logits(MIXED, w, toks)
    assert fx.rel_err(run_whole(eng, toks)[0], want).max() < TOL32
    assert fx.rel_err(run_portions(eng, toks, [1]), want).max() < TOL32
    eng.close()


def test_batches_of_unequal_requests_equal_each_alone_and_slots_are_reused(tmp_path):
    w = fx.random_weights(MIXED, 7)
    eng = engine_for(tmp_path, MIXED, w, queries=3)
    prompts = [tokens_for(MIXED, n, 10 + n) for n in (1, 37, 64, 5, 110, 2)]
    tails = [tokens_for(MIXED, 12, 50 + i) for i in range(len(prompts))]
    alone = [oracle_logits(MIXED, w, p + t) for p, t in zip(prompts, tails)]
    # three queries on three slots, twice: the second time reuses the slots of the first
    for rnd in range(2):
        qs = [eng.add_query(p) for p in prompts[3 * rnd:3 * rnd + 3]]
        assert all(q > 0 for q in qs) and eng.add_query([1, 2]) == 0          # busy: every slot is taken
        got = {q: [] for q in qs}
        assert sorted(i for i, _ in eng.infer()) == sorted(qs)                 # ONE step for the three prompts
        for q in qs:
            got[q].append(eng.last_logits_f32(q))
        for step in range(12):
            live = [q for k, q in enumerate(qs) if not (k == 0 and step >= 6)]  # the first query ends earlier
            if step == 6:
                eng.remove_query(qs[0])
            eng.commit({q: tails[3 * rnd + qs.index(q)][step] for q in live})
            assert sorted(i for i, _ in eng.infer()) == sorted(live)
            for q in live:
                got[q].append(eng.last_logits_f32(q))
        for k, q in enumerate(qs):
            g = np.concatenate(got[q], 0)
            assert fx.rel_err(g, alone[3 * rnd + k][:len(g)]).max() < TOL32, (rnd, k)
            if not (k == 0):
                eng.remove_query(q)
    eng.close()


def test_twenty_requests_start_together_and_are_decoded_together(tmp_path):
    """a step of twenty prompts of unequal lengths, then steps of twenty, later twelve, single tokens: more rows than the few-row form of the products
    takes and than the tiled attention asks for, every row a sequence of its own"""
    w = fx.random_weights(MIXED, 41)
    eng = engine_for(tmp_path, MIXED, w, queries=20)
    prompts = [tokens_for(MIXED, n, 60 + n) for n in (3, 18, 1, 40, 7, 25, 2, 33, 12, 5, 36, 37, 38, 49, 50, 51, 63, 64, 65, 4)]
    tails = [tokens_for(MIXED, 9, 80 + i) for i in range(20)]
    alone = [oracle_logits(MIXED, w, p + t) for p, t in zip(prompts, tails)]
    qs = [eng.add_query(p) for p in prompts]
    got = {q: [] for q in qs}
    assert sorted(i for i, _ in eng.infer()) == sorted(qs)
    for q in qs:
        got[q].append(eng.last_logits_f32(q))
    live = list(qs)
    for step in range(9):
        if step == 5:
            for q in qs[12:]:
                eng.remove_query(q); live.remove(q)
        eng.commit({q: tails[qs.index(q)][step] for q in live})
        assert sorted(i for i, _ in eng.infer()) == sorted(live)
        for q in live:
            got[q].append(eng.last_logits_f32(q))
    for k, q in enumerate(qs):
        g = np.concatenate(got[q], 0)
        assert fx.rel_err(g, alone[k][:len(g)]).max() < TOL32, k
    eng.close()


def plant(w, mark, probe):
    """feature 0 is set only by the token `mark`, feature 1 only by the token `probe`"""
    w["embed"][:, :2] = 0
    w["embed"][mark, 0] = 2.0; w["embed"][probe, 1] = 2.0


def marked_latent_model(shared):
    """Latent attention whose weights make one key stand out: latent channel 0 reads feature 0 alone, the last unrotated dimension of every query head
    feature 1 alone and that of the key latent channel 0 alone, so the probe's query matches the mark's key at any distance.  shared: the layer that looks
    is a second one that reads the rows of the first (whose own queries are kept blind)."""
    dn, dr, H = 12, 8, 2
    layers = [fx.latent_layer(heads=H, dim=dn, rot_dim=dr, vdim=24, kv_rank=20, scale=1.0, mlp=None)]
    if shared:
        layers.append(fx.latent_layer(heads=H, dim=dn, rot_dim=dr, vdim=16, kv_rank=20, scale=1.0, kv_from=0, mlp=None))
    cfg = fx.config(layers, width=32, vocab=50, embed_scale=2.0)
    w = fx.random_weights(cfg, 9)
    mark, probe = 7, 9
    plant(w, mark, probe)
    kv = w["l0.mix.dkv"]
    kv[:, :2] = 0; kv[0, :] = 0; kv[0, 0] = 6.0
    w["l0.mix.dkv.norm"][0] = 2.0
    for li in range(len(layers)):
        p = "l%d." % li
        w[p + "norm1"][:2] = 1.0
        q, uk = w[p + "mix.q"], w[p + "mix.uk"]
        q[:] *= 0.2; uk[:] *= 0.5; q[:, :2] = 0; uk[:, 0] = 0
        w[p + "mix.sink"][:] = 1.0
        w[p + "mix.o"][:2, :] = 0                               # the layer leaves features 0 and 1 as they were
        if shared and li == 0:
            w[p + "mix.uv"][:, 0] = 0
            continue
        w[p + "mix.uv"][:, 0] *= 3.0
        for h in range(H):
            q[h * (dn + dr) + dn - 1, :] = 0; q[h * (dn + dr) + dn - 1, 1] = 3.0
            uk[h * dn + dn - 1, :] = 0; uk[h * dn + dn - 1, 0] = 1.5
    return cfg, {k_: bf16_round(v) for k_, v in w.items()}, mark, probe


def marked_tokens(n, mark_at, mark, probe):
    filler = [t for t in range(10, 50)]
    toks = [filler[(3 * i + mark_at + n) % len(filler)] for i in range(n)]
    toks[mark_at] = mark; toks[-1] = probe
    return toks, filler


@pytest.mark.parametrize("shared", [False, True])
def test_far_keys_at_block_and_share_edges_in_prompts_and_decoding(tmp_path, shared):
    """the marked key at the borders of the tiled kernel's key blocks (32) and query tiles (128) and of the single-row kernel's chunks (16) and key
    shares (64), hundreds of tokens back"""
    cfg, w, mark, probe = marked_latent_model(shared)
    eng = engine_for(tmp_path, cfg, w, ctx=700)
    for mark_at, n in ((0, 2), (0, 33), (31, 300), (32, 300), (63, 129), (64, 129), (127, 128), (128, 130), (15, 600), (16, 600), (255, 257), (256, 258), (5, 640)):
        toks, filler = marked_tokens(n, mark_at, mark, probe)
        want = oracle_logits(cfg, w, toks)
        whole, _ = run_whole(eng, toks)
        assert fx.rel_err(whole, want).max() < TOL32, ("prompt", mark_at, n)
        dec = run_portions(eng, toks, [max(1, n - 3), 1])
        assert fx.rel_err(dec, want).max() < TOL32, ("decoded", mark_at, n)
        # the oracle itself must see the key: without the mark the last row differs clearly
        blind = list(toks); blind[mark_at] = filler[0]
        assert fx.rel_err(oracle_logits(cfg, w, blind)[-1:], want[-1:]).max() > 1e-2, (mark_at, n)
    eng.close()


def marked_chunk_model(chunk, which):
    """One attention layer in which the probe's query of map `which` matches the mark's key of that map alone (a dimension that does not turn)"""
    H, G, d, dv = 2, 1, 12, 24
    cfg = fx.config([fx.attention_layer(heads=H, kv_heads=G, dim=d, vdim=dv, chunk=chunk, rot_dims=8, scale=1.0, diff=0.4, mlp=None)], width=32, vocab=50, embed_scale=2.0)
    w = fx.random_weights(cfg, 31)
    mark, probe = 7, 9
    plant(w, mark, probe)
    w["l0.norm1"][:2] = 1.0
    q, k = w["l0.mix.q"], w["l0.mix.k"]
    q[:] *= 0.3; k[:] *= 0.5; q[:, :2] = 0; k[:, :2] = 0
    k[which * d + d - 1, :] = 0; k[which * d + d - 1, 0] = 3.0
    for h in range(H):
        r = (2 * h + which) * d + d - 1
        q[r, :] = 0; q[r, 1] = 3.0
    w["l0.mix.v"][:, 0] *= 4.0
    w["l0.mix.o"][:2, :] = 0
    return cfg, {k_: bf16_round(v) for k_, v in w.items()}, mark, probe


@pytest.mark.parametrize("which", [0, 1])
@pytest.mark.parametrize("chunk", [1, 2, 3, 16, 31, 32, 33, 64, 65, 96, 129, 250])
def test_keys_just_inside_and_just_outside_a_chunk(tmp_path, chunk, which):
    """the probe at the last, a middle and the first position of a chunk; the marked key first in that chunk (seen), last of the chunk before (not seen);
    whole prompts, portions of two tokens around the edge and decoding"""
    cfg, w, mark, probe = marked_chunk_model(chunk, which)
    eng = engine_for(tmp_path, cfg, w, ctx=900)
    start = chunk * (3 if chunk < 100 else 2)          # first position of the probe's chunk
    seen = 0
    for off in sorted({0, chunk // 2, chunk - 1}):
        n = start + off + 1
        for mark_at, inside in ((start, True), (start - 1, False)):
            if mark_at == n - 1:
                continue
            toks, filler = marked_tokens(n, mark_at, mark, probe)
            want = oracle_logits(cfg, w, toks)
            blind = list(toks); blind[mark_at] = filler[0]
            effect = fx.rel_err(oracle_logits(cfg, w, blind)[-1:], want[-1:]).max()
            assert effect > 1e-2 if inside else effect < 1e-12, (off, inside, effect)
            seen += inside
            whole, _ = run_whole(eng, toks)
            assert fx.rel_err(whole, want).max() < TOL32, ("prompt", off, inside)
            assert fx.rel_err(run_portions(eng, toks, [max(1, n - 5), 2]), want).max() < TOL32, ("portions", off, inside)
            assert fx.rel_err(run_portions(eng, toks, [max(1, start - 2), 1]), want).max() < TOL32, ("decoded", off, inside)
    assert seen == (0 if chunk == 1 else len({chunk // 2, chunk - 1}))
    eng.close()


def test_sinks_count_once_in_both_forms(tmp_path):
    """sinks far above, near and far below the scores: with a large one a head says nearly nothing, and more the more keys match"""
    cfg = fx.config([fx.latent_layer(heads=4, dim=16, rot_dim=8, vdim=16, kv_rank=24, mlp=None), fx.latent_layer(heads=4, dim=16, rot_dim=8, vdim=16, kv_rank=24, kv_from=0)], width=48, vocab=41)
    w = fx.random_weights(cfg, 61)
    toks = tokens_for(cfg, 100, 62)
    for sinks in ([9.0, 3.0, 0.0, -6.0], [-30.0] * 4, [20.0] * 4):
        for li in range(2):
            w["l%d.mix.sink" % li][:] = sinks
        w = {k: bf16_round(v) for k, v in w.items()}
        want = oracle_logits(cfg, w, toks)
        eng = engine_for(tmp_path, cfg, w)
        assert fx.rel_err(run_whole(eng, toks)[0], want).max() < TOL32
        assert fx.rel_err(run_portions(eng, toks, [60, 1]), want).max() < TOL32
        eng.close()


def test_long_decoding(tmp_path):
    cfg = fx.config([fx.latent_layer(heads=2, dim=16, rot_dim=8, vdim=8, kv_rank=24, base=200.0), fx.attention_layer(heads=2, kv_heads=1, dim=16, vdim=16, chunk=45, rot_dims=16),
                     fx.latent_layer(heads=2, dim=8, rot_dim=8, vdim=12, kv_rank=24, base=200.0, kv_from=0), fx.attention_layer(heads=4, kv_heads=2, dim=8, vdim=24, chunk=130, rot_dims=4)],
                    width=32, vocab=61)
    w = fx.random_weights(cfg, 11)
    toks = tokens_for(cfg, 330, 12)
    want = oracle_logits(cfg, w, toks)
    eng = engine_for(tmp_path, cfg, w, ctx=400)
    got = run_portions(eng, toks, [170, 1])        # 160 tokens decoded one by one, across four chunk borders
    assert fx.rel_err(got, want).max() < TOL32
    got = run_portions(eng, toks, [1])             # all of them
    assert fx.rel_err(got, want).max() < TOL32
    eng.close()


CASES = {
    # one head of one dimension (two for the rotated pair), a latent of one, a chunk of one, scales of one, nothing taken off but what the vectors say
    "ones": lambda: fx.config([fx.latent_layer(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, scale=1.0, mlp=fx.dense(1)),
                               fx.attention_layer(heads=1, kv_heads=1, dim=2, vdim=2, chunk=1, rot_dims=2, scale=1.0, diff=0.0, mlp=None),
                               fx.attention_layer(heads=1, kv_heads=1, dim=2, vdim=1, chunk=8, rot_dims=2, scale=1.0, diff=0.0, mlp=fx.dense(1))], width=16, vocab=11, embed_scale=1.0),
    # sizes that keep every 16-byte path off
    "unaligned": lambda: fx.config([fx.attention_layer(heads=3, kv_heads=3, dim=7, vdim=5, chunk=11, rot_dims=6, mlp=fx.dense(9)),
                                    fx.latent_layer(heads=3, dim=5, rot_dim=6, vdim=7, kv_rank=9, mlp=fx.dense(13)),
                                    fx.latent_layer(heads=7, dim=3, rot_dim=6, vdim=1, kv_rank=9, kv_from=1, mlp=fx.dense(3))], width=14, vocab=9),
    # the widest heads of the tiled kernels
    "wide": lambda: fx.config([fx.latent_layer(heads=2, dim=128, rot_dim=64, vdim=128, kv_rank=256, mlp=fx.dense(96)),
                               fx.attention_layer(heads=2, kv_heads=1, dim=128, vdim=256, chunk=40, rot_dims=128)], width=128, vocab=50),
    # heads beyond the tiled kernels (prompts take the single-row forms), value heads of several column groups
    "beyond": lambda: fx.config([fx.latent_layer(heads=2, dim=160, rot_dim=64, vdim=136, kv_rank=72), fx.attention_layer(heads=2, kv_heads=2, dim=132, vdim=40, chunk=33, rot_dims=20),
                                 fx.attention_layer(heads=4, kv_heads=1, dim=20, vdim=300, chunk=30, rot_dims=20, mlp=None)], width=64, vocab=23),
    # many heads on one key / value head, a group that does not fill the row kernel's blocks, a feed-forward narrower and wider than the model, no latent layer
    "heads": lambda: fx.config([fx.attention_layer(heads=16, kv_heads=1, dim=8, vdim=16, chunk=29, rot_dims=8, mlp=fx.dense(8)),
                                fx.attention_layer(heads=10, kv_heads=2, dim=36, vdim=36, chunk=64, rot_dims=12, diff=0.9, mlp=fx.dense(300))], width=40, vocab=29),
    # sizes in whole 64s: prompts in bfloat16 hand every operand on as it is read (norms, attention outputs, the squared relu); one feed-forward that does not
    "sixty_fours": lambda: fx.config([fx.latent_layer(heads=4, dim=24, rot_dim=8, vdim=16, kv_rank=64, mlp=fx.dense(128)), fx.attention_layer(heads=4, kv_heads=2, dim=16, vdim=32, chunk=40, rot_dims=16),
                                      fx.latent_layer(heads=2, dim=24, rot_dim=8, vdim=32, kv_rank=64, kv_from=0, mlp=None), fx.attention_layer(heads=2, kv_heads=1, dim=16, vdim=64, rot_dims=16, mlp=fx.dense(192))],
                                     width=128, vocab=67),
    # latent layers only, three readers of one source, the reader of another in between
    "readers": lambda: fx.config([fx.latent_layer(kv_rank=20), fx.latent_layer(kv_rank=24, rot_dim=4), fx.latent_layer(heads=1, dim=40, vdim=40, kv_rank=20, kv_from=0),
                                  fx.latent_layer(heads=6, dim=4, vdim=8, kv_rank=24, rot_dim=4, kv_from=1), fx.latent_layer(heads=2, dim=8, vdim=20, kv_rank=20, kv_from=0, mlp=None)],
                                 width=48, vocab=31, eps=1e-3),
    # no rotation, no chunks, a chunk longer than every sequence
    "plain": lambda: fx.config([fx.attention_layer(rot_dims=0, chunk=None), fx.attention_layer(chunk=5000, rot_dims=2)], width=32, vocab=40),
}


@pytest.mark.parametrize("case", sorted(CASES))
def test_other_sizes(tmp_path, case):
    cfg = CASES[case]()
    w = fx.random_weights(cfg, 13)
    toks = tokens_for(cfg, 75, 14)
    want = oracle_logits(cfg, w, toks)
    for dtype, tol in (("float32", 1e-4 if case == "ones" else TOL32), ("bfloat16", 1.0 if case == "ones" else 2 * TOL16)):          # (a head of one value keeps its sign only)
        eng = engine_for(tmp_path, cfg, w, dtype)
        whole, _ = run_whole(eng, toks)
        assert fx.rel_err(whole, want).max() < tol, (case, dtype, fx.rel_err(whole, want).max())
        parts = run_portions(eng, toks, [20, 9, 1])
        assert fx.rel_err(parts, want).max() < tol, (case, dtype, "portions", fx.rel_err(parts, want).max())
        eng.close()


def test_configurations_that_do_not_hold_are_refused(tmp_path):
    from inferflow_amd.engine import InferenceEngine
    good = fx.config([fx.latent_layer(), fx.latent_layer(kv_from=0), fx.attention_layer()], width=32, vocab=31)
    w = fx.random_weights(good, 1)

    def broken(change):
        cfg = json.loads(json.dumps(good))
        change(cfg)
        d = fx.write_model_dir(str(tmp_path / ("b%d" % len(os.listdir(tmp_path)))), cfg, w)
        with pytest.raises(Exception):
            InferenceEngine.from_model_dir(d, "float32", 64, 1, True)
    broken(lambda c: c["layers"][1]["mixer"].update(kv_from=1))                       # not an earlier layer
    broken(lambda c: c["layers"][1]["mixer"].update(kv_rank=20))                      # another latent size than the source's
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(base=2.0))                 # another rotation
    broken(lambda c: c["layers"][2]["mixer"].update(kv_from=0))                       # rows of another kind of layer
    broken(lambda c: c["layers"][2]["mixer"]["mask"].update(size=0))
    broken(lambda c: c["layers"][2]["mixer"].pop("diff"))
    broken(lambda c: c["layers"][0].update(type="other"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda c: c["layers"][0]["mixer"].update(dim=24))                          # not what the tensors hold


def test_greedy_generation_through_the_engine(tmp_path):
    w = fx.random_weights(MIXED, 15)
    prompt = tokens_for(MIXED, 29, 16)
    eng = engine_for(tmp_path, MIXED, w)
    # Generate(): prompt step + decode steps replayed from a captured graph with the token fed back on the device, across chunk borders
    q = eng.add_query(prompt)
    gen, _ = eng.generate(q, 40)
    eng.remove_query(q)
    # the serving loop: Infer -> Commit of the greedy token
    q = eng.add_query(prompt)
    loop = []
    for _ in range(40):
        (qq, tok), = eng.infer()
        loop.append(tok); eng.commit({q: tok})
    eng.remove_query(q)
    assert gen == loop
    # the oracle follows the same tokens and agrees wherever its two best logits are clearly apart

    def follows(prompt, gen):
        want = oracle_logits(MIXED, w, prompt + gen)
        for i, tok in enumerate(gen):
            row = want[len(prompt) - 1 + i]
            top2 = np.sort(row)[-2:]
            if top2[1] - top2[0] > 1e-3 * np.abs(row).max():
                assert tok == int(row.argmax()), i
    follows(prompt, gen)
    # a second generation on the same slot replays the captured step against a new sequence
    q = eng.add_query(prompt[:7])
    gen2, _ = eng.generate(q, 10)
    eng.remove_query(q)
    follows(prompt[:7], gen2)
    # sampled queries draw from the same logits (top-k with a seed: reproducible)
    a = eng.add_query(prompt, strategy="sample.top_k", seed=5)
    b = eng.add_query(prompt, strategy="sample.top_k", seed=5)
    out = dict(eng.infer())
    assert out[a] == out[b] and 0 <= out[a] < MIXED["vocab"]
    eng.close()


def test_generation_right_behind_a_step_of_several_prompts(tmp_path):
    """the decode step is captured after a step of three long prompts: its launches must be shaped for one row, and replay on every slot"""
    w = fx.random_weights(MIXED, 71)
    eng = engine_for(tmp_path, MIXED, w, queries=4)
    prompts = [tokens_for(MIXED, n, 72 + n) for n in (60, 41, 100)]
    qs = [eng.add_query(p) for p in prompts]
    eng.infer()
    for q in qs[:2]:
        eng.remove_query(q)
    short = tokens_for(MIXED, 3, 79)
    for prompt in (short, prompts[1], short):
        q = eng.add_query(prompt)
        gen, _ = eng.generate(q, 8)
        eng.remove_query(q)
        want = oracle_logits(MIXED, w, prompt + gen)
        for i, tok in enumerate(gen):
            row = want[len(prompt) - 1 + i]
            top2 = np.sort(row)[-2:]
            if top2[1] - top2[0] > 1e-3 * np.abs(row).max():
                assert tok == int(row.argmax()), (len(prompt), i)
    eng.close()


def test_ini_route_and_trace_replay_tool(tmp_path):
    from inferflow_amd.engine import InferenceEngine
    w = fx.random_weights(MIXED, 17)
    d = fx.write_model_dir(str(tmp_path / "model"), MIXED, w)
    ini = tmp_path / "serve.ini"
    ini.write_text("[transformer_engine]\nmodels = m\ndevices = 0\nmax_concurrent_queries = 2\nreturn_output_tensors_f32 = true\n\n"
                   "[model.m]\nmodel_dir = %s/\ncompute_dtype = float32\nmax_context_len = 100\n" % d)
    eng = InferenceEngine.from_ini(str(ini))
    toks = tokens_for(MIXED, 30, 18)
    lg, _ = run_whole(eng, toks)
    want = oracle_logits(MIXED, w, toks)
    assert fx.rel_err(lg, want).max() < TOL32
    assert eng.model_info("vocab_size") == MIXED["vocab"] and eng.model_info("decoder_layers") == len(MIXED["layers"])
    eng.close()
    # the trace tool: two requests start together, go on token by token, one ends earlier
    a, b = tokens_for(MIXED, 46, 19), tokens_for(MIXED, 9, 20)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:34], "want": [0, 33]}, {"id": "b", "tokens": b[:6], "want": [5]}], "end": []}]
    for s in range(1, 13):
        ent = [{"id": "a", "tokens": [a[33 + s]], "want": [0]}]
        if s <= 3:
            ent.append({"id": "b", "tokens": [b[5 + s]], "want": [0] if s != 2 else []})
        steps.append({"step": s, "entries": ent, "end": (["b"] if s == 3 else []) + (["a"] if s == 12 else [])})
    out = tmp_path / "out"; out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out", str(out), "--max-tokens", "64"],
                       input="".join(json.dumps(s) + "\n" for s in steps).encode(), stdout=subprocess.PIPE, stderr=subprocess.PIPE, timeout=900)
    assert r.returncode == 0, r.stderr.decode()[-2000:]
    assert [l for l in r.stdout.decode().split() if l != "done"] == [str(s) for s in range(13)]
    wa, wb = oracle_logits(MIXED, w, a), oracle_logits(MIXED, w, b)
    V = MIXED["vocab"]
    g0 = np.fromfile(out / "0.f32", np.float32).reshape(-1, V)
    assert fx.rel_err(g0, np.stack([wa[0], wa[33], wb[5]])).max() < TOL32
    for s in range(1, 13):
        g = np.fromfile(out / ("%d.f32" % s), np.float32).reshape(-1, V)
        exp = [wa[33 + s]] + ([wb[5 + s]] if s <= 3 and s != 2 else [])
        assert fx.rel_err(g, np.stack(exp)).max() < TOL32, s
