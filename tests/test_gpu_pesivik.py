"""GPU tests of the Pesivik design in the layer-stack model class: every operator alone with planted values, every mechanism as a one-layer
model, then whole models of small random configurations through the engine — against tests/pesivik_oracle.py (float64, whole sequences,
keys and values up-projected, no cache, no pages).

f32 models must agree with the oracle to f32 rounding, bf16 models to bf16 rounding; and the logits of a position must not depend on how
its prompt was cut, on the rest of the batch or on the pages it got.
"""
import json
import math
import os
import struct
import subprocess
import sys

import numpy as np
import pytest

from tests import pesivik_oracle as po
from tests.test_gpu_stack import BF16, F32, build, check, empty, from_dev, raw, rel, to_dev, tokens_of
from tests.test_gpu_stack import _buffers_live_until_the_test_ends  # noqa: F401  (autouse: device buffers outlive the launches)
from vllm_rs_amd import _lib, checkpoint

pytestmark = pytest.mark.gpu

f32 = lambda a: raw(a, np.float32)


def mixer(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=48, q_rank=40, scale=0.25, size=70, base=2000.0):
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale, mask=dict(size=size), rot=dict(base=base, dims=rot_dim))


def moe(experts=6, top=2, ff=40, groups=(3, 2), shared=24):
    m = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if groups:
        m["router"]["groups"] = dict(count=groups[0], keep=groups[1])
    if shared:
        m["shared"] = dict(ff=shared)
    return m


def layer(mx=None, mlp=None, **kw):
    return dict(type="latent_attention", mixer=mx or mixer(), mlp=mlp, **kw)


def config(layers, width=96, vocab=160, eps=2e-5, scale=4.0, cap=9.0):
    return dict(architecture="Pesivik", width=width, vocab=vocab, norm=dict(eps=eps), embedding=dict(scale=scale), logit_softcap=cap, layers=layers)


def config_a():
    """sizes on the matrix-core paths; windows longer and shorter than a page; layers that share tensors (one with a forward reference), a layer
    without feed-forward, routers with and without groups, with and without a shared expert, top 1"""
    return config([
        layer(mlp=moe()),
        layer(mixer(heads=5, dim=8, rot_dim=16, vdim=16, kv_rank=32, q_rank=24, size=9, scale=0.4, base=50.0)),
        layer(mlp=moe(), weights_of=0),
        layer(mixer(heads=2, size=200), mlp=moe(experts=4, top=1, groups=None, shared=None), weights_of=4),
        layer(mixer(heads=2, size=200), mlp=moe(experts=4, top=1, groups=None, shared=None)),
        layer(mixer(heads=4, dim=24, rot_dim=8, vdim=32, kv_rank=64, q_rank=56, size=64), mlp=moe(experts=8, top=3, ff=24, groups=(4, 1 + 1), shared=72)),
    ])


def config_b():
    """sizes off every 16-byte path: width 50, heads of 5 / 7 channels, ranks 9 and 11, a window of 5, groups of one expert, top = every expert"""
    return config([
        layer(mixer(heads=2, dim=5, rot_dim=2, vdim=7, kv_rank=9, q_rank=11, size=5, scale=0.6, base=100.0), mlp=moe(experts=3, top=3, ff=11, groups=(3, 3), shared=13)),
        layer(mixer(heads=3, dim=7, rot_dim=6, vdim=5, kv_rank=13, q_rank=7, size=33, scale=0.5, base=1e5), mlp=moe(experts=4, top=2, ff=9, groups=(4, 2), shared=None)),
        layer(mixer(heads=2, dim=5, rot_dim=2, vdim=7, kv_rank=9, q_rank=11, size=5, scale=0.6, base=100.0), mlp=moe(experts=3, top=3, ff=11, groups=(3, 3), shared=13), weights_of=0),
    ], width=50, vocab=70, eps=1e-6, scale=0.7, cap=4.0)


def agree(got, ref, dt, what=""):
    """rows against the oracle's.  f32: every row to f32 rounding.  bf16: a close call of a router (a discrete choice) may turn a token, so the
    rows are judged one by one: the typical row to bf16 rounding, three in four within a few times that"""
    got, ref = np.asarray(got, np.float64), np.asarray(ref, np.float64)
    got, ref = got.reshape(-1, got.shape[-1]), ref.reshape(-1, ref.shape[-1])
    rows = np.sqrt(((got - ref) ** 2).mean(-1)) / np.maximum(np.sqrt((ref ** 2).mean(-1)), 1e-30)
    if dt == F32:
        assert rows.max() < 2e-4 and rel(got, ref) < 3e-5, (what, rows.max(), rel(got, ref))
    else:
        assert np.median(rows) < 4e-2 and np.quantile(rows, 0.75) < 8e-2, (what, float(np.median(rows)), float(np.quantile(rows, 0.75)))


def same(a, b, dt):
    """the same rows computed in two ways"""
    return rel(a, b) < (1e-5 if dt == F32 else 3e-2)


def every(n):
    return list(range(n))


# ------------------------------------------------------------------------------------------------ operators alone
@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("T,W,E,top,groups,keep", [(9, 96, 6, 3, 3, 2), (3, 51, 5, 5, 0, 0), (200, 256, 32, 4, 8, 3), (7, 64, 8, 2, 8, 5), (5, 128, 72, 3, 8, 2), (1, 2048, 16, 2, 4, 2),
                                                   (150, 1032, 20, 3, 5, 5), (2, 4100, 9, 2, 3, 1)])
def test_seam_with_layer_norms_and_normalised_router(dt, T, W, E, top, groups, keep):
    """x += LN(sum_j w_j part_j + part2) * w; h = LN(x) * w; the router: sigmoid scores, corrected choice inside the groups whose two best
    corrected scores sum highest, weights = the chosen scores over their sum.  Rows with a large common offset (the mean must be taken off
    before squaring); every choice score negative; equal logits (the lower index wins)."""
    L = _lib.load()
    r = np.random.default_rng(W + E)
    eps, n1 = 1e-5, 2
    f = lambda *s: r.standard_normal(s).astype(np.float32)
    x, p1, p2, pw = f(T, W) + 30.0, 3.0 * f(T * n1, W) - 5.0, 0.2 * f(T, W), r.random(T * n1).astype(np.float32)
    post, pre = 1 + 0.2 * f(W), 1 + 0.2 * f(W)
    rw = po.bf16_round(3.0 * f(E, W) / math.sqrt(W))
    corr = (0.3 * f(E) - 2.0).astype(np.float32)
    s = (pw[:, None].astype(np.float64) * p1).reshape(T, n1, W).sum(1) + p2
    x_ref = x + po.layer_norm(s, post, eps)
    h_ref = po.layer_norm(x_ref, pre, eps)
    router = dict(top=top)
    if groups:
        router["groups"] = dict(count=groups, keep=keep)
    chosen, wt = po.route(h_ref, router, {"router": rw.astype(np.float64), "correction": corr.astype(np.float64)}, "")
    xd, hd, h32 = f32(x), empty(T * W * 4), empty(T * W * 4)
    pe, pwt = empty(T * top * 4), empty(T * top * 4)
    d = lambda a: f32(a).ptr

    def seam(xd, rw, corr, with_parts=True):
        L.vra_stack_op_seam(xd.ptr, d(p1) if with_parts else None, n1, d(pw), None, 1.0, d(p2) if with_parts else None, None, 1.0, None, None, 2,
                            d(post) if with_parts else None, None, 1.0, d(pre), None, 1.0, hd.ptr, h32.ptr, eps, T, W, to_dev(rw, dt).ptr, d(corr), 2, E, top,
                            groups, keep, 0, pe.ptr, pwt.ptr, None, dt, 0)
        check()
        return pe.numpy(np.int32, (T, top)), pwt.numpy(np.float32, (T, top))
    experts, weights = seam(xd, rw, corr)
    assert rel(xd.numpy(np.float32, (T, W)) - 30.0, x_ref - 30.0) < 2e-6 and rel(h32.numpy(np.float32, (T, W)), h_ref) < 5e-6
    assert rel(from_dev(hd, (T, W), dt), h_ref) < (5e-6 if dt == F32 else 4e-3)
    for t in range(T):
        order = np.argsort(experts[t])
        assert experts[t][order].tolist() == sorted(chosen[t].tolist()), t
        assert np.allclose(weights[t][order], wt[t][np.argsort(chosen[t])], atol=1e-5)
        assert abs(weights[t].sum() - 1.0) < 1e-5
    # no logits: the correction alone chooses.  The best expert's group loses against one whose two best sum higher.
    if groups and groups < E and keep < groups and top <= keep * (E // groups):
        per = E // groups
        c2 = np.full(E, -4.0, np.float32)
        c2[per - 1] = -1.0                                  # the best single expert, alone in the first group: worth -1 - 4
        for g in range(groups - keep, groups):
            c2[g * per], c2[g * per + 1] = -2.0, -2.5       # `keep` groups of worth -4.5
        experts, weights = seam(f32(x), np.zeros((E, W), np.float32), c2, False)
        allowed = {e for g in range(groups - keep, groups) for e in range(g * per, (g + 1) * per)}
        assert set(experts.reshape(-1).tolist()) <= allowed and np.allclose(weights, 1.0 / top, atol=1e-6)
    experts, weights = seam(f32(x), np.zeros((E, W), np.float32), np.zeros(E, np.float32), False)
    if not groups or top <= keep * (E // groups):
        assert (np.sort(experts, -1) == np.arange(top)[None, :]).all() and np.allclose(weights, 1.0 / top, atol=1e-6)


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("M,N,K", [(3, 40, 96), (70, 136, 64), (1100, 2064, 96), (20, 33, 51)])
def test_element_wise_epilogues(dt, M, N, K):
    """exact gelu (epi 2, bf16 or f32 output) and the soft cap of f32 logits, for every matrix kernel (few rows, 64-row tiles, 128-row tiles,
    FMA), and with rows gathered by expert"""
    L = _lib.load()
    r = np.random.default_rng(M)
    a, w = po.bf16_round(r.standard_normal((M, K)).astype(np.float32)), po.bf16_round((2.0 * r.standard_normal((N, K)) / math.sqrt(K)).astype(np.float32))
    z = a.astype(np.float64) @ w.astype(np.float64).T
    ad, wd = to_dev(a, dt), to_dev(w, dt)
    out = empty(M * N * 4)
    L.vra_stack_op_gemm_post(ad.ptr, K, wd.ptr, 0, out.ptr, N, 0, M, N, K, 1.0, None, None, 0, None, None, 2, 3, 0.0, dt, 0)
    check()
    assert rel(from_dev(out, (M, N), dt), po.gelu_erf(z)) < (2e-6 if dt == F32 else 4e-3)
    L.vra_stack_op_gemm_post(ad.ptr, K, wd.ptr, 0, out.ptr, N, 1, M, N, K, 3.0, None, None, 0, None, None, 0, 0, 2.5, dt, 0)
    check()
    got = out.numpy(np.float32, (M, N))
    assert rel(got, 2.5 * np.tanh(3.0 * z / 2.5)) < 3e-6 and np.abs(got).max() <= 2.5
    # two experts: granules of 16 rows, gathered rows, rows that hold no pair
    rows = np.full(48, -1, np.int32)
    rows[:11], rows[16:33] = r.integers(0, M, 11), r.integers(0, M, 17)
    groups = np.array([1, 0, 0], np.int32)
    w2 = np.stack([w, -0.5 * w])
    res = empty(48 * N * 4)
    L.vra_stack_op_gemm_post(ad.ptr, K, to_dev(w2, dt).ptr, N * K, res.ptr, N, 1, 48, N, K, 1.0, None, raw(groups, np.int32).ptr, 16, raw(rows, np.int32).ptr, None, 2, 3, 0.0, dt, 0)
    check()
    got = res.numpy(np.float32, (48, N))
    for i in range(48):
        if rows[i] >= 0:
            assert rel(got[i], po.gelu_erf(a[rows[i]].astype(np.float64) @ w2[groups[i // 16]].astype(np.float64).T)) < 5e-6


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("rd,base", [(8, 500.0), (32, 5e5), (2, 10.0)])
def test_rotate_half_layout(dt, rd, base):
    """the rotated key part of a latent row and the rotated tail of every head's query, far positions included"""
    L = _lib.load()
    r = np.random.default_rng(rd)
    pos = np.array([0, 1, 63, 64, 700, 4095, 100000], np.int64)
    T, qr, kr, H, dim = len(pos), 12, 20, 3, 6
    fr = base ** (-2.0 * np.arange(rd // 2) / rd)
    fh = fr.astype(np.float32)
    fl = (fr - fh.astype(np.float64)).astype(np.float32)
    rows = r.standard_normal((T, qr + kr + rd)).astype(np.float32)
    cq, cache = empty(T * qr * 4), empty(T * (kr + rd) * 4)
    qn, kn = (1 + 0.2 * r.standard_normal(qr)).astype(np.float32), (1 + 0.2 * r.standard_normal(kr)).astype(np.float32)
    L.vra_stack_op_latent_prep(f32(rows).ptr, qr + kr + rd, qr, kr, rd, f32(qn).ptr, f32(kn).ptr, 1e-5, cq.ptr, cache.ptr, kr + rd,
                               raw(np.arange(T)[::-1], np.int64).ptr, raw(pos, np.int64).ptr, f32(fh).ptr, f32(fl).ptr, rd // 2, 1.0, 1, T, dt, 0)
    check()
    got = from_dev(cache, (T, kr + rd), dt)[::-1]
    tol = 3e-5 if dt == F32 else 3e-2
    assert np.abs(got[:, kr:] - po.rotate_half(rows[:, qr + kr:].astype(np.float64), pos, base)).max() < tol
    assert rel(got[:, :kr], po.rms_norm(rows[:, qr:qr + kr].astype(np.float64), kn, 1e-5)) < (2e-6 if dt == F32 else 4e-3)
    assert rel(from_dev(cq, (T, qr), dt), po.rms_norm(rows[:, :qr].astype(np.float64), qn, 1e-5)) < (2e-6 if dt == F32 else 4e-3)
    q = po.bf16_round(r.standard_normal((T, H, dim + rd)).astype(np.float32))
    out = empty(T * H * (kr + rd) * 4).fill_bytes(0)
    L.vra_stack_op_rope_heads(to_dev(q.reshape(T, -1), dt).ptr, H * (dim + rd), dim + rd, dim, out.ptr, H * (kr + rd), kr + rd, kr, rd, H, raw(pos, np.int64).ptr,
                              f32(fh).ptr, f32(fl).ptr, rd // 2, 1.0, 1, T, dt, 0)
    check()
    got = from_dev(out, (T, H, kr + rd), dt)
    assert np.abs(got[:, :, kr:] - po.rotate_half(q[:, :, dim:].astype(np.float64), pos, base)).max() < tol and (got[:, :, :kr] == 0).all()


def latent_cache(rows, BS, r, dt, extra=3):
    """cache rows of ONE sequence over shuffled pages; every other slot holds large values that nobody may read"""
    Tk = rows.shape[0]
    nb = (Tk + BS - 1) // BS
    table = r.permutation(nb + extra)[:nb].astype(np.uint32)
    pool = np.full(((nb + extra) * BS, rows.shape[1]), 1e4, np.float32)
    for j in range(Tk):
        pool[int(table[j // BS]) * BS + j % BS] = rows[j]
    return to_dev(pool, dt), table


def run_latent(L, q, positions, rows, vdim, scale, window, gate, dt, form, r, sink=None, BS=64, splits=3):
    """form: "prompt" (all queries in one step), "decoded" (one launch per query), "parts" (decoded, the key range in parts)"""
    Tq, H, kd = q.shape
    cache, table = latent_cache(rows, BS, r, dt)
    sk = f32(sink).ptr if sink is not None else None
    tb = raw(table, np.uint32).ptr
    if form == "prompt":
        out = empty(Tq * H * vdim * 4)
        L.vra_stack_op_attention_latent(to_dev(q.reshape(Tq, -1), dt).ptr, H * kd, out.ptr, cache.ptr, kd, raw(positions, np.int64).ptr, tb,
                                        raw([rows.shape[0]], np.uint32).ptr, raw([0, Tq], np.uint32).ptr, 1, Tq, Tq, H, kd, vdim, BS, len(table), scale, window, sk, None,
                                        f32(gate).ptr, H, None, 0, 0, dt, 0)
        check()
        return from_dev(out, (Tq, H, vdim), dt)
    out = empty(Tq * H * vdim * 4)  # all queries as sequences of one batch that share their pages
    scratch = empty(Tq * splits * H * (vdim + 2) * 4)
    L.vra_stack_op_attention_latent(to_dev(q.reshape(Tq, -1), dt).ptr, H * kd, out.ptr, cache.ptr, kd, raw(positions, np.int64).ptr,
                                    raw(np.tile(table, (Tq, 1)), np.uint32).ptr, raw(np.asarray(positions) + 1, np.uint32).ptr, None, Tq, Tq, 1, H, kd, vdim, BS,
                                    len(table), scale, window, sk, None, f32(gate).ptr, H, scratch.ptr if form == "parts" else None,
                                    Tq * splits * H * (vdim + 2) * 4, splits, dt, 0)
    check()
    return from_dev(out, (Tq, H, vdim), dt)


def latent_reference(q, positions, rows, vdim, scale, window, gate):
    H = q.shape[1]
    k = np.repeat(rows.astype(np.float64)[:, None, :], H, 1)
    vis = po.in_window(positions, rows.shape[0], window if window > 0 else 10 ** 9)
    return po.windowed_attention(q.astype(np.float64), k, k[:, :, :vdim], scale, vis) * po.sigmoid(gate.astype(np.float64))[:, :, None]


# row width, value width, heads: every instantiation of the matrix-core kernels (rows up to 128 / 192 / 256 / 384 / 576) and shapes off their paths
LATENT_SHAPES = [(72, 48, 3), (128, 96, 4), (160, 112, 2), (192, 160, 5), (256, 192, 16), (248, 240, 1), (320, 272, 2), (576, 512, 20), (35, 13, 2), (600, 560 - 48, 1), (300, 300 - 20, 2)]


@pytest.mark.parametrize("form,dt", [("prompt", F32), ("prompt", BF16), ("decoded", F32), ("decoded", BF16), ("parts", BF16)])
@pytest.mark.parametrize("kd,vdim,H", LATENT_SHAPES)
def test_latent_attention_against_the_oracle(form, dt, kd, vdim, H):
    """random rows, queries across page borders, several windows; first tokens of a sequence included"""
    L = _lib.load()
    r = np.random.default_rng(kd + H)
    Tk = 300
    rows = po.bf16_round(r.standard_normal((Tk, kd)).astype(np.float32))
    positions = np.array([0, 1, 2, 31, 32, 63, 64, 65, 127, 128, 200, 298, 299] if form != "prompt" else list(range(0, 40)) + list(range(230, 300)), np.int64)
    q = po.bf16_round((2.0 * r.standard_normal((len(positions), H, kd))).astype(np.float32))
    gate = r.standard_normal((len(positions), H)).astype(np.float32)
    sc = 1.0 / math.sqrt(kd)
    for window in (1, 33, 64, 100, 0):
        ref = latent_reference(q, positions, rows, vdim, sc, window, gate)
        for splits in ((1, 3, 7) if form == "parts" else (3,)):
            got = run_latent(L, q, positions, rows, vdim, sc, window, gate, dt, form, r, splits=splits)
            assert rel(got, ref) < (1e-5 if dt == F32 else 4e-3), (window, splits)


@pytest.mark.parametrize("form,dt", [("prompt", F32), ("prompt", BF16), ("decoded", F32), ("decoded", BF16), ("parts", BF16)])
@pytest.mark.parametrize("window,kr,rd", [(150, 32, 8), (64, 192, 64), (70, 96, 32), (1, 64, 16), (0, 512, 64)])
def test_planted_key_at_window_edges(form, dt, window, kr, rd):
    """one key stands out among 900 (its latent is a marker).  A query at the key's position or up to window - 1 positions behind it returns the
    marker — also across page borders; a query one position further, or before the key, does not feel it at all"""
    L = _lib.load()
    r = np.random.default_rng(window + kr)
    Tk, H = 900, 3
    base = po.bf16_round((0.1 * r.standard_normal((Tk, kr + rd))).astype(np.float32))
    u = np.zeros(kr + rd, np.float32)
    u[kr + 3] = 1.0  # (the stand-out score lives in the rotated part: the marker in the latent stays a plain value)
    w = window if window > 0 else Tk
    for j in (0, 63, 64, 400, 899 - min(w - 1, 5)):
        rows = base.copy()
        rows[j] = 16.0 * u
        rows[j, :kr] = 5.0
        positions = np.array(sorted({p for p in (j - 1, j, j + 1, j + w - 2, j + w - 1, j + w, j + w + 1, 899) if 0 <= p < Tk}), np.int64)
        q = np.tile(8.0 * u, (len(positions), H, 1)).astype(np.float32)
        gate = r.standard_normal((len(positions), H)).astype(np.float32)
        got = run_latent(L, q, positions, rows, kr, 0.25, window, gate, dt, form, r, splits=4)
        ref = latent_reference(q, positions, rows, kr, 0.25, window, gate)
        g = po.sigmoid(gate.astype(np.float64))[:, :, None]
        for i, p in enumerate(positions):
            if j <= p < j + w:
                assert np.abs(got[i] / g[i] - 5.0).max() < 4e-2, (j, p)
            else:
                assert np.abs(got[i]).max() < 1.0, (j, p)
        assert rel(got, ref) < (2e-5 if dt == F32 else 6e-3)


@pytest.mark.parametrize("form", ["prompt", "parts"])
def test_scores_that_rise_by_little_and_by_much(form):
    """the running reference of a row moves only when a score exceeds it by more than a margin: scores that climb in small steps, jump, and
    fall, over several tiles; and a sink above or below them"""
    L = _lib.load()
    r = np.random.default_rng(5)
    Tk, kr, rd, H = 400, 64, 16, 2
    rows = po.bf16_round((0.2 * r.standard_normal((Tk, kr + rd))).astype(np.float32))
    climb = np.concatenate([np.linspace(-30, 30, 200), np.linspace(60, -60, 100), np.full(100, 50.0)])
    rows[:, kr] = po.bf16_round(climb.astype(np.float32))
    positions = np.array([5, 40, 100, 190, 201, 250, 320, 399], np.int64)
    q = po.bf16_round((0.2 * r.standard_normal((len(positions), H, kr + rd))).astype(np.float32))
    q[:, :, kr] = 1.0
    gate = np.full((len(positions), H), 40.0, np.float32)
    for window in (0, 90):
        ref = latent_reference(q, positions, rows, kr, 1.0, window, gate)
        assert rel(run_latent(L, q, positions, rows, kr, 1.0, window, gate, BF16, form, r), ref) < 4e-3
        low = run_latent(L, q, positions, rows, kr, 1.0, window, gate, BF16, form, r, sink=np.full(H, -200.0, np.float32))
        assert rel(low, ref) < 4e-3
        high = run_latent(L, q, positions, rows, kr, 1.0, window, gate, BF16, form, r, sink=np.full(H, 150.0, np.float32))
        assert np.abs(high).max() < 1e-20


def test_prompt_rows_do_not_depend_on_their_neighbours():
    """one query row alone, in a short portion and in a step that fills the chip (another workgroup size): the same bits"""
    L = _lib.load()
    r = np.random.default_rng(9)
    Tk, kr, rd, H = 2200, 64, 16, 16
    rows = po.bf16_round(r.standard_normal((Tk, kr + rd)).astype(np.float32))
    q = po.bf16_round((2.0 * r.standard_normal((Tk, H, kr + rd))).astype(np.float32))
    gate = r.standard_normal((Tk, H)).astype(np.float32)
    pos = np.arange(Tk, dtype=np.int64)
    whole = run_latent(L, q, pos, rows, kr, 0.1, 300, gate, BF16, "prompt", r)
    for a, b in ((0, 5), (1000, 1037), (2199, 2200), (511, 513)):
        part = run_latent(L, q[a:b], pos[a:b], rows[:b], kr, 0.1, 300, gate[a:b], BF16, "prompt", r)
        assert (part == whole[a:b]).all(), (a, b)


# ------------------------------------------------------------------------------------------------ each mechanism as a one-layer model
ALONE = {
    "attention": [layer()],
    "attention-one-head": [layer(mixer(heads=1, dim=24, rot_dim=8, vdim=16, kv_rank=32, q_rank=32, size=40))],
    "attention-wide-latent": [layer(mixer(heads=2, dim=32, rot_dim=64, vdim=16, kv_rank=512, q_rank=72, size=100, scale=0.05))],
    "attention-latent-320": [layer(mixer(heads=4, dim=16, rot_dim=32, vdim=16, kv_rank=320, q_rank=48, size=90, scale=0.05))],
    "experts": [layer(mlp=moe())],
    "experts-top1-plain": [layer(mlp=moe(experts=5, top=1, groups=None, shared=None))],
    "experts-all": [layer(mlp=moe(experts=4, top=4, groups=(2, 2), shared=8))],
    "experts-many": [layer(mlp=moe(experts=80, top=6, ff=16, groups=(8, 3), shared=40))],
    "experts-best-group": [layer(mlp=moe(experts=12, top=2, ff=32, groups=(4, 1), shared=None))],
}


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("name", sorted(ALONE))
def test_each_mechanism_alone(name, dt):
    """a 150-token prompt whole, then in portions with single tokens between them — the layer's output and the logits against the oracle"""
    cfg = config(ALONE[name])
    tensors = po.random_tensors(cfg, 7, dt == BF16)
    toks = tokens_of(cfg, 150, 3)
    ref, lay = po.forward(cfg, tensors, toks, True)
    eng = build(cfg, tensors, dt, blocks=8, max_model_len=256)
    eng.layer_trace(True)
    got = eng.replay_step([(1, toks, every(150))], [1])
    trace = eng.read_layer_trace(150)
    eng.layer_trace(False)
    agree(trace[0], lay[0], dt, "layer")
    agree(got, ref, dt, "whole")
    rows, at = [], 0
    for c in (1, 2, 60, 1, 1, 5, 64, 1, 15):
        rows.append(eng.replay_step([(2, toks[at:at + c], every(c))], [2] if at + c == 150 else []))
        at += c
    eng.close()
    assert at == 150
    agree(np.concatenate(rows), ref, dt, "portions")
    assert same(np.concatenate(rows), got, dt)


def test_layer_scale_soft_cap_and_embedding_scale_show():
    """a model whose scales and cap differ from 1 / none gives other logits than one without them, and the framework follows the oracle in both"""
    base = config([layer(mlp=moe())], scale=1.0, cap=None)
    tensors = po.random_tensors(base, 5)
    flat = dict(tensors, **{"l0.ls1": np.ones(96, np.float32), "l0.ls2": np.ones(96, np.float32)})
    toks = tokens_of(base, 20, 2)
    seen = []
    for cfg, t in ((base, flat), (base, tensors), (dict(base, logit_softcap=3.0), flat), (dict(base, embedding=dict(scale=0.05)), flat)):
        eng = build(cfg, t, F32, blocks=2, max_model_len=64)
        got = eng.replay_step([(1, toks, every(20))], [1])
        eng.close()
        agree(got, po.forward(cfg, t, toks), F32)
        seen.append(got)
    for other in seen[1:]:
        assert rel(other, seen[0]) > 0.05


def test_first_tokens_of_a_sequence():
    cfg = config([layer(mixer(size=2), mlp=moe()), layer(mixer(size=3))])
    tensors = po.random_tensors(cfg, 9)
    eng = build(cfg, tensors, F32, blocks=4, max_model_len=128)
    for toks in ([5], [5, 5], [7, 5], [5, 7, 5, 5]):
        ref = po.forward(cfg, tensors, toks)
        agree(eng.replay_step([(1, toks, every(len(toks)))], [1]), ref, F32, str(toks))
        one = np.stack([eng.replay_step([(2, toks[p:p + 1], [0])], [2] if p == len(toks) - 1 else [])[0] for p in range(len(toks))])
        agree(one, ref, F32, str(toks) + " token by token")
    eng.close()


@pytest.mark.parametrize("decode", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("size,dt", [(7, F32), (64, F32), (70, F32), (7, BF16), (64, BF16), (70, BF16), (1, F32)])
def test_window_edges(size, dt, decode):
    """a changed token reaches its own position and the size - 1 positions behind it and nothing beyond — exactly.  Portions cut inside windows;
    decoding past the window."""
    cfg = config([layer(mixer(size=size, heads=4))])
    tensors = po.random_tensors(cfg, 11)
    n = 3 * size + 5
    toks = tokens_of(cfg, n, 4)
    other = list(toks)
    at = size + size // 2
    other[at] = (toks[at] + 3) % cfg["vocab"]
    ref_a, ref_b = po.forward(cfg, tensors, toks), po.forward(cfg, tensors, other)
    eng = build(cfg, tensors, dt, blocks=8, max_model_len=320)

    def run(rid, t):
        if not decode:
            cuts = [c for c in (size - 2, 5, size, n - 2 * size - 3) if c > 0]
            cuts[-1] += n - sum(cuts)
            out, p = [], 0
            for i, c in enumerate(cuts):
                out.append(eng.replay_step([(rid, t[p:p + c], every(c))], [rid] if i == len(cuts) - 1 else []))
                p += c
            return np.concatenate(out)
        first = eng.replay_step([(rid, t[:3], every(3))], [])
        return np.concatenate([first] + [eng.replay_step([(rid, t[p:p + 1], [0])], [rid] if p == n - 1 else []) for p in range(3, n)])
    a, b = run(1, toks), run(2, other)
    eng.close()
    agree(a, ref_a, dt), agree(b, ref_b, dt)
    edge = at + size  # the first position that no longer sees the changed token
    changed = np.abs(a - b).max(-1)
    assert (changed[:at] == 0).all() and (changed[edge:] == 0).all() and (changed[at:edge] > 1e-6).all()
    assert (np.abs(ref_a - ref_b).max(-1)[at:edge] > 1e-6).all()


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
def test_a_far_key_among_hundreds(dt):
    """a token hundreds of positions back whose key answers the last token's query: one score stands out, so the last logits are mostly that
    token's value — whole prompt, decoding across page borders, 2-token portions; just outside the window it is not felt at all"""
    n, size = 640, 600
    cfg = config([layer(mixer(heads=2, dim=32, rot_dim=8, vdim=24, kv_rank=64, q_rank=48, size=size, scale=0.25))], scale=1.0, cap=None)
    tensors = po.random_tensors(cfg, 13)
    # the query of token 155 is the (plain) key of token 156: W_uq = k (x) c_q / |c_q|^2 with the normed latents of the two tokens
    p = "l0.mix."
    w = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
    h = po.layer_norm(w["embed"], w["l0.norm1"], cfg["norm"]["eps"])
    cq = po.rms_norm(h[155] @ w[p + "dq"].T, w[p + "dq.norm"], cfg["norm"]["eps"])
    key = (po.rms_norm((h[156] @ w[p + "dkv"].T)[:64], w[p + "dkv.norm"], cfg["norm"]["eps"]) @ w[p + "uk"].T).reshape(2, 32)
    uq = np.zeros((2, 40, 48))
    uq[:, :32] = key[:, :, None] * cq / (cq @ cq)
    tensors[p + "uq"] = po.bf16_round(uq.reshape(80, 48).astype(np.float32))
    r = np.random.default_rng(1)
    toks = [int(t) for t in r.integers(0, 150, n)]
    toks[n - 1] = 155
    for back, felt in ((size - 1, True), (size, False), (300, True)):
        a, b = list(toks), list(toks)
        a[n - 1 - back], b[n - 1 - back] = 156, 157
        ra, rb = po.forward(cfg, tensors, a)[-1], po.forward(cfg, tensors, b)[-1]
        gap = rel(ra, rb)
        assert (gap > 0.05) if felt else (gap < 1e-12)
        eng = build(cfg, tensors, dt, blocks=24, max_model_len=704)
        whole = eng.replay_step([(1, a, [n - 1])], [1])[0]
        eng.replay_step([(2, a[:40], [])], [])
        for q in range(40, n - 1):
            eng.replay_step([(2, a[q:q + 1], [])], [])
        dec = eng.replay_step([(2, a[n - 1:], [0])], [2])[0]
        for q in range(0, n - 2, 2):
            eng.replay_step([(3, a[q:q + 2], [])], [])
        por = eng.replay_step([(3, a[n - 2:], [1])], [3])[0]
        eng.close()
        for got in (whole, dec, por):
            assert rel(got, ra) < (1e-4 if dt == F32 else 3e-2)
            if felt:
                assert rel(got, rb) > gap / 2


# ------------------------------------------------------------------------------------------------ whole models
@pytest.fixture(scope="module", params=[("a", F32), ("a", BF16), ("b", F32), ("b", BF16)], ids=["a-f32", "a-bf16", "b-f32", "b-bf16"])
def model(request):
    name, dt = request.param
    cfg = config_a() if name == "a" else config_b()
    tensors = po.random_tensors(cfg, 17 if name == "a" else 18, dt == BF16)
    eng = build(cfg, tensors, dt, blocks=12, max_model_len=512)
    yield cfg, tensors, dt, eng
    eng.close()


def test_layers_one_by_one(model):
    cfg, tensors, dt, eng = model
    toks = tokens_of(cfg, 90, 1)
    eng.layer_trace(True)
    got = eng.replay_step([(1, toks, every(90))], [1])
    trace = eng.read_layer_trace(90)
    eng.layer_trace(False)
    ref, layers = po.forward(cfg, tensors, toks, True)
    for i, x in enumerate(layers):
        agree(trace[i], x, dt, f"layer {i}")
    agree(got, ref, dt)


def test_prefill_against_token_by_token_decoding(model):
    cfg, tensors, dt, eng = model
    toks = tokens_of(cfg, 150, 2)
    ref = po.forward(cfg, tensors, toks)
    whole = eng.replay_step([(1, toks, every(150))], [1])
    agree(whole, ref, dt, "whole")
    one = np.stack([eng.replay_step([(2, toks[p:p + 1], [0])], [2] if p == 149 else [])[0] for p in range(150)])
    agree(one, ref, dt, "token by token")
    if dt == F32:
        assert same(one, whole, dt)


@pytest.mark.parametrize("sizes", [[2] * 30, [37, 3, 37, 2, 5], [64, 64, 2], [63, 2, 63, 2], [1, 5, 1, 1, 70, 1], [71, 9, 2, 70]])
def test_portions(model, sizes):
    """a prompt cut anywhere (down to two tokens, at and across page borders and window edges) gives the logits of the whole prompt"""
    cfg, tensors, dt, eng = model
    n = sum(sizes)
    toks = tokens_of(cfg, n, 3)
    whole = eng.replay_step([(1, toks, every(n))], [1])
    got, at = [], 0
    for i, c in enumerate(sizes):
        got.append(eng.replay_step([(2, toks[at:at + c], every(c))], [2] if i == len(sizes) - 1 else []))
        at += c
    got = np.concatenate(got)
    if dt == F32:
        assert same(got, whole, dt)
    agree(got, po.forward(cfg, tensors, toks), dt)


def test_unequal_batch_against_each_alone(model):
    cfg, tensors, dt, eng = model
    lens = [70, 3, 129, 1]
    prompts = [tokens_of(cfg, n, 10 + i) for i, n in enumerate(lens)]
    alone = [eng.replay_step([(1, p, every(len(p)))], [1]) for p in prompts]
    batch = eng.replay_step([(10 + i, p, every(len(p))) for i, p in enumerate(prompts)], [10, 11, 12, 13])
    agree(batch, np.concatenate(alone), dt, "batch")
    cut = [n // 2 for n in lens]
    first = eng.replay_step([(20 + i, p[:c], every(c)) for i, (p, c) in enumerate(zip(prompts, cut)) if c], [])
    second = eng.replay_step([(20 + i, p[c:], every(len(p) - c)) for i, (p, c) in enumerate(zip(prompts, cut))], [20, 21, 22, 23])
    a1 = a2 = 0
    for i, (p, c) in enumerate(zip(prompts, cut)):
        got = np.concatenate([first[a1:a1 + c], second[a2:a2 + len(p) - c]])
        a1, a2 = a1 + c, a2 + len(p) - c
        agree(got, alone[i], dt, f"request {i}")


def test_mixed_steps_with_reused_pages(model):
    """12 pages for 8 requests that come and go: decoded tokens beside portions of prompts, a finished request's pages taken by the next one at
    once; every logit row equals the request's own run"""
    cfg, tensors, dt, eng = model
    r = np.random.default_rng(4)
    lens = [130, 60, 200, 90, 33, 150, 64, 128]
    prompts = [tokens_of(cfg, n, 40 + i) for i, n in enumerate(lens)]
    ref = [po.forward(cfg, tensors, p) for p in prompts]
    waiting, live = list(range(len(prompts))), {}
    got_rows, ref_rows = [], []
    while waiting or live:
        while waiting and len(live) < 4 and sum((lens[i] + 63) // 64 for i in list(live) + [waiting[0]]) <= 12:
            live[waiting.pop(0)] = 0
        entries, ends, spans = [], [], []
        for i, at in live.items():
            if at and r.random() < 0.2 and len(live) > 1:
                continue  # (left out of a step)
            left = lens[i] - at
            c = 1 if (at > 0 and r.random() < 0.5) else int(min(left, r.choice([2, 3, 17, 64, 100])))
            entries.append((1000 + i, prompts[i][at:at + c], every(c)))
            spans.append((i, at, c))
            if at + c == lens[i]:
                ends.append(1000 + i)
        if not entries:
            continue
        out = eng.replay_step(entries, ends)
        o = 0
        for i, at, c in spans:
            got_rows.append(out[o:o + c]), ref_rows.append(ref[i][at:at + c])
            o += c
            live[i] = at + c
            if live[i] == lens[i]:
                del live[i]
    agree(np.concatenate(got_rows), np.concatenate(ref_rows), dt)


def test_long_decoding(model):
    """310 decoded tokens behind a 20-token prompt: window edges and page borders pass under decoded tokens"""
    cfg, tensors, dt, eng = model
    toks = tokens_of(cfg, 330, 5)
    ref = po.forward(cfg, tensors, toks)
    eng.replay_step([(1, toks[:20], [])], [])
    rows = [eng.replay_step([(1, toks[p:p + 1], [0])], [1] if p == len(toks) - 1 else [])[0] for p in range(20, len(toks))]
    agree(np.stack(rows), ref[20:], dt)


def test_long_prompt_in_one_step_and_in_portions():
    """a 1500-token prompt with 16 heads (bf16 prompt steps of this size take the eight-wave attention and the large matrix tiles), whole and in
    three portions; logits also just inside and just outside the window of the first portion's last token"""
    cfg = config([layer(mixer(heads=16, dim=32, rot_dim=16, vdim=32, kv_rank=128, q_rank=96, size=192, scale=0.12), mlp=moe(experts=8, top=2, ff=48, groups=(4, 2), shared=64)),
                  layer(mixer(heads=2, kv_rank=80, size=500))], width=128)
    tensors = po.random_tensors(cfg, 23, True)
    toks = tokens_of(cfg, 1500, 8)
    want = sorted(set(list(range(0, 1500, 47)) + [191, 192, 193, 499, 500, 501, 699, 700, 890, 891, 1499]))
    ref = po.forward(cfg, tensors, toks)[want]
    for dt in (F32, BF16):
        eng = build(cfg, tensors, dt, blocks=48, max_model_len=1536)
        whole = eng.replay_step([(1, toks, want)], [1])
        agree(whole, ref, dt, "whole")
        parts, at = [], 0
        for c in (700, 40, 760):
            parts.append(eng.replay_step([(2, toks[at:at + c], [w - at for w in want if at <= w < at + c])], [2] if at + c == 1500 else []))
            at += c
        eng.close()
        parts = np.concatenate(parts)
        agree(parts, ref, dt, "portions")
        if dt == F32:
            assert same(parts, whole, dt)


@pytest.mark.parametrize("use_graph", [False, True], ids=["eager", "graphs"])
@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
def test_greedy_generation_through_the_scheduler(use_graph, dt):
    """Engine.generate: the engine's own scheduler, block manager, prefill and decode steps (captured decode graphs when asked) and its argmax —
    against the oracle's greedy continuation; five requests of unequal length for four places, the fifth on used pages"""
    cfg = config_a()
    tensors = po.random_tensors(cfg, 19, dt == BF16)
    eng = build(cfg, tensors, dt, blocks=16, max_model_len=256, use_graph=use_graph)
    prompts = [tokens_of(cfg, n, 60 + n) for n in (5, 70, 31, 64, 120)]
    outs = eng.generate(prompts, max_tokens=12, ignore_eos=True)
    again = eng.generate(prompts[:2], max_tokens=12, ignore_eos=True)  # (used pages, replayed graphs)
    eng.close()
    close = 1e-3 if dt == F32 else 0.35
    turned = 0
    for p, out in zip(prompts + prompts[:2], outs + again):
        assert len(out) == 12
        seq = list(p)
        for t in out:
            lg = po.forward(cfg, tensors, seq)[-1]
            turned += not (int(t) == int(lg.argmax()) or lg.max() - lg[int(t)] < close)
            seq.append(int(t))
    assert turned == 0 if dt == F32 else turned <= 6  # (bf16: a router's close call may turn a token)


def test_sampled_generation_stays_inside_the_top_k():
    cfg = config_a()
    tensors = po.random_tensors(cfg, 21)
    eng = build(cfg, tensors, F32, blocks=16, max_model_len=256)
    prompts = [tokens_of(cfg, n, 80 + n) for n in (9, 40)]
    outs = eng.generate(prompts, max_tokens=8, ignore_eos=True, sampling=dict(temperature=0.9, top_k=3, top_p=1.0))
    eng.close()
    for p, out in zip(prompts, outs):
        seq = list(p)
        assert len(out) == 8
        for t in out:
            lg = po.forward(cfg, tensors, seq)[-1]
            assert lg[int(t)] >= np.sort(lg)[-3] - 1e-3, (len(p), len(seq))
            seq.append(int(t))


def test_prefix_cache_reuses_latent_rows():
    """the design keeps nothing but cache rows, so the engine's prefix cache may serve it: a second request with the same long prefix"""
    cfg = config([layer(mixer(size=90), mlp=moe()), layer(mixer(size=500))])
    tensors = po.random_tensors(cfg, 27)
    eng = build(cfg, tensors, F32, blocks=24, max_model_len=512, enable_prefix_cache=True)
    common = tokens_of(cfg, 200, 1)
    prompts = [common + tokens_of(cfg, n, 2 + n) for n in (7, 40)]
    outs = [eng.generate([p], max_tokens=6, ignore_eos=True)[0] for p in prompts + prompts[:1]]
    eng.close()
    for p, out in zip(prompts + prompts[:1], outs):
        seq = list(p)
        for t in out:
            lg = po.forward(cfg, tensors, seq)[-1]
            assert lg.max() - lg[int(t)] < 1e-3
            seq.append(int(t))


def test_synthetic_weights_and_cache_plan():
    from vllm_rs_amd.engine import Engine
    cfg = checkpoint.parse_config(config_a())
    eng = Engine(cfg, max_num_seqs=4, max_model_len=256, kv_fraction=0.01, use_graph=False).init_synthetic()
    assert eng.num_gpu_blocks > 16
    out = eng.generate([list(range(1, 40)), list(range(3, 9))], max_tokens=5, ignore_eos=True)
    assert [len(o) for o in out] == [5, 5]
    eng.close()


def test_trace_runner_on_a_model_folder(tmp_path):
    """bin/trace_run as a user starts it: config.json + model.safetensors in a folder, steps on standard input (a prompt in portions beside
    another request's single tokens; a pool of three pages used again), logits files out — against the oracle"""
    cfg = config_a()
    tensors = po.random_tensors(cfg, 31, True)
    model_dir = tmp_path / "model"
    model_dir.mkdir()
    (model_dir / "config.json").write_text(json.dumps(cfg))
    header, blobs, off = {}, [], 0
    for name, a in tensors.items():
        b = checkpoint.f32_to_bf16_bits(np.asarray(a, np.float32)).tobytes()
        header[name] = dict(dtype="BF16", shape=list(np.shape(a)), data_offsets=[off, off + len(b)])
        off += len(b)
        blobs.append(b)
    h = json.dumps(header).encode()
    (model_dir / "model.safetensors").write_bytes(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    p1, p2, p3 = tokens_of(cfg, 100, 1), tokens_of(cfg, 40, 2), tokens_of(cfg, 64, 3)
    steps = [dict(entries=[dict(id="x", tokens=p1[:37], want=every(37)), dict(id="y", tokens=p2[:38], want=[])], end=[]),
             dict(entries=[dict(id="x", tokens=p1[37:99], want=every(62)), dict(id="y", tokens=p2[38:39], want=[0])], end=[]),
             dict(entries=[dict(id="y", tokens=p2[39:], want=[0])], end=["y"]),
             dict(entries=[dict(id="x", tokens=p1[99:], want=[0])], end=["x"]),
             dict(entries=[dict(id="z", tokens=p3, want=every(64))], end=["z"])]
    for i, s in enumerate(steps):
        s["step"] = i
    r1, r2, r3 = (po.forward(cfg, tensors, p) for p in (p1, p2, p3))
    want = [r1[:37], np.concatenate([r1[37:99], r2[38:39]]), r2[39:], r1[99:], r3]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    for dtype, dt in (("float32", F32), ("bfloat16", BF16)):
        out = tmp_path / ("out_" + dtype)
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(model_dir), "--dtype", dtype, "--out", str(out),
                            "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps).encode() + b"\n", capture_output=True, timeout=110)
        assert r.returncode == 0, r.stderr.decode()[-1500:]
        assert [ln for ln in r.stdout.decode().split("\n") if ln.startswith("done")] == ["done %d" % i for i in range(5)]
        got = [np.fromfile(out / ("%d.f32" % i), "<f4").reshape(-1, cfg["vocab"]) for i in range(5)]
        assert [g.shape[0] for g in got] == [w.shape[0] for w in want]
        agree(np.concatenate(got), np.concatenate(want), dt, dtype)
