"""GPU tests of the Kemavik design in the layer-stack model class: every operator alone with planted values, every mechanism as a one-layer
model, then whole models of small random configurations through the engine — against tests/kemavik_oracle.py (float64, whole sequences, no
cache, no pages, the recurrence token by token).

f32 models must agree with the oracle to f32 rounding, bf16 models to bf16 rounding; and the logits of a position must not depend on how
its prompt was cut, on the rest of the batch or on the pages and state slots it got.
"""
import json
import math
import os
import struct
import subprocess
import sys

import numpy as np
import pytest

from tests import kemavik_oracle as ko
from tests.test_gpu_stack import BF16, F32, build, check, empty, from_dev, raw, rel, to_dev, tokens_of
from tests.test_gpu_stack import _buffers_live_until_the_test_ends  # noqa: F401  (autouse: device buffers outlive the launches)
from vllm_rs_amd import _lib, checkpoint

pytestmark = pytest.mark.gpu

f32 = lambda a: raw(a, np.float32)


def attn(heads=6, kv_heads=3, dim=16, vdim=32, scale=0.3, diff=0.35, kv_from=None, **kw):
    mx = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, diff=diff)
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return dict(type="attention", mixer=mx, mlp=None, **kw)


def wkv(heads=3, dim=24):
    return dict(type="wkv", mixer=dict(heads=heads, dim=dim), mlp=None)


def dense(ff=88):
    return dict(kind="dense", ff=ff)


def moe(experts=6, top=2, ff=40, identity=3, scale=1.7, shared=24):
    m = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if identity:
        m["router"]["identity"] = identity
    if scale is not None:
        m["router"]["scale"] = scale
    if shared:
        m["shared"] = dict(ff=shared)
    return m


def config(layers, width=96, vocab=160, eps=3e-5):
    return dict(architecture="Kemavik", width=width, vocab=vocab, norm=dict(eps=eps), layers=layers)


def config_a():
    """sizes on the matrix-core paths: head counts 6:3, 4:1 and 2:2, two layers that borrow the keys of two others, time mixing between them and
    twice in a row, every form of the feed-forward (none, dense, mixture with and without identity experts, scale and shared expert)"""
    return config([
        dict(attn(), mlp=moe()),
        dict(wkv(), mlp=dense()),
        dict(attn(heads=4, kv_heads=1, dim=8, vdim=48, scale=0.5, diff=0.6), mlp=None),
        dict(attn(scale=0.2, diff=0.1, kv_from=0), mlp=moe(experts=5, top=1, ff=24, identity=0, scale=None, shared=None)),
        dict(wkv(heads=2, dim=40), mlp=moe(experts=8, top=3, ff=32, identity=1, scale=0.8)),
        dict(wkv(heads=1, dim=64), mlp=None),
        dict(attn(heads=4, kv_heads=1, dim=8, vdim=48, scale=0.7, diff=0.25, kv_from=2), mlp=dense(40)),
        dict(attn(heads=2, kv_heads=2, dim=32, vdim=16), mlp=moe(identity=2, shared=56)),
    ])


def config_b():
    """sizes off every 16-byte path: width 50, heads of 5 / 7 / 9 channels, odd feed-forwards, every expert chosen"""
    return config([
        dict(wkv(heads=3, dim=7), mlp=dense(13)),
        dict(attn(heads=4, kv_heads=2, dim=5, vdim=9, scale=0.6), mlp=moe(experts=3, top=4, ff=11, identity=1, scale=1.3, shared=13)),
        dict(attn(heads=4, kv_heads=2, dim=5, vdim=9, scale=0.9, diff=0.0, kv_from=1), mlp=None),
        dict(wkv(heads=5, dim=9), mlp=moe(experts=4, top=2, ff=9, identity=0, scale=2.1, shared=None)),
    ], width=50, vocab=70, eps=1e-6)


def agree(got, ref, dt, what=""):
    """rows against the oracle's.  f32: every row to f32 rounding.  bf16: a close call of a router (a discrete choice) may turn a token, so the
    rows are judged one by one: the typical row to bf16 rounding, three in four within a few times that"""
    got, ref = np.asarray(got, np.float64), np.asarray(ref, np.float64)
    got, ref = got.reshape(-1, got.shape[-1]), ref.reshape(-1, ref.shape[-1])
    rows = np.sqrt(((got - ref) ** 2).mean(-1)) / np.maximum(np.sqrt((ref ** 2).mean(-1)), 1e-30)
    if dt == F32:
        assert rows.max() < 2e-4 and rel(got, ref) < 3e-5, (what, rows.max(), rel(got, ref))
    else:
        assert np.median(rows) < 3e-2 and np.quantile(rows, 0.75) < 6e-2, (what, float(np.median(rows)), float(np.quantile(rows, 0.75)))


def same(a, b, dt):
    """the same rows computed in two ways"""
    return rel(a, b) < (1e-5 if dt == F32 else 3e-2)


def every(n):
    return list(range(n))


# ------------------------------------------------------------------------------------------------ operators alone
def paged(rows, BS, table, nb, dt):
    """rows of ONE sequence over shuffled pages; every other slot holds large values that nobody may read"""
    pool = np.full((nb * BS, rows.shape[1]), 1e4, np.float32)
    for j in range(rows.shape[0]):
        pool[int(table[j // BS]) * BS + j % BS] = rows[j]
    return to_dev(pool, dt)


def run_differential(L, q, positions, k, v, scale, lam, diff, eps, dt, form, r, BS=64, splits=3):
    """q [Tq, H, 2, D], k [Tk, G, 2, D], v [Tk, G, V]; form: "prompt" (one step), "decoded" (a batch of sequences that share their pages),
    "parts" (the same, the key range in parts)"""
    Tq, H, _, D = q.shape
    Tk, G, V = v.shape
    nb = (Tk + BS - 1) // BS + 3
    table = r.permutation(nb)[:nb - 3].astype(np.uint32)
    kc, vc = paged(k.reshape(Tk, -1), BS, table, nb, dt), paged(v.reshape(Tk, -1), BS, table, nb, dt)
    out = empty(Tq * H * V * 4)
    qd, pos = to_dev(q.reshape(Tq, -1), dt), raw(positions, np.int64)
    args = (qd.ptr, H * 2 * D, out.ptr, kc.ptr, vc.ptr, pos.ptr)
    tail = (H, G, D, V, BS, len(table), scale, lam, eps, 1.0 - diff)
    if form == "prompt":
        L.vra_stack_op_attention_differential(*args, raw(table, np.uint32).ptr, raw([Tk], np.uint32).ptr, raw([0, Tq], np.uint32).ptr, 1, Tq, Tq, *tail, None, 0, 0, dt, 0)
    else:
        n = Tq * splits * H * 2 * (V + 2) * 4
        scratch = empty(n)
        L.vra_stack_op_attention_differential(*args, raw(np.tile(table, (Tq, 1)), np.uint32).ptr, raw(np.asarray(positions) + 1, np.uint32).ptr, None, Tq, Tq, 1, *tail,
                                              scratch.ptr if form == "parts" else None, n, splits, dt, 0)
    check()
    return from_dev(out, (Tq, H, V), dt)


def differential_reference(q, positions, k, v, scale, lam, diff, eps):
    """every query alone on the keys up to its position (the oracle's own function, one query at a time)"""
    k, v = k.astype(np.float64), v.astype(np.float64)
    return np.concatenate([ko.differential_heads(q[i:i + 1].astype(np.float64), k[:p + 1], v[:p + 1], scale, lam, diff, eps) for i, p in enumerate(positions)])


FORMS = [("prompt", F32), ("prompt", BF16), ("decoded", F32), ("decoded", BF16), ("parts", F32), ("parts", BF16)]


@pytest.mark.parametrize("form,dt", FORMS)
@pytest.mark.parametrize("H,G,D,V", [(6, 3, 16, 32), (4, 1, 8, 16), (2, 2, 64, 64), (4, 2, 64, 128), (3, 3, 40, 112), (2, 1, 128, 128), (2, 1, 128, 256), (2, 1, 160, 192), (4, 2, 5, 9), (2, 2, 24, 20),
                                     (1, 1, 32, 304)])
def test_differential_attention_against_the_oracle(form, dt, H, G, D, V):
    """every matrix-core instantiation and sizes off its paths, grouped heads, 200 keys over shuffled pages; the two maps' scores unlike each other"""
    L = _lib.load()
    r = np.random.default_rng(H * 1000 + D + V)
    Tk = 200
    q = ko.bf16_round(r.standard_normal((90, H, 2, D)).astype(np.float32))
    k = ko.bf16_round(r.standard_normal((Tk, G, 2, D)).astype(np.float32))
    v = ko.bf16_round(r.standard_normal((Tk, G, V)).astype(np.float32))
    positions = np.arange(110, 200, dtype=np.int64)
    scale = 1.5 / math.sqrt(D)
    for lam, diff in ((0.37, 0.2), (1.4, 0.7)):
        got = run_differential(L, q, positions, k, v, scale, lam, diff, 1e-5, dt, form, r)
        ref = differential_reference(q, positions, k, v, scale, lam, diff, 1e-5)
        assert rel(got, ref) < (3e-6 if dt == F32 else 6e-3), (lam, rel(got, ref))


@pytest.mark.parametrize("form,dt", FORMS)
@pytest.mark.parametrize("D,V", [(64, 128), (16, 16), (6, 10)])
def test_planted_keys_in_either_map(form, dt, D, V):
    """in 900 keys one stands out for the first map and another for the second: the head returns marker 1 - lambda * marker 2, at the first
    token, around page borders, far back, at the query's own position; a key one position after the query is not felt although it lies in
    the cache"""
    L = _lib.load()
    r = np.random.default_rng(D)
    Tk, H, G, lam, diff, eps = 900, 4, 2, 0.6, 0.3, 1e-5
    base_k = ko.bf16_round((0.1 * r.standard_normal((Tk, G, 2, D))).astype(np.float32))
    base_v = ko.bf16_round((0.1 * r.standard_normal((Tk, G, V))).astype(np.float32))
    u = np.zeros(D, np.float32)
    u[3] = 1.0
    m1, m2 = ko.bf16_round(2.0 + r.random(V).astype(np.float32)), ko.bf16_round(-1.0 - 3.0 * r.random(V).astype(np.float32))
    for j1, j2 in ((0, 899), (63, 64), (64, 63), (400, 0), (898, 700), (127, 895)):
        k, v = base_k.copy(), base_v.copy()
        k[j1, :, 0], k[j2, :, 1] = 16.0 * u, 16.0 * u  # score 8 * 16 * 0.25 = 32 against |scores| < 1 elsewhere
        v[j1], v[j2] = m1, m2
        positions = sorted({p for p in (j1 - 1, j1, j1 + 1, j2 - 1, j2, j2 + 1, 899) if 0 <= p < Tk})
        q = np.tile(8.0 * u, (len(positions), H, 2, 1)).astype(np.float32)
        got = run_differential(L, q, positions, k, v, 0.25, lam, diff, eps, dt, form, r)
        assert rel(got, differential_reference(q, positions, k, v, 0.25, lam, diff, eps)) < (2e-5 if dt == F32 else 1e-2), (j1, j2)
        for i, p in enumerate(positions):
            if p >= max(j1, j2):  # both felt: the markers alone
                o = m1.astype(np.float64) - lam * m2
                o = o / math.sqrt((o * o).mean() + eps) * (1 - diff)
                assert np.abs(got[i] - o).max() < 2e-2, (j1, j2, p)


def test_prompt_rows_do_not_depend_on_their_neighbours():
    """bf16 prompt attention: a row is the same to the last bit in a step of its own, in a long step and behind another sequence"""
    L = _lib.load()
    r = np.random.default_rng(5)
    H, G, D, V, Tk, BS = 4, 2, 64, 128, 300, 64
    k = r.standard_normal((Tk, G, 2, D)).astype(np.float32)
    v = r.standard_normal((Tk, G, V)).astype(np.float32)
    q = r.standard_normal((Tk, H, 2, D)).astype(np.float32)
    whole = run_differential(L, q, np.arange(Tk), k, v, 0.2, 0.5, 0.3, 1e-5, BF16, "prompt", r)
    for a, b in ((299, 300), (130, 195), (63, 65), (0, 2)):
        part = run_differential(L, q[a:b], np.arange(a, b), k, v, 0.2, 0.5, 0.3, 1e-5, BF16, "prompt", r)
        assert (part == whole[a:b]).all(), (a, b)


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("W,n", [(96, 5), (51, 5), (1032, 2), (4, 1)])
def test_token_shift(dt, W, n):
    """mixes of a row with the one before it: three sequences in one step (one that starts, one that goes on, one of a single row that goes on),
    then their next rows in the decode form; a slot that held something else is not felt by a sequence that starts; a padded lane (slot -1)
    touches nothing"""
    L = _lib.load()
    r = np.random.default_rng(W)
    mu = r.random((n, W)).astype(np.float32)
    before = r.standard_normal((4, W)).astype(np.float32)
    state = f32(before)
    lens, starts, slots = [4, 3, 1], [0, 7, 12], [2, 0, 3]
    x = r.standard_normal((8, W)).astype(np.float32)
    pos = np.concatenate([np.arange(s, s + c) for s, c in zip(starts, lens)])
    out = empty(n * 8 * W * 4)
    L.vra_stack_op_token_shift(f32(x).ptr, f32(mu).ptr, n, state.ptr, raw(pos, np.int64).ptr, raw([0, 4, 7, 8], np.uint32).ptr, raw(slots, np.int32).ptr, out.ptr, 8, 3, W, dt, 0)
    check()
    got = from_dev(out, (n, 8, W), dt)
    seqs = [x[:4], np.concatenate([before[0:1], x[4:7]]), np.concatenate([before[3:4], x[7:8]])]
    skip = [0, 1, 1]
    x64 = [s.astype(np.float64) for s in seqs]
    tol = 1e-6 if dt == F32 else 2e-2
    for m in range(n):
        ref = np.concatenate([(s + (ko.shifted(s) - s) * mu[m])[k:] for s, k in zip(x64, skip)])
        assert np.abs(got[m] - ref).max() < tol, m
    st = state.numpy(np.float32, (4, W))
    assert (st[[2, 0, 3]] == x[[3, 6, 7]]).all() and (st[1] == before[1]).all()
    y = r.standard_normal((4, W)).astype(np.float32)
    out = empty(n * 4 * W * 4)
    L.vra_stack_op_token_shift(f32(y).ptr, f32(mu).ptr, n, state.ptr, raw([4, 10, 13, 0], np.int64).ptr, None, raw([2, 0, 3, -1], np.int32).ptr, out.ptr, 4, 4, W, dt, 0)
    check()
    got = from_dev(out, (n, 4, W), dt)
    prev = x[[3, 6, 7]].astype(np.float64)
    for m in range(n):
        assert np.abs(got[m, :3] - (y[:3] + (prev - y[:3]) * mu[m])).max() < tol
    st = state.numpy(np.float32, (4, W))
    assert (st[[2, 0, 3]] == y[:3]).all() and (st[1] == before[1]).all()


@pytest.mark.parametrize("H,rep,D,V", [(2, 1, 8, 8), (3, 1, 5, 7), (4, 2, 16, 24), (2, 1, 48, 48), (2, 2, 128, 128), (1, 1, 200, 9), (2, 1, 24, 300), (1, 1, 256, 64)])
def test_bonus_recurrence(H, rep, D, V):
    """the recurrence whose output reads the state before the token's decay, with the token itself through the bonus: every lane grouping, value
    sizes off the workgroup's column count, grouped q / k heads; whole, in portions down to one token and in the decode form, with the
    state waiting in a slot that held other values; the bonus enters only its own token"""
    L = _lib.load()
    r = np.random.default_rng(D * 7 + V)
    T = 75
    q = r.standard_normal((T, H // rep, D)).astype(np.float32)
    k = (r.standard_normal((T, H // rep, D)) / math.sqrt(D)).astype(np.float32)
    v = r.standard_normal((T, H, V)).astype(np.float32)
    decay = np.exp(-np.exp(-3.0 + 2.0 * r.standard_normal((T, H, D)))).astype(np.float32)
    u = (0.5 + r.standard_normal((H, D))).astype(np.float32)
    rp = lambda a: np.repeat(a.astype(np.float64), rep, 1)
    ref, end = ko.wkv(0.5 * rp(q), rp(k), v.astype(np.float64), decay.astype(np.float64), u.astype(np.float64))
    state = raw(r.standard_normal(3 * H * V * D).astype(np.float32) * 100.0, np.float32)
    bonus = f32(u)

    def run(cuts, slot):
        outs, at = [], 0
        for c in cuts:
            sl = slice(at, at + c)
            out = empty(c * H * V * 4)
            d = lambda a: f32(np.ascontiguousarray(a[sl].reshape(c, -1))).ptr
            L.vra_stack_op_bonus_scan(d(q), H // rep * D, d(k), H // rep * D, d(v), H * V, d(decay), H * D, bonus.ptr, 0.5, state.ptr, raw([slot], np.int32).ptr,
                                      raw(np.arange(at, at + c), np.int64).ptr, raw([0, c], np.uint32).ptr if c > 1 or at == 0 else None, out.ptr, H * V, 1, H, rep, D, V, 0)
            check()
            outs.append(out.numpy(np.float32, (c, H, V)))
            at += c
        return np.concatenate(outs)
    whole = run([T], 1)
    assert rel(whole, ref) < 1e-5
    st = state.numpy(np.float32, (3, H, V, D))[1]
    assert rel(st, end.transpose(0, 2, 1)) < 1e-5
    parts = run([1, 1, 2, 16, 1, 17, 32, 1, 4], 2)
    assert rel(parts, ref) < 1e-5 and np.abs(parts - whole).max() <= 1e-6 * np.abs(whole).max()
    assert rel(run([40, 35], 1), ref) < 1e-5  # the slot of the first run, used again
    u[:] = 0.0
    bonus = f32(u)  # without the bonus a sequence's first output is zero: the state before it is empty
    assert (run([3], 0)[0] == 0.0).all()


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("H,V", [(3, 24), (1, 50), (5, 7), (16, 128)])
def test_head_norm_with_a_weight_per_head(dt, H, V):
    L = _lib.load()
    r = np.random.default_rng(H)
    T = 9
    o, g, w = (r.standard_normal(s).astype(np.float32) for s in ((T, H, V), (T, H * V), (H * V,)))
    o[4] *= 1e-4  # (eps shows)
    out = empty(T * H * V * 4)
    L.vra_stack_op_head_norm_gate(f32(o).ptr, f32(w).ptr, 1, f32(g).ptr, H * V, 1, 1e-5, out.ptr, T, H, V, dt, 0)
    check()
    ref = ko.unit_rms(o.astype(np.float64), 1e-5).reshape(T, -1) * w * ko.silu(g.astype(np.float64))
    assert rel(from_dev(out, (T, H * V), dt), ref) < (2e-6 if dt == F32 else 4e-3)


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("T,W,E,ident,top,scale", [(9, 96, 6, 3, 3, 1.5), (3, 51, 5, 0, 5, 1.0), (200, 256, 32, 4, 4, 0.7), (5, 128, 72, 8, 3, 2.5), (1, 2048, 16, 4, 2, 1.5),
                                                   (150, 1032, 20, 1, 3, 1.0), (300, 1028, 9, 2, 2, 3.0), (2, 4100, 9, 2, 1, 0.5)])
def test_seam_of_blocks_that_read_the_residual_stream(dt, T, W, E, ident, top, scale):
    """x += RMS(sum_j w_j part_j + shared part + (identity weight) x) (1 + w) with rows left out for identity picks; h = x itself; the router on x:
    softmax over all outputs, corrected choice, weights = scores times the constant, identity picks as -1 with their weights summed"""
    L = _lib.load()
    r = np.random.default_rng(W + E)
    eps, n1 = 1e-5, 2
    f = lambda *s: r.standard_normal(s).astype(np.float32)
    x, p1, p2, pw, xw = f(T, W), 2.0 * f(T * n1, W), f(T, W), r.random(T * n1).astype(np.float32), r.random(T).astype(np.float32)
    pe_in = np.where(r.random(T * n1) < 0.3, -1, 1).astype(np.int32)
    p1[pe_in < 0] = np.nan  # (rows of identity picks are never written: nobody may read them)
    post = 1 + 0.2 * f(W)
    rw = ko.bf16_round(2.0 * f(E + ident, W) / math.sqrt(W))
    corr = (0.2 * f(E + ident)).astype(np.float32)
    parts = np.where(pe_in[:, None] < 0, 0.0, pw[:, None].astype(np.float64) * np.nan_to_num(p1)).reshape(T, n1, W).sum(1)
    s = parts + p2 + xw[:, None].astype(np.float64) * x
    x_ref = x + ko.unit_rms(s, eps) * post
    chosen, wt = ko.route(x_ref, dict(top=top, scale=scale), {"router": rw.astype(np.float64), "correction": corr.astype(np.float64)}, "")
    d = lambda a: f32(a).ptr
    xd, hd = f32(x), empty(T * W * 4)
    pe, pwt, idw = empty(T * top * 4), empty(T * top * 4), empty(T * 4)
    L.vra_stack_op_seam_post(xd.ptr, d(p1), n1, d(pw), raw(pe_in, np.int32).ptr, d(p2), d(xw), d(post), hd.ptr, eps, T, W, to_dev(rw, dt).ptr, d(corr), E + ident, top, ident,
                             scale, pe.ptr, pwt.ptr, idw.ptr if ident else None, dt, 0)
    check()
    assert rel(xd.numpy(np.float32, (T, W)), x_ref) < 2e-6
    assert rel(from_dev(hd, (T, W), dt), x_ref) < (2e-6 if dt == F32 else 4e-3)
    experts, weights = pe.numpy(np.int32, (T, top)), pwt.numpy(np.float32, (T, top))
    close = 0
    for t in range(T):
        ref = [(-1 if e >= E else int(e), float(w)) for e, w in zip(chosen[t], wt[t])]
        got = list(zip(experts[t].tolist(), weights[t].tolist()))
        ok = sorted(e for e, _ in ref) == sorted(e for e, _ in got) and np.allclose(sorted(w for _, w in ref), sorted(w for _, w in got), rtol=2e-4, atol=1e-7)
        close += not ok
        if ok and ident:
            assert abs(idw.numpy(np.float32, (T,))[t] - sum(w for e, w in ref if e < 0)) < 1e-4
    assert close <= T // 100  # (a close call of two choice scores in f32)
    # without parts and router: h is x as it stands
    hd2 = empty(T * W * 4)
    L.vra_stack_op_seam_post(xd.ptr, None, 1, None, None, None, None, None, hd2.ptr, eps, T, W, None, None, 0, 0, 0, 1.0, None, None, None, dt, 0)
    check()
    assert (from_dev(hd2, (T, W), dt) == from_dev(hd, (T, W), dt)).all()


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("M,N,K", [(3, 40, 96), (70, 136, 64), (1100, 2064, 96), (20, 33, 51), (300, 64, 1024), (130, 48, 2056)])
def test_element_wise_epilogues(dt, M, N, K):
    """squared relu, tanh and exp(-exp) behind a product with a bias, in every matrix kernel (the last two shapes: few columns over a long K)"""
    L = _lib.load()
    r = np.random.default_rng(N)
    a, w = ko.bf16_round(r.standard_normal((M, K)).astype(np.float32)), ko.bf16_round((r.standard_normal((N, K)) / math.sqrt(K)).astype(np.float32))
    b = r.standard_normal(N).astype(np.float32)
    z = a.astype(np.float64) @ w.T.astype(np.float64) + b
    for act, fn in ((4, lambda t: np.maximum(t, 0) ** 2), (5, np.tanh), (6, lambda t: np.exp(-np.exp(t)))):
        out = empty(M * N * 4)
        L.vra_stack_op_gemm_post(to_dev(a, dt).ptr, K, to_dev(w, dt).ptr, 0, out.ptr, N, 1, M, N, K, 1.0, f32(b).ptr, None, 0, None, None, 2, act, 0.0, dt, 0)
        check()
        assert np.abs(out.numpy(np.float32, (M, N)) - fn(z)).max() < 4e-5 * max(1.0, np.abs(fn(z)).max()), act


# ------------------------------------------------------------------------------------------------ each mechanism alone
ALONE = {
    "attention": [attn()],
    "attention-plain-heads": [attn(heads=3, kv_heads=3, dim=32, vdim=16, diff=0.0)],
    "attention-one-group": [attn(heads=4, kv_heads=1, dim=64, vdim=128, scale=0.1)],
    "attention-wide": [attn(heads=2, kv_heads=1, dim=128, vdim=256, scale=0.08, diff=0.8)],
    "attention-odd": [attn(heads=4, kv_heads=2, dim=7, vdim=11)],
    "borrowed-keys": [attn(), attn(scale=0.5, diff=0.1, kv_from=0)],
    "borrowed-past-another": [attn(), attn(dim=8, heads=2, kv_heads=2), attn(kv_from=0), attn(dim=8, heads=2, kv_heads=2, kv_from=1)],
    "wkv": [wkv()],
    "wkv-one-head": [wkv(heads=1, dim=128)],
    "wkv-odd": [wkv(heads=5, dim=9)],
    "wkv-twice": [wkv(), wkv(heads=2, dim=16)],
    "dense": [dict(wkv(), mlp=dense(72))],
    "experts": [dict(wkv(), mlp=moe())],
    "experts-plain": [dict(wkv(), mlp=moe(experts=7, top=1, identity=0, scale=None, shared=None))],
    "experts-identity-only-scale": [dict(attn(), mlp=moe(experts=4, top=3, identity=6, scale=2.3, shared=None))],
    "experts-all-chosen": [dict(attn(), mlp=moe(experts=3, top=5, identity=2, ff=24))],
    "experts-many": [dict(wkv(), mlp=moe(experts=80, top=4, identity=7, ff=8))],
}


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("name", sorted(ALONE))
def test_each_mechanism_alone(name, dt):
    """one mechanism (no feed-forward unless it is the subject): a 150-token prompt whole, then in portions with single tokens between them"""
    cfg = config(ALONE[name])
    tensors = ko.random_tensors(cfg, 7, steady=dt == BF16)
    toks = tokens_of(cfg, 150, 3)
    ref, lay = ko.forward(cfg, tensors, toks, True)
    eng = build(cfg, tensors, dt, blocks=8, max_model_len=256)
    eng.layer_trace(True)
    got = eng.replay_step([(1, toks, every(150))], [1])
    trace = eng.read_layer_trace(150)
    eng.layer_trace(False)
    for i, x in enumerate(lay):
        agree(trace[i], x, dt, f"layer {i}")
    agree(got, ref, dt, "whole")
    rows, at = [], 0
    for c in (1, 2, 60, 1, 1, 5, 64, 1, 15):
        rows.append(eng.replay_step([(2, toks[at:at + c], every(c))], [2] if at + c == 150 else []))
        at += c
    eng.close()
    assert at == 150
    agree(np.concatenate(rows), ref, dt, "portions")
    if dt == F32:
        assert rel(np.concatenate(rows), got) < 1e-5


@pytest.mark.parametrize("rank", [1, 6, 17, 48])
def test_rank_of_the_decays_comes_from_the_tensors(rank):
    cfg = config([wkv()])
    tensors = ko.random_tensors(cfg, 29, rank=rank)
    toks = tokens_of(cfg, 70, 1)
    ref = ko.forward(cfg, tensors, toks)
    for dt in (F32, BF16):
        eng = build(cfg, tensors, dt, blocks=4, max_model_len=128)
        agree(eng.replay_step([(1, toks, every(70))], [1]), ref, dt)
        eng.close()


def test_first_tokens_of_a_sequence():
    """sequences of one, two and four tokens, whole and token by token, in slots other sequences left behind: nothing before the first token"""
    cfg = config([wkv(), attn(), wkv(heads=1, dim=16)])
    tensors = ko.random_tensors(cfg, 9)
    eng = build(cfg, tensors, F32, blocks=4, max_model_len=128)
    for toks in ([5], [5, 5], [7, 5], [5, 7, 5, 5]):
        ref = ko.forward(cfg, tensors, toks)
        agree(eng.replay_step([(1, toks, every(len(toks)))], [1]), ref, F32, str(toks))
        one = np.stack([eng.replay_step([(2, toks[p:p + 1], [0])], [2] if p == len(toks) - 1 else [])[0] for p in range(len(toks))])
        agree(one, ref, F32, str(toks) + " token by token")
    eng.close()


def three_ways(eng, toks):
    """the last token's logits: whole prompt; decoded across page borders; portions of two"""
    n = len(toks)
    whole = eng.replay_step([(1, toks, [n - 1])], [1])[0]
    eng.replay_step([(2, toks[:40], [])], [])
    for p in range(40, n - 1):
        eng.replay_step([(2, toks[p:p + 1], [])], [])
    dec = eng.replay_step([(2, toks[n - 1:], [0])], [2])[0]
    cut = n % 2
    if cut:
        eng.replay_step([(3, toks[:1], [])], [])
    for p in range(cut, n - 2, 2):
        eng.replay_step([(3, toks[p:p + 2], [])], [])
    por = eng.replay_step([(3, toks[n - 2:], [1])], [3])[0]
    return whole, dec, por


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("borrowed", [False, True], ids=["own", "borrowed"])
@pytest.mark.parametrize("map_", [0, 1])
def test_a_far_key_among_hundreds(map_, borrowed, dt):
    """a token hundreds of positions back whose key in one of the two maps answers the last token's query: one score stands out, and the last
    logits are mostly that token's value — with the layer's own keys or with those of the layer before it"""
    n, D, width = 640, 32, 96
    layers = [attn(heads=2, kv_heads=1, dim=D, vdim=64, scale=0.5, diff=0.2)]
    if borrowed:
        layers.append(attn(heads=2, kv_heads=1, dim=D, vdim=64, scale=0.5, diff=0.2, kv_from=0))
    cfg = config(layers, width=width)
    tensors = ko.random_tensors(cfg, 13)
    p = "l%d.mix." % (len(layers) - 1)
    w = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
    if borrowed:  # the first layer leaves the stream alone (its output norm weighs nothing), so that the second reads embeddings
        tensors["l0.norm1"] = np.full_like(tensors["l0.norm1"], -1.0)
    # the query of token 155 in map `map_` points along the key of token 156:  W_q = key (x) x / |x|^2, without a bias
    x155, x156 = w["embed"][155], w["embed"][156]
    key = ((w["l0.mix.k"] @ x156 + w["l0.mix.k.b"]).reshape(1, 2, D)[0, map_])
    key = key / math.sqrt((key * key).mean() + cfg["norm"]["eps"]) * w["l0.mix.k.norm"]
    wq = w[p + "q"].reshape(2, 2, D, width).copy()
    wq[:, map_] = np.outer(key, x155) / (x155 @ x155)
    qb = w[p + "q.b"].reshape(2, 2, D).copy()
    qb[:, map_] = 0.0
    tensors[p + "q"], tensors[p + "q.b"] = ko.bf16_round(wq.reshape(-1, width).astype(np.float32)), ko.bf16_round(qb.reshape(-1).astype(np.float32))
    tensors[p + "q.norm"] = np.full_like(tensors[p + "q.norm"], 2.0)
    r = np.random.default_rng(1)
    toks = [int(t) for t in r.integers(0, 150, n)]
    toks[n - 1] = 155
    eng = build(cfg, tensors, dt, blocks=24, max_model_len=704)
    for back in (639, 300, 65, 64, 1):
        a, b = list(toks), list(toks)
        a[n - 1 - back], b[n - 1 - back] = 156, 157
        ra, rb = ko.forward(cfg, tensors, a)[-1], ko.forward(cfg, tensors, b)[-1]
        gap = rel(ra, rb)
        assert gap > 0.1, back
        for got in three_ways(eng, a) if back in (639, 64) else (eng.replay_step([(1, a, [n - 1])], [1])[0],):
            assert rel(got, ra) < (1e-4 if dt == F32 else 3e-2) and rel(got, rb) > gap / 2, back
    eng.close()


@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
def test_a_far_token_stays_in_the_state(dt):
    """a token hundreds of positions back reaches the last logits only through the matrix state (slow decays, small embeddings elsewhere)"""
    cfg = config([wkv(heads=2, dim=16)])
    tensors = ko.random_tensors(cfg, 13)
    tensors["l0.mix.w0"] = ko.bf16_round(np.full_like(tensors["l0.mix.w0"], -9.0))
    tensors["l0.mix.w2"] = np.zeros_like(tensors["l0.mix.w2"])
    tensors["embed"][:150] = ko.bf16_round(tensors["embed"][:150] * 0.05)
    n = 641
    toks = [t % 150 for t in tokens_of(cfg, n, 5)]
    other = list(toks)
    toks[20], other[20] = 158, 159
    ref_a, ref_b = ko.forward(cfg, tensors, toks)[-1], ko.forward(cfg, tensors, other)[-1]
    gap = rel(ref_a, ref_b)
    assert gap > 0.1
    eng = build(cfg, tensors, dt, blocks=24, max_model_len=704)
    for got in three_ways(eng, other):
        assert rel(got, ref_b) < (1e-4 if dt == F32 else 4e-2) and rel(got, ref_a) > gap / 2
    eng.close()


def test_the_previous_token_counts_across_every_cut():
    """the bonus and the shift reach exactly one token back: with a state that forgets at once (decays of zero) a changed token is felt at its own
    position and the two behind it (shift; key of a shifted row) and nowhere else — exactly, in portions and in decoding"""
    cfg = config([wkv(heads=2, dim=16)])
    tensors = ko.random_tensors(cfg, 11)
    tensors["l0.mix.w0"] = ko.bf16_round(np.full_like(tensors["l0.mix.w0"], 8.0))  # exp(-exp(8)) = 0 in f32
    tensors["l0.mix.w2"] = np.zeros_like(tensors["l0.mix.w2"])
    n, at = 90, 63
    toks = tokens_of(cfg, n, 4)
    other = list(toks)
    other[at] = (toks[at] + 3) % cfg["vocab"]
    ref_a, ref_b = ko.forward(cfg, tensors, toks), ko.forward(cfg, tensors, other)
    eng = build(cfg, tensors, F32, blocks=8, max_model_len=128)

    def run(t, cuts):
        out, p = [], 0
        for i, c in enumerate(cuts):
            out.append(eng.replay_step([(1, t[p:p + c], every(c))], [1] if i == len(cuts) - 1 else []))
            p += c
        return np.concatenate(out)
    for cuts in ([90], [63, 2, 25], [64, 2, 24], [62, 2, 2, 24], [5] + [1] * 85, [63] + [1] * 27):
        a, b = run(toks, cuts), run(other, cuts)
        agree(a, ref_a, F32), agree(b, ref_b, F32)
        changed = np.abs(a - b).max(-1)
        assert (changed[:at] == 0).all() and (changed[at + 3:] == 0).all() and (changed[at:at + 3] > 1e-6).all(), cuts
    eng.close()


# ------------------------------------------------------------------------------------------------ whole models
@pytest.fixture(scope="module", params=[("a", F32), ("a", BF16), ("b", F32), ("b", BF16)], ids=["a-f32", "a-bf16", "b-f32", "b-bf16"])
def model(request):
    name, dt = request.param
    cfg = config_a() if name == "a" else config_b()
    tensors = ko.random_tensors(cfg, 17 if name == "a" else 18, steady=dt == BF16)
    eng = build(cfg, tensors, dt, blocks=12, max_model_len=512, num_state_slots=4)
    yield cfg, tensors, dt, eng
    eng.close()


def test_layers_one_by_one(model):
    cfg, tensors, dt, eng = model
    toks = tokens_of(cfg, 90, 1)
    eng.layer_trace(True)
    got = eng.replay_step([(1, toks, every(90))], [1])
    trace = eng.read_layer_trace(90)
    eng.layer_trace(False)
    ref, layers = ko.forward(cfg, tensors, toks, True)
    for i, x in enumerate(layers):
        agree(trace[i], x, dt, f"layer {i}")
    agree(got, ref, dt)
    plain = eng.replay_step([(2, toks, every(90))], [2])  # (without the trace the layers' seams are one launch: the same sums)
    assert (plain == got).all()


def test_prefill_against_token_by_token_decoding(model):
    cfg, tensors, dt, eng = model
    toks = tokens_of(cfg, 150, 2)
    ref = ko.forward(cfg, tensors, toks)
    whole = eng.replay_step([(1, toks, every(150))], [1])
    agree(whole, ref, dt, "whole")
    one = np.stack([eng.replay_step([(2, toks[p:p + 1], [0])], [2] if p == 149 else [])[0] for p in range(150)])
    agree(one, ref, dt, "token by token")
    if dt == F32:
        assert same(one, whole, dt)


@pytest.mark.parametrize("sizes", [[2] * 30, [37, 3, 37, 2, 5], [64, 64, 2], [63, 2, 63, 2], [1, 5, 1, 1, 70, 1], [71, 9, 2, 70]])
def test_portions(model, sizes):
    """a prompt cut anywhere (down to two tokens, at and across page borders) gives the logits of the whole prompt"""
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
    agree(got, ko.forward(cfg, tensors, toks), dt)


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


def test_mixed_steps_with_reused_pages_and_slots(model):
    """12 pages and four slots for 8 requests that come and go: decoded tokens beside portions of prompts, some requests left out of a step, a
    finished request's pages and slot taken by the next one at once; every logit row equals the request's own run"""
    cfg, tensors, dt, eng = model
    r = np.random.default_rng(4)
    lens = [130, 60, 200, 90, 33, 150, 64, 128]
    prompts = [tokens_of(cfg, n, 40 + i) for i, n in enumerate(lens)]
    ref = [ko.forward(cfg, tensors, p) for p in prompts]
    waiting, live = list(range(len(prompts))), {}
    got_rows, ref_rows = [], []
    while waiting or live:
        while waiting and len(live) < 4 and sum((lens[i] + 63) // 64 for i in list(live) + [waiting[0]]) <= 12:
            live[waiting.pop(0)] = 0
        entries, ends, spans = [], [], []
        for i, at in live.items():
            if at and r.random() < 0.2 and len(live) > 1:
                continue
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


def test_a_fifth_request_waits_for_a_slot(model):
    cfg, tensors, dt, eng = model
    for i in range(4):
        eng.replay_step([(500 + i, [1, 2, 3], [])], [])
    with pytest.raises(RuntimeError, match="state slot"):
        eng.replay_step([(504, [1, 2, 3], [])], [])
    eng.replay_step([], [500, 501, 502, 503, 504])
    toks = tokens_of(cfg, 10, 1)
    agree(eng.replay_step([(505, toks, every(10))], [505]), ko.forward(cfg, tensors, toks), dt)


def test_long_decoding(model):
    """310 decoded tokens behind a 20-token prompt: page borders and the states pass under decoded tokens"""
    cfg, tensors, dt, eng = model
    toks = tokens_of(cfg, 330, 5)
    ref = ko.forward(cfg, tensors, toks)
    eng.replay_step([(1, toks[:20], [])], [])
    rows = [eng.replay_step([(1, toks[p:p + 1], [0])], [1] if p == len(toks) - 1 else [])[0] for p in range(20, len(toks))]
    agree(np.stack(rows), ref[20:], dt)


def test_long_prompt_in_one_step_and_in_portions():
    """a 1500-token prompt (bf16 prompt steps of this size take the large matrix tiles), whole, in three portions and with its last tokens decoded
    (more key tiles than one workgroup's waves)"""
    cfg = config([dict(attn(heads=4, kv_heads=2, dim=64, vdim=128, scale=0.12), mlp=moe(experts=8, top=2, ff=48, identity=2, shared=64)),
                  dict(attn(heads=4, kv_heads=2, dim=64, vdim=128, scale=0.2, kv_from=0), mlp=None), dict(wkv(heads=2, dim=64), mlp=dense(128))], width=128)
    tensors = ko.random_tensors(cfg, 23, rank=16, steady=True)
    toks = tokens_of(cfg, 1500, 8)
    want = sorted(set(list(range(0, 1500, 47)) + [699, 700, 1490, 1495, 1499]))
    ref = ko.forward(cfg, tensors, toks)[want]
    for dt in (F32, BF16):
        eng = build(cfg, tensors, dt, blocks=48, max_model_len=1536)
        whole = eng.replay_step([(1, toks, want)], [1])
        agree(whole, ref, dt, "whole")
        parts, at = [], 0
        for c in [700, 40, 750] + [1] * 10:
            parts.append(eng.replay_step([(2, toks[at:at + c], [w - at for w in want if at <= w < at + c])], [2] if at + c == 1500 else []))
            at += c
        eng.close()
        parts = np.concatenate([x for x in parts if len(x)])
        agree(parts, ref, dt, "portions")
        if dt == F32:
            assert same(parts, whole, dt)


@pytest.mark.parametrize("use_graph", [False, True], ids=["eager", "graphs"])
@pytest.mark.parametrize("dt", [F32, BF16], ids=["f32", "bf16"])
def test_greedy_generation_through_the_scheduler(use_graph, dt):
    """Engine.generate: the engine's own scheduler, block manager, state slots, prefill and decode steps (captured decode graphs when asked) and
    its argmax — against the oracle's greedy continuation; five requests of unequal length for four places, the fifth on used pages and a
    used slot, then two again through replayed graphs"""
    cfg = config_a()
    tensors = ko.random_tensors(cfg, 19, steady=dt == BF16)
    eng = build(cfg, tensors, dt, blocks=16, max_model_len=256, use_graph=use_graph)
    prompts = [tokens_of(cfg, n, 60 + n) for n in (5, 70, 31, 64, 120)]
    outs = eng.generate(prompts, max_tokens=12, ignore_eos=True)
    again = eng.generate(prompts[:2], max_tokens=12, ignore_eos=True)
    eng.close()
    close = 1e-3 if dt == F32 else 0.35
    turned = 0
    for p, out in zip(prompts + prompts[:2], outs + again):
        assert len(out) == 12
        seq = list(p)
        for t in out:
            lg = ko.forward(cfg, tensors, seq)[-1]
            turned += not (int(t) == int(lg.argmax()) or lg.max() - lg[int(t)] < close)
            seq.append(int(t))
    assert turned == 0 if dt == F32 else turned <= 6  # (bf16: a router's close call may turn a token)


def test_sampled_generation_stays_inside_the_top_k():
    cfg = config_a()
    tensors = ko.random_tensors(cfg, 21)
    eng = build(cfg, tensors, F32, blocks=16, max_model_len=256)
    prompts = [tokens_of(cfg, n, 80 + n) for n in (9, 40)]
    outs = eng.generate(prompts, max_tokens=8, ignore_eos=True, sampling=dict(temperature=0.9, top_k=3, top_p=1.0))
    eng.close()
    for p, out in zip(prompts, outs):
        seq = list(p)
        assert len(out) == 8
        for t in out:
            lg = ko.forward(cfg, tensors, seq)[-1]
            assert lg[int(t)] >= np.sort(lg)[-3] - 1e-3, (len(p), len(seq))
            seq.append(int(t))


def test_prefix_cache_serves_stacks_without_time_mixing_and_is_refused_by_the_others():
    """a stack of attention layers keeps nothing but cache rows: a second request with the same long prefix reuses them; a stack with a state refuses"""
    cfg = config([dict(attn(), mlp=moe()), dict(attn(kv_from=0), mlp=dense())])
    tensors = ko.random_tensors(cfg, 27)
    eng = build(cfg, tensors, F32, blocks=24, max_model_len=512, enable_prefix_cache=True)
    common = tokens_of(cfg, 200, 1)
    prompts = [common + tokens_of(cfg, n, 2 + n) for n in (7, 40)]
    outs = [eng.generate([p], max_tokens=6, ignore_eos=True)[0] for p in prompts + prompts[:1]]
    eng.close()
    for p, out in zip(prompts + prompts[:1], outs):
        seq = list(p)
        for t in out:
            lg = ko.forward(cfg, tensors, seq)[-1]
            assert lg.max() - lg[int(t)] < 1e-3
            seq.append(int(t))
    cfg = config([attn(), wkv()])
    with pytest.raises(RuntimeError, match="prefix cache"):
        build(cfg, ko.random_tensors(cfg, 1), F32, blocks=8, max_model_len=128, enable_prefix_cache=True).generate([[1, 2, 3]], max_tokens=2)


def test_synthetic_weights_and_state_plan():
    from vllm_rs_amd.engine import Engine
    for dtype in (None, "float32"):
        cfg = checkpoint.parse_config(config_a(), dtype)
        eng = Engine(cfg, max_num_seqs=4, max_model_len=256, kv_fraction=0.01, use_graph=False).init_synthetic()
        assert eng.num_gpu_blocks > 16
        out = eng.generate([list(range(1, 40)), list(range(3, 9))], max_tokens=5, ignore_eos=True)
        assert [len(o) for o in out] == [5, 5]
        eng.close()


def test_trace_runner_on_a_model_folder(tmp_path):
    """bin/trace_run as a user starts it: config.json + model.safetensors in a folder, steps on standard input (a prompt in portions beside
    another request's single tokens; a pool of three pages used again), logits files out — against the oracle"""
    cfg = config_a()
    tensors = ko.random_tensors(cfg, 31, steady=True)
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
    r1, r2, r3 = (ko.forward(cfg, tensors, p) for p in (p1, p2, p3))
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
