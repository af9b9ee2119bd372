"""CPU tests of the Pesivik design in the layer-stack model class: the reader of its config.json (every size and constant, optional
mechanisms), the native parser of the layer list it writes and its use by the scheduler (host-only engine: no GPU touched), and the
float64 oracle's mechanisms checked by hand (tests/pesivik_oracle.py)."""
import ctypes as C
import math

import numpy as np
import pytest

from tests import pesivik_oracle as po
from vllm_rs_amd import _lib, checkpoint
from vllm_rs_amd.engine import model_config


def mixer(heads=3, dim=8, rot_dim=4, vdim=6, kv_rank=12, q_rank=10, scale=0.4, size=9, base=300.0):
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale, mask=dict(size=size), rot=dict(base=base, dims=rot_dim))


def small_config():
    moe = dict(kind="moe", expert=dict(ff=20), router=dict(experts=6, top=3, groups=dict(count=3, keep=2)), shared=dict(ff=28))
    return dict(architecture="Pesivik", width=24, vocab=50, norm=dict(eps=2e-5), embedding=dict(scale=3.5), logit_softcap=11.0, layers=[
        dict(type="latent_attention", mixer=mixer(), mlp=moe),
        dict(type="latent_attention", mixer=mixer(heads=2, dim=5, rot_dim=2, vdim=7, kv_rank=9, q_rank=11, scale=0.7, size=17, base=70.0), mlp=None),
        dict(type="latent_attention", mixer=mixer(), mlp=moe, weights_of=0),
        dict(type="latent_attention", mixer=mixer(size=1), mlp=dict(kind="moe", expert=dict(ff=8), router=dict(experts=3, top=1))),
    ])


def fields(line):
    return dict(kv.split("=") for kv in line.split()[1:])


def test_config_reader_takes_every_size_and_constant_from_the_config():
    cfg = checkpoint.parse_config(small_config())
    assert cfg["arch"] == "stack" and cfg["design"] == "Pesivik" and cfg["hidden_size"] == 24 and cfg["vocab_size"] == 50 and cfg["num_layers"] == 4
    lines = cfg["spec"].strip().split("\n")
    top = fields(lines[0])
    assert (top["block"], top["norm"], top["pos"], float(top["eps"]), int(top["layer_scale"])) == ("sandwich", "layer", "none", 2e-5, 1)
    assert (float(top["embed_scale"]), float(top["logit_softcap"])) == (3.5, 11.0)
    l0, l1, l2, l3 = (fields(x) for x in lines[1:])
    assert (l0["mixer"], int(l0["heads"]), int(l0["kv_heads"]), int(l0["dim"]), int(l0["rot_dim"]), int(l0["vdim"]), int(l0["kv_rank"]), int(l0["q_rank"])) == ("latent", 3, 1, 8, 4, 6, 12, 10)
    assert (float(l0["scale"]), int(l0["window"]), int(l0["rot_dims"]), float(l0["rot_base"]), l0["rot_layout"], int(l0["head_gate"])) == (0.4, 9, 4, 300.0, "half", 1)
    assert (l0["mlp"], int(l0["ff"]), int(l0["experts"]), int(l0["top"]), l0["router"], l0["act"], int(l0["groups"]), int(l0["keep"]), int(l0["shared_ff"])) == ("moe", 20, 6, 3, "sigmoid_norm", "gelu", 3, 2, 28)
    assert (int(l1["heads"]), int(l1["dim"]), int(l1["rot_dim"]), int(l1["vdim"]), int(l1["kv_rank"]), int(l1["q_rank"]), float(l1["scale"]), int(l1["window"]), float(l1["rot_base"])) == (2, 5, 2, 7, 9, 11, 0.7, 17, 70.0)
    assert l1["mlp"] == "none" and "weights_of" not in l1 and int(l2["weights_of"]) == 0
    # what the config leaves out is off: no groups, no shared expert
    assert int(l3["window"]) == 1 and int(l3["top"]) == 1 and "groups" not in l3 and "shared_ff" not in l3
    plain = small_config()
    del plain["logit_softcap"], plain["embedding"]
    t = fields(checkpoint.parse_config(plain)["spec"].split("\n")[0])
    assert float(t["logit_softcap"]) == 0.0 and float(t["embed_scale"]) == 1.0
    assert checkpoint.parse_config(small_config(), "float32")["dtype"] == checkpoint.F32


def test_config_reader_rejects_what_the_design_does_not_have():
    for edit in (lambda c: c["layers"][0].update(type="attention"), lambda c: c["layers"][0]["mlp"].update(kind="dense"),
                 lambda c: c["layers"][1]["mixer"]["rot"].update(dims=4)):
        bad = small_config()
        edit(bad)
        with pytest.raises(ValueError):
            checkpoint.parse_config(bad)
    with pytest.raises(ValueError):
        checkpoint.parse_config(small_config(), "float16")


def create(spec, cfg, **kw):
    L = _lib.load()
    mc = model_config(cfg)
    ec = _lib.EngineConfig(**dict(dict(block_size=64, max_num_seqs=4, max_model_len=256, num_gpu_blocks=8, prefill_chunk=8192, device=-1), **kw))
    h = L.vra_engine_create_spec(C.byref(mc), C.byref(ec), spec.encode())
    assert h
    return L, h


def test_native_parser_accepts_the_layer_list():
    cfg = checkpoint.parse_config(small_config())
    L, h = create(cfg["spec"], cfg)
    assert L.vra_engine_finalize_weights(h) == 0, L.vra_engine_last_error(h).decode()
    L.vra_engine_destroy(h)


@pytest.mark.parametrize("edit,why", [
    (lambda s: s.replace("block=sandwich", "block=sequential"), "layer norms belong to sandwich blocks"),
    (lambda s: s.replace("norm=layer", "norm=dyt"), "layer_scale belongs"),
    (lambda s: s.replace("norm=layer", "norm=batch"), "norm must be"),
    (lambda s: s.replace("kv_rank=12", "kv_rank=513", 1), "0 < kv_rank <= 512"),
    (lambda s: s.replace("rot_dims=4", "rot_dims=3", 1), "even rot_dims"),
    (lambda s: s.replace("rot_layout=half", "rot_layout=thirds", 1), "rot_layout half or pairs"),
    (lambda s: s.replace("groups=3 keep=2", "groups=4 keep=2", 1), "groups must divide"),
    (lambda s: s.replace("groups=3 keep=2", "groups=3 keep=4", 1), "keep <= groups"),
    (lambda s: s.replace("router=sigmoid_norm", "router=dice", 1), "router is sigmoid or softmax or softmax_all or sigmoid_norm"),
    (lambda s: s.replace("act=gelu", "act=relu", 1), "clamped or silu or gelu"),
    (lambda s: s.replace("router=sigmoid_norm", "router=softmax", 1), "without a gate belong"),
    (lambda s: s.replace("weights_of=0", "weights_of=2"), "must name another layer"),
    (lambda s: s.replace("weights_of=0", "weights_of=1"), "has the shapes of the layer it names"),
    (lambda s: s.replace("weights_of=0", "weights_of=0 identity=1"), "identity experts belong"),
    (lambda s: s.replace("window=17", "window=17 branch_norm=1"), "branch_norm belong"),
])
def test_native_parser_refuses_inconsistent_lists(edit, why):
    """the refusal surfaces at the first call that needs the model (loading a tensor), with the reason"""
    cfg = checkpoint.parse_config(small_config())
    L, h = create(edit(cfg["spec"]), cfg)
    a = np.zeros((50, 24), np.uint16)
    shape = (C.c_int64 * 2)(50, 24)
    assert L.vra_engine_load_tensor(h, b"embed", a.ctypes.data_as(C.c_void_p), shape, 2, 2) != 0
    assert why in L.vra_engine_last_error(h).decode()
    L.vra_engine_destroy(h)


def test_scheduler_batches_by_pages_alone():
    """the design keeps no state per sequence: requests wait for pages only (8 pages, requests of three, two and four pages and one more)"""
    cfg = checkpoint.parse_config(small_config())
    L, h = create(cfg["spec"], cfg)
    assert L.vra_engine_finalize_weights(h) == 0, L.vra_engine_last_error(h).decode()
    rids = []
    for n in (150, 70, 200, 5):
        p = (np.arange(1, n + 1) % 49).astype(np.uint32)
        rids.append(L.vra_engine_add_request(h, p.ctypes.data_as(C.c_void_p), n, 2, 1, None, 0))
    seen, served = [], set()
    for _ in range(40):
        pf, m = C.c_int32(0), _lib.StepMeta()
        n = L.vra_engine_dry_schedule(h, C.byref(pf), C.byref(m))
        assert n >= 0, L.vra_engine_last_error(h).decode()
        if n == 0:
            if not L.vra_engine_has_unfinished(h):
                break
            continue
        seen.append([int(m.request_ids[i]) for i in range(n)])
        served |= set(seen[-1])
        t = np.full(n, 9, np.uint32)
        assert L.vra_engine_dry_commit(h, t.ctypes.data_as(C.c_void_p), n) == n
    assert served == set(rids) and not L.vra_engine_has_unfinished(h)
    assert rids[2] not in seen[0] and {rids[0], rids[1]} <= set(seen[0])  # (3 + 2 + 4 pages do not fit into 8)
    L.vra_engine_destroy(h)


# ------------------------------------------------------------------------------------------------ the oracle's mechanisms by hand
def test_layer_norm_takes_the_mean_off():
    x = np.array([[1.0, 3.0], [101.0, 103.0]])
    out = po.layer_norm(x, np.array([2.0, 5.0]), 0.0)
    assert np.allclose(out, [[-2.0, 5.0], [-2.0, 5.0]])  # (a common offset does not show)
    assert np.allclose(po.layer_norm(x, np.ones(2), 3.0), [[-0.5, 0.5], [-0.5, 0.5]])  # eps inside the root: 1 / sqrt(1 + 3)


def test_gelu_is_the_exact_one():
    z = np.array([-1.0, 0.0, 2.0])
    assert np.allclose(po.gelu_erf(z), [-1 * 0.15865525393145707, 0.0, 2 * 0.9772498680518208])
    assert abs(po.gelu_erf(np.array([2.0]))[0] - 0.5 * 2 * (1 + math.tanh(math.sqrt(2 / math.pi) * (2 + 0.044715 * 8)))) > 1e-5


def test_rotary_pairs_the_halves():
    v = np.array([[1.0, 0.0, 0.0, 2.0]])  # pairs (0, 2) and (1, 3); position 3, base 100
    out = po.rotate_half(v, [3], 100.0)[0]
    assert np.allclose(out, [math.cos(3.0), -2 * math.sin(0.3), math.sin(3.0), 2 * math.cos(0.3)])


def test_window_counts_the_query_itself():
    vis = po.in_window([4, 1], 6, 3)
    assert vis[0].tolist() == [False, False, True, True, True, False] and vis[1].tolist() == [True, True, False, False, False, False]
    q, k = np.zeros((2, 1, 1)), np.zeros((2, 1, 1))
    v = np.array([[[1.0]], [[3.0]]])
    assert np.allclose(po.windowed_attention(q, k, v, 1.0, po.in_window([0, 1], 2, 2))[:, 0, 0], [1.0, 2.0])
    assert np.allclose(po.windowed_attention(q, k, v, 1.0, po.in_window([0, 1], 2, 1))[:, 0, 0], [1.0, 3.0])


def test_router_groups_correction_and_weights():
    w = {"router": np.zeros((6, 1)), "correction": np.zeros(6)}
    logit = lambda s: math.log(s / (1 - s))
    s = np.array([0.9, 0.1, 0.6, 0.5, 0.7, 0.35])
    w["router"][:, 0] = [logit(v) for v in s]
    h = np.ones((1, 1))
    r = dict(top=2, groups=dict(count=3, keep=1))
    chosen, wt = po.route(h, r, w, "")  # worth 1.0, 1.1, 1.05: the second group, although the best expert sits in the first
    assert chosen[0].tolist() == [2, 3] and np.allclose(wt[0], [0.6 / 1.1, 0.5 / 1.1])
    w["correction"] = np.array([-3.0, -2.0, -3.0, -3.0, -3.0, -2.5])  # every choice score negative: left-out experts are -inf, not 0
    chosen, wt = po.route(h, dict(top=3, groups=dict(count=3, keep=2)), w, "")
    c = s + w["correction"]
    worth = c.reshape(3, 2).sum(1)
    kept = sorted(np.argsort(-worth)[:2])
    allowed = [2 * g + i for g in kept for i in range(2)]
    best = sorted(allowed, key=lambda e: -c[e])[:3]
    assert chosen[0].tolist() == best and np.allclose(wt[0], s[best] / s[best].sum())  # the correction is not in the weights
    assert po.route(h, dict(top=1), w, "")[0][0].tolist() == [int(np.argmax(c))]
    assert np.allclose(po.keep_best_groups(np.array([0.5, -1.0, 2.0]), 3, 1), [-np.inf, -np.inf, 2.0])  # groups of one expert


def test_absorbed_scores_equal_the_textbook_ones():
    """q . (W_uk c) = (W_uk^T q) . c and W_uv (sum a c) = sum a (W_uv c): what the cache of latents rests on"""
    r = np.random.default_rng(0)
    c, uk, uv, q = r.standard_normal((7, 5)), r.standard_normal((4, 5)), r.standard_normal((3, 5)), r.standard_normal(4)
    assert np.allclose((c @ uk.T) @ q, c @ (uk.T @ q))
    a = r.random(7)
    assert np.allclose(a @ (c @ uv.T), uv @ (a @ c))


def test_whole_model():
    cfg = small_config()
    w = po.random_tensors(cfg, 3)
    lg, layers = po.forward(cfg, w, [1, 2, 3, 4, 5], True)
    assert lg.shape == (5, 50) and layers.shape == (4, 5, 24) and np.abs(lg).max() < 11.0
    assert np.allclose(po.forward(cfg, w, [1, 2, 3]), lg[:3])  # causal
    assert "l2.mix.dq" not in w and "l1.ls2" not in w  # a layer that shares weights has none, a layer without feed-forward has no second scale
    flat = dict(w, **{"l%d.ls%d" % (i, j): np.zeros(24) for i in range(4) for j in (1, 2)})
    _, lay = po.forward(cfg, flat, [1, 2], True)
    assert np.allclose(lay[-1], w["embed"][[1, 2]] * 3.5)  # scales of zero leave the scaled embedding
