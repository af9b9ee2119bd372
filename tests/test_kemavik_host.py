"""CPU tests of the Kemavik design in the layer-stack model class: the reader of its config.json (every size and constant, optional mechanisms),
the native parser of the layer list it writes and the scheduler's state slots (host-only engine: no GPU touched), and the float64 oracle's
mechanisms checked by hand (tests/kemavik_oracle.py)."""
import ctypes as C
import math

import numpy as np
import pytest

from tests import kemavik_oracle as ko
from vllm_rs_amd import _lib, checkpoint
from vllm_rs_amd.engine import model_config


def small_config():
    at = dict(heads=4, kv_heads=2, dim=5, vdim=6, scale=0.4, diff=0.35)
    moe = dict(kind="moe", expert=dict(ff=20), router=dict(experts=5, identity=3, scale=1.25, top=2), shared=dict(ff=28))
    return dict(architecture="Kemavik", width=24, vocab=50, norm=dict(eps=2e-5), layers=[
        dict(type="attention", mixer=at, mlp=moe),
        dict(type="wkv", mixer=dict(heads=3, dim=7), mlp=dict(kind="dense", ff=33)),
        dict(type="attention", mixer=dict(at, kv_from=0, scale=0.9, diff=0.0), mlp=None),
        dict(type="attention", mixer=dict(heads=2, dim=8, diff=0.5), mlp=dict(kind="moe", expert=dict(ff=8), router=dict(experts=3))),
    ])


def fields(line):
    return dict(kv.split("=") for kv in line.split()[1:])


def test_config_reader_takes_every_size_and_constant_from_the_config():
    cfg = checkpoint.parse_config(small_config())
    assert cfg["arch"] == "stack" and cfg["design"] == "Kemavik" and cfg["hidden_size"] == 24 and cfg["vocab_size"] == 50 and cfg["num_layers"] == 4
    lines = cfg["spec"].strip().split("\n")
    top = fields(lines[0])
    assert (top["block"], top["norm"], top["pos"], float(top["eps"]), float(top["norm_offset"])) == ("post", "rms", "none", 2e-5, 1.0)
    l0, l1, l2, l3 = (fields(x) for x in lines[1:])
    assert (l0["mixer"], int(l0["heads"]), int(l0["kv_heads"]), int(l0["dim"]), int(l0["vdim"]), float(l0["scale"]), float(l0["diff"]), int(l0["kv_from"])) == ("differential", 4, 2, 5, 6, 0.4, 0.35, -1)
    assert (l0["mlp"], int(l0["ff"]), int(l0["experts"]), int(l0["identity"]), float(l0["router_scale"]), int(l0["top"]), l0["router"], l0["act"], int(l0["shared_ff"])) == ("moe", 20, 5, 3, 1.25, 2, "softmax_all", "silu", 28)
    assert (l1["mixer"], int(l1["heads"]), int(l1["dim"]), l1["mlp"], int(l1["ff"])) == ("wkv", 3, 7, "relu2", 33)
    assert (int(l2["kv_from"]), float(l2["scale"]), float(l2["diff"]), l2["mlp"]) == (0, 0.9, 0.0, "none")
    # what the config leaves out has its default: as many key/value heads as heads, value size = key size, scale 1 / sqrt(dim), no identity experts,
    # weights as they are, one expert a token, no shared expert
    assert (int(l3["kv_heads"]), int(l3["vdim"])) == (2, 8) and abs(float(l3["scale"]) - 8 ** -0.5) < 1e-12
    assert (int(l3["identity"]), float(l3["router_scale"]), int(l3["top"])) == (0, 1.0, 1) and "shared_ff" not in l3
    assert checkpoint.parse_config(small_config(), "float32")["dtype"] == checkpoint.F32


def test_config_reader_rejects_what_the_design_does_not_have():
    for edit in (lambda c: c["layers"][0].update(type="latent_attention"), lambda c: c["layers"][1]["mlp"].update(kind="gated")):
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
    (lambda s: s.replace("block=post", "block=sandwich"), "post blocks hold differential and wkv"),
    (lambda s: s.replace("block=post", "block=middle"), "block must be parallel or sequential or sandwich or post"),
    (lambda s: s.replace("norm=rms", "norm=dyt"), "post blocks have rms norms"),
    (lambda s: s.replace("norm=rms", "norm=layer"), "layer norms belong to sandwich blocks"),
    (lambda s: s.replace("mixer=wkv", "mixer=lightning"), "post blocks hold differential and wkv"),
    (lambda s: s.replace("mixer=wkv", "mixer=thunder"), "unknown mixer"),
    (lambda s: s.replace("heads=3 dim=7", "heads=3 dim=300"), "wkv needs dim <= 256"),
    (lambda s: s.replace("heads=3 dim=7", "heads=3 vdim=8 dim=7"), "vdim = dim"),
    (lambda s: s.replace("rank_a=32", "rank_a=0"), "rank_a"),
    (lambda s: s.replace("kv_from=0", "kv_from=1"), "projections of its own"),
    (lambda s: s.replace("kv_from=0", "kv_from=3"), "earlier layer"),
    (lambda s: s.replace("kv_from=0 mlp=none", "kv_from=0 mlp=clamped ff=8"), "post blocks have"),
    (lambda s: s.replace("dim=5 vdim=6 scale=0.9", "dim=6 vdim=6 scale=0.9"), "equal key / value shapes"),
    (lambda s: s.replace("vdim=6", "vdim=600"), "value sizes up to 512"),
    (lambda s: s.replace("kv_heads=2", "kv_heads=3", 1), "multiple of kv_heads"),
    (lambda s: s.replace("router=softmax_all", "router=softmax", 1), "router=softmax_all and act=silu"),
    (lambda s: s.replace("act=silu", "act=gelu", 1), "act=silu"),
    (lambda s: s.replace("mlp=relu2 ff=33", "mlp=relu2 ff=0"), "without ff"),
    (lambda s: s.replace("top=2", "top=9"), "1 <= top <= experts"),
])
def test_native_parser_refuses_inconsistent_lists(edit, why):
    """the refusal surfaces at the first call that needs the model (loading a tensor), with the reason"""
    cfg = checkpoint.parse_config(small_config())
    assert edit(cfg["spec"]) != cfg["spec"]
    L, h = create(edit(cfg["spec"]), cfg)
    a = np.zeros((50, 24), np.uint16)
    shape = (C.c_int64 * 2)(50, 24)
    assert L.vra_engine_load_tensor(h, b"embed", a.ctypes.data_as(C.c_void_p), shape, 2, 2) != 0
    assert why in L.vra_engine_last_error(h).decode()
    L.vra_engine_destroy(h)


def serve(L, h, lens, max_tokens=2):
    rids, seen = [], []
    for n in lens:
        p = (np.arange(1, n + 1) % 49).astype(np.uint32)
        rids.append(L.vra_engine_add_request(h, p.ctypes.data_as(C.c_void_p), n, max_tokens, 1, None, 0))
    for _ in range(40):
        pf, m = C.c_int32(0), _lib.StepMeta()
        n = L.vra_engine_dry_schedule(h, C.byref(pf), C.byref(m))
        assert n >= 0, L.vra_engine_last_error(h).decode()
        if n == 0:
            if not L.vra_engine_has_unfinished(h):
                break
            continue
        seen.append([int(m.request_ids[i]) for i in range(n)])
        t = np.full(n, 9, np.uint32)
        assert L.vra_engine_dry_commit(h, t.ctypes.data_as(C.c_void_p), n) == n
    assert not L.vra_engine_has_unfinished(h)
    return rids, seen


def test_scheduler_hands_out_state_slots_and_takes_them_back():
    """two state slots, three requests: the scheduler batches two, the third waits although pages are free, and runs when a slot comes back"""
    cfg = checkpoint.parse_config(small_config())
    L, h = create(cfg["spec"], cfg, num_state_slots=2)
    assert L.vra_engine_finalize_weights(h) == 0, L.vra_engine_last_error(h).decode()
    rids, seen = serve(L, h, (5, 7, 3))
    assert sorted(seen[0]) == sorted(rids[:2]) and max(len(s) for s in seen) == 2 and any(rids[2] in s for s in seen[1:])
    L.vra_engine_destroy(h)


def test_a_stack_of_attention_layers_needs_no_slots():
    c = small_config()
    del c["layers"][1]
    c["layers"][1]["mixer"]["kv_from"] = 0
    cfg = checkpoint.parse_config(c)
    L, h = create(cfg["spec"], cfg, num_state_slots=1)
    assert L.vra_engine_finalize_weights(h) == 0, L.vra_engine_last_error(h).decode()
    rids, seen = serve(L, h, (5, 7, 3))
    assert sorted(seen[0]) == sorted(rids)
    L.vra_engine_destroy(h)


# ------------------------------------------------------------------------------------------------ the oracle's mechanisms by hand
def test_norms():
    x = np.array([[3.0, 4.0]])
    assert np.allclose(ko.unit_rms(x, 0.0), x / math.sqrt(12.5))
    assert np.allclose(ko.unit_rms(x, 87.5), x / 10.0)  # eps inside the root
    assert np.allclose(ko.output_norm(x, np.array([0.0, -1.0]), 0.0), [[3.0 / math.sqrt(12.5), 0.0]])  # weights around zero


def test_two_maps_over_the_same_values():
    """two keys: map 1 weighs them (1, 0) in effect, map 2 (1/2, 1/2)"""
    q = np.zeros((1, 1, 2, 1))
    q[0, 0, 0] = 100.0
    k = np.zeros((2, 1, 2, 1))
    k[0, 0, 0] = 1.0
    v = np.array([[[2.0, 0.0]], [[0.0, 4.0]]])
    out = ko.differential_heads(q, k, v, 1.0, 0.5, 0.25, 0.0)[0, 0]
    o = np.array([2.0, 0.0]) - 0.5 * np.array([1.0, 2.0])
    assert np.allclose(out, o / math.sqrt((o * o).mean()) * 0.75)
    one = ko.differential_heads(q, k[:1], v[:1], 1.0, 0.5, 0.25, 0.0)[0, 0]  # a sequence's first token: both maps return its own value
    assert np.allclose(one, np.array([math.sqrt(2.0), 0.0]) * 0.75)


def test_lambda():
    w = {"lq1": np.array([1.0, 2.0]), "lk1": np.array([0.5, 0.25]), "lq2": np.array([1.0, 0.0]), "lk2": np.array([-1.0, 9.0])}
    assert abs(ko.head_lambda(w, "", 0.3) - (math.e - math.exp(-1.0) + 0.3)) < 1e-12


def test_grouped_heads_and_causality():
    r = np.random.default_rng(0)
    q, k, v = r.standard_normal((5, 4, 2, 3)), r.standard_normal((5, 2, 2, 3)), r.standard_normal((5, 2, 6))
    out = ko.differential_heads(q, k, v, 0.7, 0.4, 0.2, 1e-5)
    assert np.allclose(ko.differential_heads(q[:, 2:3], k[:, 1:], v[:, 1:], 0.7, 0.4, 0.2, 1e-5)[:, 0], out[:, 2])  # heads 2 and 3 read group 1
    assert np.allclose(ko.differential_heads(q[:3], k[:3], v[:3], 0.7, 0.4, 0.2, 1e-5), out[:3])
    assert np.allclose(ko.differential_heads(q[3:], k, v, 0.7, 0.4, 0.2, 1e-5), out[3:])


def test_recurrence_of_two_tokens():
    r1, r2, k1, k2 = (np.array(a)[None, None] for a in ([1.0, 2.0], [3.0, 1.0], [0.5, 1.0], [2.0, -1.0]))
    v1, v2 = np.array([[[4.0]]]), np.array([[[10.0]]])
    u, w = np.array([[0.1, 0.2]]), np.array([[[0.5, 0.25]]])
    o, S = ko.wkv(np.concatenate([r1, r2]), np.concatenate([k1, k2]), np.concatenate([v1, v2]), np.concatenate([w, w]), u)
    assert np.isclose(o[0, 0, 0], (0.1 * 0.5 * 1 + 0.2 * 1 * 2) * 4)               # nothing but the bonus
    assert np.isclose(o[1, 0, 0], (0.5 * 3 + 1.0 * 1) * 4 + (0.1 * 2 * 3 + 0.2 * -1 * 1) * 10)  # the state is read before its decay
    assert np.allclose(S[0, :, 0], [0.5 * 0.5 * 4 + 2 * 10, 0.25 * 1 * 4 - 10])
    rest, _ = ko.wkv(r2, k2, v2, w, u, state=ko.wkv(r1, k1, v1, w, u)[1])
    assert np.isclose(rest[0, 0, 0], o[1, 0, 0])


def test_token_shift_and_decays():
    x = np.array([[1.0], [3.0], [4.0]])
    assert ko.shifted(x)[:, 0].tolist() == [0.0, 1.0, 3.0]
    w = {"w1": np.array([[2.0]]), "w2": np.array([[3.0], [0.0]]), "w0": np.array([0.5, -1.0])}
    d = ko.decays(np.array([[0.25]]), w, "")
    assert np.allclose(d, [[math.exp(-math.exp(3 * math.tanh(0.5) + 0.5)), math.exp(-math.exp(-1.0))]])


def test_router_correction_scale_and_identity():
    w = {"router": np.log(np.array([[0.4], [0.3], [0.2], [0.1]])), "correction": np.array([0.0, 0.0, 0.0, 0.25])}
    h = np.ones((1, 1))
    chosen, wt = ko.route(h, dict(top=2, scale=2.0), w, "")  # choice scores 0.4, 0.3, 0.2, 0.35
    assert chosen[0].tolist() == [0, 3] and np.allclose(wt[0], [0.8, 0.2])  # the correction is not in the weights; not renormalised
    assert np.allclose(ko.route(h, dict(top=1), w, "")[1], [[0.4]])
    w.update({"e0.gate": np.array([[1.0]]), "e0.up": np.array([[2.0]]), "e0.down": np.array([[3.0]])})
    w.update({"e%d.%s" % (e, n): np.array([[0.0]]) for e in (1, 2) for n in ("gate", "up", "down")})
    mlp = dict(router=dict(experts=3, identity=1, top=2, scale=2.0))
    expert = float(ko.silu(1.0)) * 2 * 3
    assert np.allclose(ko.mixture(h, mlp, w, ""), [[0.8 * expert + 0.2]])  # the last output hands its input back
    w.update({"shared." + n: w["e0." + n] for n in ("gate", "up", "down")})
    assert np.allclose(ko.mixture(h, dict(mlp, shared=dict(ff=1)), w, ""), [[1.8 * expert + 0.2]])


def test_dense_is_a_squared_relu():
    w = {"up": np.array([[1.0], [-1.0]]), "down": np.array([[1.0, 10.0]])}
    assert np.allclose(ko.dense(np.array([[3.0], [-2.0]]), w, ""), [[9.0], [40.0]])


def test_whole_model():
    cfg = small_config()
    cfg["layers"][3]["mixer"].update(kv_heads=2, vdim=8, scale=0.3)
    w = ko.random_tensors(cfg, 3)
    lg, layers = ko.forward(cfg, w, [1, 2, 3, 4, 5], True)
    assert lg.shape == (5, 50) and layers.shape == (4, 5, 24)
    assert np.allclose(ko.forward(cfg, w, [1, 2, 3]), lg[:3])  # causal
    assert "l2.mix.k" not in w and "l2.mix.lq1" in w and "l2.norm2" not in w  # a borrowing layer has no keys, a layer without feed-forward no second norm
    flat = dict(w, **{"l%d.norm%d" % (i, j): np.full(24, -1.0) for i in range(4) for j in (1, 2)})
    _, lay = ko.forward(cfg, flat, [1, 2], True)
    assert np.allclose(lay[-1], w["embed"][[1, 2]])  # norms that weigh nothing leave the embedding
