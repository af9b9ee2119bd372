"""Float64 numpy statement of the Kemavik design: one function per mechanism, a whole sequence at a time, no cache, no pages, the recurrence one
token after the other, experts one at a time.  Shares no code with the product path; the tests compare the engine with it.

A model is (cfg, w): cfg the dict of a config.json of the design, w a dict tensor name -> array.

Notation: x residual stream [T, width], N(v) = v / sqrt(mean(v^2) + eps) * (1 + weight); a layer reads x itself and norms what comes out:
    x <- x + N(mixer(x)),   x <- x + N(ff(x))
"""
import math

import numpy as np


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * np.asarray(z, np.float64)))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    """divided by its root mean square over the last axis, eps inside the root"""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def output_norm(x, weight, eps):
    """weight stored around zero"""
    return unit_rms(x, eps) * (1.0 + weight)


# ------------------------------------------------------------------------------------------------ differential attention
def causal_softmax(scores):
    """scores [Tq, Tk] of the last Tq of Tk tokens -> weights"""
    Tq, Tk = scores.shape
    seen = np.arange(Tk)[None, :] <= np.arange(Tk - Tq, Tk)[:, None]
    s = np.where(seen, scores, -np.inf)
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def head_lambda(w, p, diff):
    return math.exp(float(w[p + "lq1"] @ w[p + "lk1"])) - math.exp(float(w[p + "lq2"] @ w[p + "lk2"])) + diff


def differential_heads(q, k, v, scale, lam, diff, eps):
    """q [Tq, H, 2, D], k [Tk, G, 2, D], v [Tk, G, V] -> [Tq, H, V]: two maps over the same values, the second taken off lam times; the
    difference is divided by its root mean square and shrunk by 1 - diff"""
    H, G = q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        a1, a2 = (causal_softmax((q[:, h, m] @ k[:, g, m].T) * scale) @ v[:, g] for m in (0, 1))
        out.append(unit_rms(a1 - lam * a2, eps) * (1.0 - diff))
    return np.stack(out, 1)


def keys_values(x, mx, w, p, eps):
    T, G, D, V = x.shape[0], int(mx["kv_heads"]), int(mx["dim"]), int(mx["vdim"])
    k = (x @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, 2, D)
    v = (x @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, V)
    return unit_rms(k, eps) * w[p + "k.norm"], v


def attention(x, mx, w, p, eps, kv):
    T, H, D = x.shape[0], int(mx["heads"]), int(mx["dim"])
    q = unit_rms((x @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, 2, D), eps) * w[p + "q.norm"]
    diff = float(mx["diff"])
    o = differential_heads(q, kv[0], kv[1], float(mx["scale"]), head_lambda(w, p, diff), diff, eps)
    return o.reshape(T, -1) @ w[p + "o"].T + w[p + "o.b"]


# ------------------------------------------------------------------------------------------------ time mixing
def shifted(x):
    """the previous token's row, zeros for the first token"""
    return np.concatenate([np.zeros_like(x[:1]), x[:-1]], 0)


def wkv(r, k, v, decay, u, state=None):
    """r, k, decay [T, H, D], v [T, H, V], u [H, D] -> (o [T, H, V], the state [H, D, V] after the last token):
    o_t = (S + diag(u) k v^T)^T r,  then  S <- diag(decay) S + k v^T"""
    T, H, D = r.shape
    S = np.zeros((H, D, v.shape[2])) if state is None else state.copy()
    o = np.zeros(v.shape)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S + u[:, :, None] * kv, r[t])
        S = decay[t][:, :, None] * S + kv
    return o, S


def decays(mix, w, p):
    """exp(-exp(low-rank projection + offset)), per channel"""
    return np.exp(-np.exp(np.tanh(mix @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]))


def time_mixing(x, mx, w, p, eps):
    T, H, D = x.shape[0], int(mx["heads"]), int(mx["dim"])
    d = shifted(x) - x
    mix = {c: x + d * w[p + "mu." + c] for c in "rkvgw"}
    r, k, v = ((mix[c] @ w[p + c].T).reshape(T, H, D) for c in "rkv")
    o, _ = wkv(r, k, v, decays(mix["w"], w, p).reshape(T, H, D), w[p + "u"].reshape(H, D))
    o = unit_rms(o, eps).reshape(T, H * D) * w[p + "norm"] * silu(mix["g"] @ w[p + "g"].T)
    return o @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def dense(h, w, p):
    return np.maximum(h @ w[p + "up"].T, 0.0) ** 2 @ w[p + "down"].T


def gated(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, router, w, p):
    """-> (chosen [T, top], weights [T, top]): softmax over all outputs; a correction takes part in the choice alone; the weights are the chosen
    scores times a constant"""
    z = h @ w[p + "router"].T
    e = np.exp(z - z.max(-1, keepdims=True))
    s = e / e.sum(-1, keepdims=True)
    chosen = np.argsort(-(s + w[p + "correction"]), axis=-1, kind="stable")[:, :int(router.get("top", 1))]
    return chosen, np.take_along_axis(s, chosen, -1) * float(router.get("scale", 1.0))


def mixture(h, mlp, w, p):
    chosen, wt = route(h, mlp["router"], w, p)
    E = int(mlp["router"]["experts"])
    out = np.zeros_like(h)
    for e in range(E + int(mlp["router"].get("identity") or 0)):
        hit = chosen == e
        rows = np.nonzero(hit.any(-1))[0]
        if len(rows):
            y = gated(h[rows], w, "%se%d." % (p, e)) if e < E else h[rows]  # the last outputs hand their input back
            out[rows] += (wt * hit).sum(-1)[rows, None] * y
    if mlp.get("shared"):
        out = out + gated(h, w, p + "shared.")
    return out


def feed_forward(h, mlp, w, p):
    return dense(h, w, p) if mlp["kind"] == "dense" else mixture(h, mlp, w, p)


# ------------------------------------------------------------------------------------------------ the model
def forward(cfg, w, tokens, return_layers=False):
    """-> logits [T, vocab] (and the residual stream after every layer [L, T, width])"""
    eps = float(cfg["norm"]["eps"])
    w = {k: np.asarray(v, np.float64) for k, v in w.items()}
    x = w["embed"][np.asarray(tokens)]
    trace, kv = [], {}
    for i, layer in enumerate(cfg["layers"]):
        p, mx = "l%d." % i, layer["mixer"]
        if layer["type"] == "wkv":
            m = time_mixing(x, mx, w, p + "mix.", eps)
        else:
            j = mx.get("kv_from")
            kv[i] = keys_values(x, mx, w, p + "mix.", eps) if j is None else kv[int(j)]
            m = attention(x, mx, w, p + "mix.", eps, kv[i])
        x = x + output_norm(m, w[p + "norm1"], eps)
        if layer.get("mlp"):
            x = x + output_norm(feed_forward(x, layer["mlp"], w, p + "mlp."), w[p + "norm2"], eps)
        trace.append(x.copy())
    logits = output_norm(x, w["final.norm"], eps) @ w["head"].T
    return (logits, np.stack(trace)) if return_layers else logits


# ------------------------------------------------------------------------------------------------ random models for the tests
def bf16_round(a):
    """float32 array rounded to bfloat16 (nearest even), returned as float32"""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    return (((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16).astype(np.uint32).view(np.float32).reshape(np.shape(a))


def tensor_shapes(cfg, rank=6):
    """rank: of the decays' low-rank projections (the config does not name it, the tensors' shapes do)"""
    W, V = int(cfg["width"]), int(cfg["vocab"])
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        p, mx, mlp = "l%d." % i, layer["mixer"], layer.get("mlp")
        H, D = int(mx["heads"]), int(mx["dim"])
        m = p + "mix."
        out[p + "norm1"] = (W,)
        if layer["type"] == "wkv":
            out.update({m + "mu." + c: (W,) for c in "rkvgw"})
            out.update({m + c: (H * D, W) for c in "rkvg"})
            out.update({m + "w1": (rank, W), m + "w2": (H * D, rank), m + "w0": (H * D,), m + "u": (H, D), m + "norm": (H * D,), m + "o": (W, H * D)})
        else:
            G, vd = int(mx["kv_heads"]), int(mx["vdim"])
            out.update({m + "q": (H * 2 * D, W), m + "q.b": (H * 2 * D,), m + "q.norm": (D,), m + "o": (W, H * vd), m + "o.b": (W,)})
            out.update({m + n: (D,) for n in ("lq1", "lk1", "lq2", "lk2")})
            if mx.get("kv_from") is None:
                out.update({m + "k": (G * 2 * D, W), m + "k.b": (G * 2 * D,), m + "k.norm": (D,), m + "v": (G * vd, W), m + "v.b": (G * vd,)})
        if not mlp:
            continue
        out[p + "norm2"] = (W,)
        f = p + "mlp."
        if mlp["kind"] == "dense":
            out.update({f + "up": (int(mlp["ff"]), W), f + "down": (W, int(mlp["ff"]))})
            continue
        E, ff, ident = int(mlp["router"]["experts"]), int(mlp["expert"]["ff"]), int(mlp["router"].get("identity") or 0)
        out.update({f + "router": (E + ident, W), f + "correction": (E + ident,)})
        for e in range(E):
            out.update({"%se%d.gate" % (f, e): (ff, W), "%se%d.up" % (f, e): (ff, W), "%se%d.down" % (f, e): (W, ff)})
        if mlp.get("shared"):
            sf = int(mlp["shared"]["ff"])
            out.update({f + "shared.gate": (sf, W), f + "shared.up": (sf, W), f + "shared.down": (W, sf)})
    return out


def random_tensors(cfg, seed, rank=6, steady=False):
    """bfloat16-representable float32 tensors: projections ~ N(0, 1.5 / sqrt(fan in)), norm weights around zero (the layers' own) or one, shift
    mixes between 0 and 1, decays between a few tokens and hundreds, a correction large enough to move the choice.  steady: the correction
    outweighs the scores' spread, so that few tokens stand before a close call (a 16-bit model's rounding then turns few choices)"""
    rg = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, rank).items():
        last = name.split(".")[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            a = 0.2 * rg.standard_normal(shape)
        elif last == "norm":
            a = 1.0 + 0.2 * rg.standard_normal(shape)
        elif ".mu." in name:
            a = rg.random(shape)
        elif last == "w0":
            a = -3.0 + 2.0 * rg.standard_normal(shape)
        elif last == "u":
            a = 0.5 + 0.5 * rg.standard_normal(shape)
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            a = 0.5 * rg.standard_normal(shape) / math.sqrt(math.sqrt(shape[0]))
        elif last == "b":
            a = 0.3 * rg.standard_normal(shape)
        elif last == "correction":
            a = (0.5 if steady else 0.1) * rg.standard_normal(shape)
        elif last == "embed":
            a = rg.standard_normal(shape)
        elif last == "router":
            a = (0.3 if steady else 1.5) * rg.standard_normal(shape) / math.sqrt(shape[-1])
        else:
            a = 1.5 * rg.standard_normal(shape) / math.sqrt(shape[-1])
        out[name] = bf16_round(np.asarray(a, np.float32))
    return out
