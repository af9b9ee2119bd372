"""Float64 numpy statement of the Pesivik design: one function per mechanism, a whole sequence at a time, keys and values up-projected, no
cache, no pages, no absorbed projections, experts one token at a time.  Shares no code with the product path; the tests compare the engine
with it.

A model is (cfg, w): cfg the dict of a config.json of the design, w a dict tensor name -> array.

Notation: x residual stream [T, width], positions 0 .. T-1, N a layer norm with a weight; a layer is
    x <- x + s1 * N(mixer(N(x))),   x <- x + s2 * N(ff(N(x)))        (s1, s2: one factor per channel)
"""
import math

import numpy as np


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * np.asarray(z, np.float64)))


_erf = np.vectorize(math.erf, otypes=[np.float64])


def gelu_erf(z):
    """z times the normal distribution function of z"""
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def layer_norm(x, weight, eps):
    """the row's mean is taken off, then the row is divided by its standard deviation; a weight, no offset"""
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * weight


def rms_norm(x, weight, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * weight


# ------------------------------------------------------------------------------------------------ latent attention
def rotate_half(x, positions, base):
    """x [T, ..., n]: dimension i turns with dimension i + n/2 by the angle p * base^(-2i/n)"""
    n = x.shape[-1]
    if n == 0:
        return x
    f = float(base) ** (-2.0 * np.arange(n // 2) / n)
    a = np.asarray(positions, np.float64)[:, None] * f[None, :]
    a = a.reshape((x.shape[0],) + (1,) * (x.ndim - 2) + (n // 2,))
    u, v = x[..., :n // 2], x[..., n // 2:]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)], -1)


def in_window(query_positions, n_keys, size):
    """[Tq, n_keys] bool: the query's own position and the size - 1 before it"""
    d = np.asarray(query_positions)[:, None] - np.arange(n_keys)[None, :]
    return (d >= 0) & (d < size)


def softmax_over_visible(scores, vis):
    """scores [..., Tq, Tk] -> weights; invisible keys weigh nothing"""
    s = np.where(vis, scores, -np.inf)
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def windowed_attention(q, k, v, scale, vis):
    """q [Tq, H, D], k [Tk, H, D], v [Tk, H, V] -> [Tq, H, V]"""
    return np.stack([softmax_over_visible((q[:, h] @ k[:, h].T) * scale, vis) @ v[:, h] for h in range(q.shape[1])], 1)


def latent_attention(h, mx, w, p, eps):
    T = h.shape[0]
    H, dim, rd, vdim, kr = (int(mx[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    pos = np.arange(T)
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(T, H, dim + rd)
    down = h @ w[p + "dkv"].T
    c = rms_norm(down[:, :kr], w[p + "dkv.norm"], eps)
    base = mx["rot"]["base"]
    k_rot = rotate_half(down[:, kr:], pos, base)
    q = np.concatenate([q[..., :dim], rotate_half(q[..., dim:], pos, base)], -1)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, dim), np.repeat(k_rot[:, None, :], H, 1)], -1)
    v = (c @ w[p + "uv"].T).reshape(T, H, vdim)
    out = windowed_attention(q, k, v, float(mx["scale"]), in_window(pos, T, int(mx["mask"]["size"])))
    out = out * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return out.reshape(T, H * vdim) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def keep_best_groups(choice, count, keep):
    """choice [n] -> the same with every entry outside the `keep` best groups at -inf; a group's worth is the sum of its two largest entries"""
    g = choice.reshape(count, -1)
    worth = np.sort(g, axis=1)[:, ::-1][:, :2].sum(1)
    best = np.argsort(-worth, kind="stable")[:keep]
    out = np.full_like(g, -np.inf)
    out[best] = g[best]
    return out.reshape(-1)


def route(h, router, w, p):
    """-> (chosen [T, top], weights [T, top]): sigmoid scores; a correction takes part in the choice (and in the groups' worth) and not in the
    weights, which are the chosen scores divided by their sum"""
    s = sigmoid(h @ w[p + "router"].T)
    choice = s + w[p + "correction"]
    groups = router.get("groups")
    if groups:
        choice = np.stack([keep_best_groups(c, int(groups["count"]), int(groups["keep"])) for c in choice])
    chosen = np.argsort(-choice, axis=-1, kind="stable")[:, :int(router["top"])]
    wt = np.take_along_axis(s, chosen, -1)
    return chosen, wt / (wt.sum(-1, keepdims=True) + 1e-20)


def two_matrix_ff(h, w, p):
    return gelu_erf(h @ w[p + "up"].T) @ w[p + "down"].T


def mixture(h, mlp, w, p):
    chosen, wt = route(h, mlp["router"], w, p)
    out = np.zeros_like(h)
    for e in range(int(mlp["router"]["experts"])):
        hit = chosen == e
        rows = np.nonzero(hit.any(-1))[0]
        if len(rows):
            out[rows] += (wt * hit).sum(-1)[rows, None] * two_matrix_ff(h[rows], w, "%se%d." % (p, e))
    if mlp.get("shared"):
        out = out + two_matrix_ff(h, w, p + "shared.")
    return out


# ------------------------------------------------------------------------------------------------ the model
def forward(cfg, w, tokens, return_layers=False):
    """-> logits [T, vocab] (and the residual stream after every layer [L, T, width])"""
    eps = float(cfg["norm"]["eps"])
    w = {k: np.asarray(v, np.float64) for k, v in w.items()}
    x = w["embed"][np.asarray(tokens)] * float(cfg["embedding"]["scale"])
    trace = []
    for i, layer in enumerate(cfg["layers"]):
        j = i
        while cfg["layers"][j].get("weights_of") is not None:
            j = int(cfg["layers"][j]["weights_of"])
        p = "l%d." % j
        m = latent_attention(layer_norm(x, w[p + "norm1"], eps), layer["mixer"], w, p + "mix.", eps)
        x = x + layer_norm(m, w[p + "norm1b"], eps) * w[p + "ls1"]
        if layer.get("mlp"):
            f = mixture(layer_norm(x, w[p + "norm2"], eps), layer["mlp"], w, p + "mlp.")
            x = x + layer_norm(f, w[p + "norm2b"], eps) * w[p + "ls2"]
        trace.append(x.copy())
    logits = layer_norm(x, w["final.norm"], eps) @ w["head"].T
    cap = cfg.get("logit_softcap")
    if cap:
        logits = float(cap) * np.tanh(logits / float(cap))
    return (logits, np.stack(trace)) if return_layers else logits


# ------------------------------------------------------------------------------------------------ random models for the tests
def bf16_round(a):
    """float32 array rounded to bfloat16 (nearest even), returned as float32"""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    return (((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16).astype(np.uint32).view(np.float32).reshape(np.shape(a))


def tensor_shapes(cfg):
    W, V = int(cfg["width"]), int(cfg["vocab"])
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, mx, mlp = "l%d." % i, layer["mixer"], layer.get("mlp")
        H, dim, rd, vdim, kr, qr = (int(mx[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
        out.update({p + "norm1": (W,), p + "norm1b": (W,), p + "ls1": (W,)})
        m = p + "mix."
        out.update({m + "dq": (qr, W), m + "dq.norm": (qr,), m + "uq": (H * (dim + rd), qr), m + "dkv": (kr + rd, W), m + "dkv.norm": (kr,),
                    m + "uk": (H * dim, kr), m + "uv": (H * vdim, kr), m + "g": (H, W), m + "o": (W, H * vdim)})
        if not mlp:
            continue
        out.update({p + "norm2": (W,), p + "norm2b": (W,), p + "ls2": (W,)})
        f, E, ff = p + "mlp.", int(mlp["router"]["experts"]), int(mlp["expert"]["ff"])
        out.update({f + "router": (E, W), f + "correction": (E,)})
        for e in range(E):
            out.update({"%se%d.up" % (f, e): (ff, W), "%se%d.down" % (f, e): (W, ff)})
        if mlp.get("shared"):
            sf = int(mlp["shared"]["ff"])
            out.update({f + "shared.up": (sf, W), f + "shared.down": (W, sf)})
    return out


def random_tensors(cfg, seed, steady=False):
    """bfloat16-representable float32 tensors: projections ~ N(0, 1.5 / sqrt(fan in)), norm weights around one, layer scales spread over both
    signs, corrections large enough to move the choice.  steady: the corrections outweigh the scores' spread, so that few tokens stand before a
    close call (a 16-bit model's rounding then turns few choices)"""
    r = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.split(".")[-1]
        if last in ("norm1", "norm1b", "norm2", "norm2b", "norm"):
            a = 1.0 + 0.2 * r.standard_normal(shape)
        elif last in ("ls1", "ls2"):
            a = 0.7 + 0.5 * r.standard_normal(shape)
        elif last == "correction":
            a = (1.0 if steady else 0.5) * r.standard_normal(shape)
        elif last == "embed":
            a = r.standard_normal(shape) / float(cfg["embedding"]["scale"])
        elif last == "router":
            a = (0.4 if steady else 2.0) * r.standard_normal(shape) / math.sqrt(shape[-1])
        else:
            a = 1.5 * r.standard_normal(shape) / math.sqrt(shape[-1])
        out[name] = bf16_round(np.asarray(a, np.float32))
    return out
