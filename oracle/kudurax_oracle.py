"""CPU restatement (numpy, float64) of the Kudurax decoder, one function per mechanism, written straight from the equations
and without regard to speed.  TEST INFRASTRUCTURE ONLY: imported by tests/, never by the product path, with which it shares
no code.

Every function takes whole sequences (row t = position t) and knows no cache: the product's prompts cut into portions and
its token-by-token decoding are compared with one evaluation of the whole sequence here.

``forward`` returns the logits of every position, and the residual stream after every layer when asked.  ``tensors`` is
``{name: array}`` with the checkpoint's names, ``cfg`` the parsed config.json.
"""
from __future__ import annotations

import math

import numpy as np

f64 = np.float64


# ------------------------------------------------------------------------------------------------- small pieces
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def relu_squared(z):
    return np.maximum(z, 0.0) ** 2


def softmax(z):
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def linear(w, z):
    """z [..., in] through a weight stored [out, in]."""
    return z @ w.T


def layer_norm(z, w, b, eps):
    c = z - z.mean(axis=-1, keepdims=True)
    return c / np.sqrt((c * c).mean(axis=-1, keepdims=True) + eps) * w + b


def rms_norm(z, w, eps):
    return z / np.sqrt((z * z).mean(axis=-1, keepdims=True) + eps) * w


# ------------------------------------------------------------------------------------------------- rotation
def frequencies(rot):
    """(angle per position of each pair, factor on cos and sin)."""
    dims, base = rot["dims"], f64(rot["base"])
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def turns_at(t):                     # the (fractional) dimension whose pair turns t times over the original length
        return dims * math.log(s["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(turns_at(s["fast"])), 0), min(math.ceil(turns_at(s["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / s["factor"] * ramp + fi * (1.0 - ramp))
    return np.array(out), 0.1 * math.log(s["factor"]) + 1.0


def rotate_pairs(z, rot):
    """z [T, heads, dim]: dimensions 2i and 2i + 1 of the first rot.dims turn together, row t by t times the pair's frequency."""
    f, m = frequencies(rot)
    out = z.copy()
    for t in range(z.shape[0]):
        c, s = m * np.cos(t * f), m * np.sin(t * f)
        u, v = z[t, :, 0:rot["dims"]:2], z[t, :, 1:rot["dims"]:2]
        out[t, :, 0:rot["dims"]:2] = u * c - v * s
        out[t, :, 1:rot["dims"]:2] = v * c + u * s
    return out


# ------------------------------------------------------------------------------------------------- latent attention
def latents(h, t, pre, m, eps):
    """What a layer with its own down projection caches: the normed latent [T, rank] and the rotated key part [T, rot_dim]."""
    z = linear(t[pre + "dkv"], h)
    c = rms_norm(z[:, :m["kv_rank"]], t[pre + "dkv.norm"], eps)
    return c, rotate_pairs(z[:, None, m["kv_rank"]:], m["rot"])[:, 0]


def causal_attention(q, k, v, scale):
    """q, k [T, H, d], v [T, H, e] -> [T, H, e]."""
    T, H = q.shape[:2]
    out = np.empty((T, H, v.shape[2]))
    for h in range(H):
        s = scale * (q[:, h] @ k[:, h].T)
        s[np.triu_indices(T, 1)] = -np.inf
        out[:, h] = softmax(s) @ v[:, h]
    return out


def latent_attention(h, t, pre, m, kept):
    """`kept`: the (latent, rotated key part) this layer attends to."""
    T, H, d, r, e = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = kept
    q = linear(t[pre + "q"], h).reshape(T, H, d + r)
    q = np.concatenate([q[..., :d], rotate_pairs(q[..., d:], m["rot"])], axis=-1)
    k = linear(t[pre + "uk"], c).reshape(T, H, d)
    k = np.concatenate([k, np.repeat(kr[:, None], H, axis=1)], axis=-1)
    v = linear(t[pre + "uv"], c).reshape(T, H, e)
    o = causal_attention(q, k, v, m["scale"]) * sigmoid(linear(t[pre + "g"], h))[..., None]
    return linear(t[pre + "o"], o.reshape(T, H * e))


# ------------------------------------------------------------------------------------------------- feed-forward
def gated(h, t, pre):
    return linear(t[pre + "down"], silu(linear(t[pre + "gate"], h)) * linear(t[pre + "up"], h))


def route(z, top):
    """Router logits [T, E] -> chosen experts [T, top] and their weights (softmax over the chosen only)."""
    ids = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    return ids, softmax(np.take_along_axis(z, ids, axis=-1))


def mixture(h, t, pre, mlp):
    ids, w = route(linear(t[pre + "router"], h), mlp["router"]["top"])
    out = np.zeros_like(h)
    for i in range(h.shape[0]):
        for e, a in zip(ids[i], w[i]):
            out[i] += a * gated(h[i], t, f"{pre}e{e}.")
    if mlp.get("shared"):
        out += sigmoid(linear(t[pre + "shared.sg"], h)) * gated(h, t, pre + "shared.")
    return out


def feed_forward(h, t, pre, mlp):
    if mlp["kind"] == "dense":
        return linear(t[pre + "down"], relu_squared(linear(t[pre + "up"], h)))
    return mixture(h, t, pre, mlp)


# ------------------------------------------------------------------------------------------------- the model
def forward(cfg, tensors, tokens, return_layers=False):
    t = {n: np.asarray(a, f64) for n, a in tensors.items()}
    eps = cfg["norm"]["eps"]
    norm = lambda z, name: layer_norm(z, t[name], t[name + ".b"], eps)
    x = t["embed"][np.asarray(tokens)] * f64(cfg["embedding"]["scale"])
    kept, runs = {}, []
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        h = norm(x, pre + "norm1")
        source = m.get("kv_from")
        if source is None:
            kept[i] = latents(h, t, pre + "mix.", m, eps)
        x = x + latent_attention(h, t, pre + "mix.", m, kept[i if source is None else source])
        if layer.get("mlp") is not None:
            x = x + feed_forward(norm(x, pre + "norm2"), t, pre + "mlp.", layer["mlp"])
        runs.append(x)
    logits = linear(t["head"], norm(x, "final.norm"))
    return (logits, np.stack(runs)) if return_layers else logits
