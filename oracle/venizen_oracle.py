"""CPU restatement (numpy, float64) of the Venizen decoder, one function per mechanism, written straight from the
equations and without regard to speed.  TEST INFRASTRUCTURE ONLY: imported by tests/, never by the product path, with
which it shares no code.

Every function takes whole sequences (row t = position t) and knows no cache: the product's prompts cut into portions and
its token-by-token decoding are compared with one evaluation of the whole sequence here.

``forward`` returns the logits of every position, and the residual stream after every layer run when asked.  ``tensors`` is
``{name: array}`` with the checkpoint's names, ``cfg`` the parsed config.json.
"""
from __future__ import annotations

import numpy as np

f64 = np.float64


# ------------------------------------------------------------------------------------------------- small pieces
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def over_rms(z, eps):
    """z / sqrt(mean(z^2) + eps) over the last axis."""
    return z / np.sqrt(np.mean(z * z, axis=-1, keepdims=True) + eps)


def rms_norm(z, w, eps):
    return over_rms(z, eps) * w


def linear(w, z):
    """z [..., in] through a weight stored [out, in]."""
    return z @ w.T


def rotate_half(z, base, dims):
    """z [T, heads, dim]: dimension i < dims/2 turns with dimension i + dims/2 by the angle t * base^(-2 i / dims)."""
    out = z.copy()
    half = dims // 2
    t = np.arange(z.shape[0], dtype=f64)[:, None]
    ang = t * f64(base) ** (-2.0 * np.arange(half, dtype=f64) / dims)
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    u, v = z[..., :half], z[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def poly_norm(z, coef, eps):
    """Cubic without a constant, each power divided by the row's root mean square of that power, plus the last coefficient."""
    return sum(coef[n - 1] * over_rms(z ** n, eps) for n in (1, 2, 3)) + coef[3]


# ------------------------------------------------------------------------------------------------- attention
def window_mask(n, size, keep_first):
    """[n, n] bool: query i sees key j."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def talking_attention(q, k, v, talk, scale, mask):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e].  The scores of all heads are mixed by `talk` [H, H] before the softmax."""
    H, G = q.shape[1], k.shape[1]
    r = H // G
    s = np.stack([q[:, h] @ k[:, h // r].T for h in range(H)]) * scale          # [H, T, T]
    s = np.einsum("hg,gij->hij", talk, s)
    s = np.where(mask[None], s, -np.inf)
    s = s - s.max(axis=-1, keepdims=True)
    p = np.exp(s)
    p = p / p.sum(axis=-1, keepdims=True)
    return np.stack([p[h] @ v[:, h // r] for h in range(H)], axis=1)


def attention_mixer(h, t, pre, m, eps):
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(t[pre + "q"], h).reshape(T, H, d)
    k = linear(t[pre + "k"], h).reshape(T, G, d)
    v = linear(t[pre + "v"], h).reshape(T, G, e)
    q = rotate_half(rms_norm(q, t[pre + "q.norm"], eps), m["rot"]["base"], m["rot"]["dims"])
    k = rotate_half(rms_norm(k, t[pre + "k.norm"], eps), m["rot"]["base"], m["rot"]["dims"])
    mask = window_mask(T, m["mask"]["size"], m["mask"]["keep_first"])
    o = talking_attention(q, k, v, t[pre + "talk"], m["scale"], mask)
    return linear(t[pre + "o"], o.reshape(T, H * e))


# ------------------------------------------------------------------------------------------------- retention
def retention(q, k, v, decay):
    """q, k [T, H, d], v [T, H, e], decay [H] -> [T, H, e]: S <- decay S + k v^T, o = S^T q, token by token."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    out = np.empty((T, H, v.shape[2]))
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hde,hd->he", S, q[t])
    return out


def retention_mixer(h, t, pre, m, eps):
    T, H, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = rotate_half(linear(t[pre + "q"], h).reshape(T, H, d), m["rot"]["base"], m["rot"]["dims"])
    k = rotate_half(linear(t[pre + "k"], h).reshape(T, H, d), m["rot"]["base"], m["rot"]["dims"]) * f64(d) ** -0.5
    v = linear(t[pre + "v"], h).reshape(T, H, e)
    o = over_rms(retention(q, k, v, np.asarray(m["decay"], f64)), eps).reshape(T, H * e)
    return linear(t[pre + "o"], o * silu(linear(t[pre + "g"], h)))


# ------------------------------------------------------------------------------------------------- generalized delta rule
def general_delta(r, k, v, w, a):
    """All [T, H, d]: S <- (diag(w) - (a u) u^T) S + k v^T with u the unit key, o = S^T r, token by token."""
    T, H, d = r.shape
    u = k / np.sqrt(np.sum(k * k, axis=-1, keepdims=True) + 1e-6)
    S = np.zeros((H, d, d))
    out = np.empty((T, H, d))
    for t in range(T):
        uS = np.einsum("hi,hij->hj", u[t], S)
        S = w[t][:, :, None] * S - (a[t] * u[t])[:, :, None] * uS[:, None, :] + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hij,hi->hj", S, r[t])
    return out


def general_delta_mixer(h, t, pre, m, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    heads = lambda z: z.reshape(T, H, d)
    r, k, v = (heads(linear(t[pre + n], h)) for n in "rkv")
    low = np.tanh(linear(t[pre + "w1"], h))
    w = heads(np.exp(-np.exp(-0.5) * sigmoid(linear(t[pre + "w2"], low) + t[pre + "w0"])))
    a = heads(sigmoid(linear(t[pre + "a"], h) + t[pre + "a.b"]))
    o = over_rms(general_delta(r, k, v, w, a), eps).reshape(T, H * d)
    return linear(t[pre + "o"], o * t[pre + "norm"] * sigmoid(linear(t[pre + "g"], h)))


# ------------------------------------------------------------------------------------------------- the model
def mixer(h, t, pre, layer, eps):
    m = layer["mixer"]
    if layer["type"] == "parallel":
        return m["left_scale"] * attention_mixer(h, t, pre + "left.", m["left"], eps) + \
            m["right_scale"] * retention_mixer(h, t, pre + "right.", m["right"], eps)
    if layer["type"] == "general_delta":
        return general_delta_mixer(h, t, pre, m, eps)
    raise ValueError(layer["type"])


def feed_forward(h, t, pre, eps):
    return linear(t[pre + "down"], poly_norm(linear(t[pre + "up"], h), t[pre + "act"], eps))


def layer_order(cfg):
    """[(layer index, embedding output added before it)] in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(loop["start"])]
    for p in range(loop["times"]):
        order += [(i, p > 0 and i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg, tensors, tokens, return_layers=False):
    t = {n: np.asarray(a, f64) for n, a in tensors.items()}
    eps = cfg["norm"]["eps"]
    emb = t["embed"][np.asarray(tokens)]
    x, runs = emb, []
    for i, again in layer_order(cfg):
        if again:
            x = x + emb
        layer, pre = cfg["layers"][i], f"l{i}."
        x = x + mixer(rms_norm(x, t[pre + "norm1"], eps), t, pre + "mix.", layer, eps)
        if layer.get("mlp") is not None:
            x = x + feed_forward(rms_norm(x, t[pre + "norm2"], eps), t, pre + "mlp.", eps)
        runs.append(x)
    logits = linear(t["head"], rms_norm(x, t["final.norm"], eps))
    return (logits, np.stack(runs)) if return_layers else logits
