"""Small Venizen configurations, random checkpoints for them, and a writer of the checkpoint files (used by the CPU and GPU tests)."""
import json
import os
import struct

import numpy as np


def bf16(a):
    """Round f32 to the nearest bfloat16 value, as f32."""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    u = (u + 0x7fff + ((u >> 16) & 1)) & 0xffff0000
    return u.astype(np.uint32).view(np.float32).reshape(np.shape(a))


def parallel(left, right, ff=None, scales=(1.0, 1.0)):
    H, G, d, e, scale, window, keep, base, dims = left
    h2, d2, e2, decay, base2, dims2 = right
    return {"type": "parallel",
            "mixer": {"left": {"heads": H, "kv_heads": G, "dim": d, "vdim": e, "scale": scale, "mask": {"size": window, "keep_first": keep}, "rot": {"base": base, "dims": dims}},
                      "right": {"heads": h2, "dim": d2, "vdim": e2, "decay": list(decay), "rot": {"base": base2, "dims": dims2}},
                      "left_scale": scales[0], "right_scale": scales[1]},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads, dim, ff=None):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(vocab, width, layers, loop=None, eps=1e-5):
    return {"architecture": "Venizen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "loop": loop}


# name -> configuration.  Sizes that are no multiples of each other, key and value sizes that differ, one kv head and as many kv heads as
# heads, partial and full rotation, no kept tokens, a window of one, feed-forwards where the other mixer has none, loops at either end.
CONFIGS = {
    "mixed": config(101, 72, [
        parallel((6, 2, 40, 24, 0.21, 9, 3, 10000.0, 20), (3, 24, 40, (0.9, 0.97, 0.995), 5000.0, 12), 88, (0.8, 1.3)),
        delta(3, 20),
        delta(2, 36, 56),
        parallel((4, 4, 16, 32, 0.3, 24, 0, 300000.0, 16), (1, 16, 16, (0.99,), 100.0, 16), None, (1.1, 0.7))],
        {"start": 1, "stop": 3, "times": 2}, 1e-5),
    "wide": config(160, 136, [
        delta(4, 32),
        parallel((12, 3, 64, 80, 0.11, 33, 7, 2000.0, 32), (2, 72, 96, (0.95, 0.999), 10000.0, 72), 200)],
        {"start": 0, "stop": 2, "times": 3}, 3e-6),
    "one": config(64, 48, [parallel((5, 1, 8, 8, 0.5, 1, 2, 50.0, 4), (2, 8, 24, (0.5, 0.75), 50.0, 4), 40, (1.0, 0.5))], None, 1e-4),
    "plain": config(90, 66, [delta(1, 66, 70), parallel((18, 6, 12, 20, 0.25, 40, 5, 10000.0, 12), (4, 12, 12, (0.8, 0.9, 0.95, 0.99), 10000.0, 8), 30)], None, 1e-5),
}


def shapes(cfg, rank=11):
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w), "final.norm": (w,)}
    for i, la in enumerate(cfg["layers"]):
        p, m = f"l{i}.", la["mixer"]
        out[p + "norm1"] = (w,)
        if la["type"] == "parallel":
            a, r = m["left"], m["right"]
            out[p + "mix.left.q"] = (a["heads"] * a["dim"], w)
            out[p + "mix.left.k"] = (a["kv_heads"] * a["dim"], w)
            out[p + "mix.left.v"] = (a["kv_heads"] * a["vdim"], w)
            out[p + "mix.left.q.norm"] = out[p + "mix.left.k.norm"] = (a["dim"],)
            out[p + "mix.left.talk"] = (a["heads"], a["heads"])
            out[p + "mix.left.o"] = (w, a["heads"] * a["vdim"])
            for n, s in (("q", r["dim"]), ("k", r["dim"]), ("v", r["vdim"]), ("g", r["vdim"])):
                out[p + "mix.right." + n] = (r["heads"] * s, w)
            out[p + "mix.right.o"] = (w, r["heads"] * r["vdim"])
        else:
            d = m["heads"] * m["dim"]
            for n in "rkvga":
                out[p + "mix." + n] = (d, w)
            for n in ("a.b", "w0", "norm"):
                out[p + "mix." + n] = (d,)
            out[p + "mix.w1"], out[p + "mix.w2"], out[p + "mix.o"] = (rank, w), (d, rank), (w, d)
        if la.get("mlp"):
            ff = la["mlp"]["ff"]
            out[p + "norm2"], out[p + "mlp.up"], out[p + "mlp.down"], out[p + "mlp.act"] = (w,), (ff, w), (w, ff), (4,)
    return out


def tensors(cfg, seed):
    """bf16 values as f32 arrays.  Queries and keys are made large enough for attention to be selective, head mixing far from the identity,
    decay and removal rates spread over their range."""
    rng = np.random.Generator(np.random.PCG64(seed))
    out = {}
    for name, s in shapes(cfg).items():
        z = rng.standard_normal(s, dtype=np.float32)
        if name == "embed":
            a = z
        elif name.endswith("talk"):
            a = np.eye(s[0], dtype=np.float32) * 0.7 + z * 0.5
        elif name.endswith(("q.norm", "k.norm")):
            a = 1.5 + 0.3 * z
        elif name.endswith("act"):
            a = np.array([0.6, -0.4, 0.3, 0.15], dtype=np.float32)
        elif name.endswith(("w0", "a.b")):
            a = 1.5 * z
        elif name.endswith("w2"):
            a = z * 0.7
        elif len(s) == 1:
            a = 1.0 + 0.25 * z
        else:
            a = z / np.sqrt(s[1])
        out[name] = bf16(a)
    return out


def write_checkpoint(path, cfg, ts):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {"__metadata__": {"format": "pt"}}, [], 0
    for name, a in ts.items():
        b = (np.ascontiguousarray(a, dtype=np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        header[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    head = json.dumps(header).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + b"".join(blobs))


def token_ids(cfg, n, seed):
    return np.random.Generator(np.random.PCG64(seed)).integers(0, cfg["vocab"], n).tolist()


def error(got, want):
    """Largest over the positions of rms(difference) / rms(all logits)."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    return float(np.sqrt(((got - want) ** 2).mean(axis=-1)).max() / np.sqrt((want ** 2).mean()))
