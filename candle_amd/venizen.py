"""The Venizen decoder: talking-head attention beside retention, and the generalized delta rule, with a range of layers that runs several times on the same
weights (each run with its own cache and state), the embedding output added before every run but the first.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from . import decoder, mixers


class Config(decoder.Config):
    MIXERS = {"parallel": mixers.Parallel, "general_delta": mixers.GeneralDelta}
    FEED_FORWARDS = {"dense": mixers.PolyFeedForward}

    @classmethod
    def layer_runs(cls, d: dict) -> List[tuple]:
        n, loop = len(d["layers"]), d.get("loop")
        order = [(i, False) for i in range(n)]
        if loop:
            start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
            if not 0 <= start < stop <= n or times < 1:
                raise ValueError(f"loop {loop} does not fit {n} layers")
            again = [(i, i == start) for i in range(start, stop)]
            order = order[:stop] + again * (times - 1) + order[stop:]
        return order


def tensor_shapes(cfg: Config) -> Dict[str, tuple]:
    """{name: shape} of the checkpoint a configuration describes.  The rank of a delta mixer's decay is the tensors' own choice: a quarter of
    its head size here, at least 16."""
    w = cfg.width
    out = {"embed": (cfg.vocab, w), "final.norm": (w,), "head": (cfg.vocab, w)}
    for i, layer in enumerate(cfg.layers):
        pre, m = f"l{i}.", layer["mixer"]
        out[pre + "norm1"] = (w,)
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, d, e = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            out.update({pre + "mix.left." + n: s for n, s in (("q", (H * d, w)), ("k", (G * d, w)), ("v", (G * e, w)), ("q.norm", (d,)), ("k.norm", (d,)),
                                                              ("talk", (H, H)), ("o", (w, H * e)))})
            d, e = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            out.update({pre + "mix.right." + n: s for n, s in (("q", (d, w)), ("k", (d, w)), ("v", (e, w)), ("g", (e, w)), ("o", (w, e)))})
        else:
            d, rank = m["heads"] * m["dim"], max(16, m["dim"] // 4)
            out.update({pre + "mix." + n: (d, w) for n in "rkvga"})
            out.update({pre + "mix." + n: s for n, s in (("a.b", (d,)), ("w0", (d,)), ("norm", (d,)), ("w1", (rank, w)), ("w2", (d, rank)), ("o", (w, d)))})
        if layer.get("mlp"):
            ff = layer["mlp"]["ff"]
            out.update({pre + "norm2": (w,), pre + "mlp.up": (ff, w), pre + "mlp.down": (w, ff), pre + "mlp.act": (4,)})
    return out


class Model(decoder.Decoder):
    CONFIG = Config
    NORM = mixers.RmsNorm
    tensor_shapes = staticmethod(tensor_shapes)

    @classmethod
    def random_vector(cls, name: str, n: int) -> torch.Tensor:
        return torch.tensor([0.7, 0.2, 0.1, 0.0]) if name.endswith("act") else torch.ones(n)
