"""The Kudurax decoder: attention over cached latents, some layers attending to the cache of an earlier one, with YaRN-scaled rotary positions and gated heads;
squared-relu feed-forwards and mixtures of gated experts; layer norms with a bias; a factor on the embedding.
"""
from __future__ import annotations

from typing import Dict

import torch

from . import decoder, mixers


class Config(decoder.Config):
    MIXERS = {"latent_attention": mixers.LatentAttention}
    FEED_FORWARDS = {"dense": mixers.ReluSquaredFeedForward, "moe": mixers.GatedExperts}

    @classmethod
    def from_dict(cls, d: dict, ctx: int = 4096) -> "Config":
        for i, layer in enumerate(d["layers"]):
            source = layer["mixer"].get("kv_from")
            if source is None:
                continue
            if not 0 <= source < i or d["layers"][source]["mixer"].get("kv_from") is not None:
                raise ValueError(f"layer {i}: layer {source} has no latents of its own before it")
            if any(layer["mixer"][k] != d["layers"][source]["mixer"][k] for k in ("kv_rank", "rot_dim", "rot")):
                raise ValueError(f"layer {i}: its latents differ in size or rotation from those of layer {source}")
        return super().from_dict(d, ctx)


def tensor_shapes(cfg: decoder.Config) -> Dict[str, tuple]:
    """{name: shape} of the checkpoint a configuration describes."""
    w = cfg.width
    out = {"embed": (cfg.vocab, w), "head": (cfg.vocab, w)}

    def norm(name):
        out[name] = out[name + ".b"] = (w,)
    norm("final.norm")
    for i, layer in enumerate(cfg.layers):
        pre, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        H, d, t, e, r = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        norm(pre + "norm1")
        out.update({pre + "mix." + n: s for n, s in (("q", (H * (d + t), w)), ("uk", (H * d, r)), ("uv", (H * e, r)), ("g", (H, w)), ("o", (w, H * e)))})
        if m.get("kv_from") is None:
            out.update({pre + "mix.dkv": (r + t, w), pre + "mix.dkv.norm": (r,)})
        if not mlp:
            continue
        norm(pre + "norm2")
        if mlp["kind"] == "dense":
            out.update({pre + "mlp.up": (mlp["ff"], w), pre + "mlp.down": (w, mlp["ff"])})
            continue
        gated = lambda name, ff: out.update({f"{name}.gate": (ff, w), f"{name}.up": (ff, w), f"{name}.down": (w, ff)})
        out[pre + "mlp.router"] = (mlp["router"]["experts"], w)
        for x in range(mlp["router"]["experts"]):
            gated(f"{pre}mlp.e{x}", mlp["expert"]["ff"])
        if mlp.get("shared"):
            gated(pre + "mlp.shared", mlp["shared"]["ff"])
            out[pre + "mlp.shared.sg"] = (1, w)
    return out


class Model(decoder.Decoder):
    CONFIG = Config
    NORM = mixers.LayerNorm
    tensor_shapes = staticmethod(tensor_shapes)

    @classmethod
    def random_vector(cls, name: str, n: int) -> torch.Tensor:
        return torch.zeros(n) if name.endswith(".b") else torch.ones(n)
