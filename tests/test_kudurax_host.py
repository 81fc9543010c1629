"""CPU tests around the Kudurax decoder: the oracle against independent formulations of its mechanisms, the sensitivity of the test configurations to small
mistakes, rotation tables, configuration reading, argument checks of the entry points."""
import copy
import ctypes
import math

import numpy as np
import pytest
import torch

from candle_amd import _lib, mixers
from candle_amd.cache import SequenceCache
from candle_amd.kudurax import Config
from oracle import kudurax_oracle as ko
from tests import kudurax_cases as kc


def rnd(seed, *shape):
    return np.random.Generator(np.random.PCG64(seed)).standard_normal(shape)


# ---------------------------------------------------------------------------------------------- oracle against other formulations
def test_attention_over_latents_equals_attention_with_absorbed_matrices():
    T, H, d, r, e, rank = 9, 3, 6, 4, 5, 7
    m = {"heads": H, "dim": d, "rot_dim": r, "vdim": e, "kv_rank": rank, "scale": 0.3, "rot": kc.rot(r, 100.0)}
    w = 11
    t = {"q": rnd(1, H * (d + r), w), "uk": rnd(2, H * d, rank), "uv": rnd(3, H * e, rank), "g": rnd(4, H, w), "o": rnd(5, w, H * e)}
    h, c, kr = rnd(6, T, w), rnd(7, T, rank), rnd(8, T, r)
    got = ko.latent_attention(h, t, "", m, (c, kr))
    q = (h @ t["q"].T).reshape(T, H, d + r)
    qr = ko.rotate_pairs(q[..., d:], m["rot"])
    for i in range(T):
        out = []
        for a in range(H):
            lat = t["uk"][a * d:(a + 1) * d].T @ q[i, a, :d]                     # the key matrix applied to the query
            s = np.exp(0.3 * (c[:i + 1] @ lat + kr[:i + 1] @ qr[i, a]))
            o = t["uv"][a * e:(a + 1) * e] @ (s @ c[:i + 1] / s.sum())
            out.append(o / (1.0 + np.exp(-(t["g"][a] @ h[i]))))
        assert np.allclose(got[i], t["o"] @ np.concatenate(out))


def test_rotation_pairs_neighbours_and_depends_on_distance_only():
    rot = kc.rot(8, 50.0, None)
    z = np.repeat(rnd(1, 1, 2, 10), 20, axis=0)
    y = ko.rotate_pairs(z, rot)
    assert np.allclose(y[..., 8:], z[..., 8:])
    f = 50.0 ** (-2.0 / 8)                                                       # dimensions 2 and 3 are the second pair
    assert np.allclose(y[3, 0, 3], z[3, 0, 3] * math.cos(3 * f) + z[3, 0, 2] * math.sin(3 * f))
    dots = y[:, 0] @ y[:, 0].T
    assert np.allclose(dots[3, 1], dots[17, 15]) and np.allclose(dots[9, 2], dots[19, 12])


@pytest.mark.parametrize("dims,base,scaling", [
    (10, 10000.0, (4.0, 32.0, 1.0, 64)), (64, 1e6, (40.0, 32.0, 1.0, 4096)), (16, 300.0, (2.0, 8.0, 2.0, 40)), (2, 50.0, (3.0, 32.0, 1.0, 16)),
    (32, 10000.0, (8.0, 2.0, 2.0, 100)), (24, 500.0, (1.0, 32.0, 1.0, 2048)), (12, 10000.0, (16.0, 1e9, 1e-9, 64)), (20, 777.0, None)])
def test_rotation_tables_equal_the_oracle(dims, base, scaling):
    rot = kc.rot(dims, base, scaling)
    f, m = ko.frequencies(rot)
    got, factor = mixers.frequencies(base, dims, rot.get("scaling"))
    assert np.allclose(got, f, rtol=1e-14) and factor == pytest.approx(m, rel=1e-15)
    if scaling:
        assert factor == pytest.approx(0.1 * math.log(scaling[0]) + 1.0) and f[-1] >= base ** (-2.0 * (dims // 2 - 1) / dims) / scaling[0] * (1 - 1e-12)


def test_route_takes_the_largest_and_weighs_the_chosen_only():
    ids, w = ko.route(np.array([[0.0, 3.0, -1.0, 3.0, 2.0]]), 3)
    assert ids.tolist() == [[1, 3, 4]]
    e = np.exp([3.0, 3.0, 2.0])
    assert np.allclose(w[0], e / e.sum())


def test_layer_norm_known_values():
    y = ko.layer_norm(np.array([[1.0, 3.0]]), np.array([2.0, 2.0]), np.array([0.5, 0.0]), 3.0)
    assert np.allclose(y, [[-0.5, 1.0]])


# ---------------------------------------------------------------------------------------------- the configurations show small mistakes
def _mutations(cfg, ts):
    """(what, configuration, tensors) that a typical mistake would compute instead."""
    def edit(f):
        c = copy.deepcopy(cfg)
        f(c)
        return c

    def each_rot(f):
        def g(c):
            for la in c["layers"]:
                f(la["mixer"]["rot"])
        return g
    L = cfg["layers"]
    if any("scaling" in la["mixer"]["rot"] for la in L):
        yield "no frequency scaling", edit(each_rot(lambda r: r.pop("scaling", None))), ts
        yield "scaling of cos and sin also on the scale", edit(lambda c: [la["mixer"].update(scale=la["mixer"]["scale"] * (0.1 * math.log(4.0) + 1.0) ** 2)
                                                                         for la in c["layers"]]), ts
    if any(la["mixer"].get("kv_from") == 0 for la in L) and sum(la["mixer"].get("kv_from") is None and la["mixer"]["kv_rank"] == L[0]["mixer"]["kv_rank"] for la in L) > 1:
        yield "the nearest latents", edit(lambda c: c["layers"][-1]["mixer"].update(kv_from=2)), ts
    for i, la in enumerate(L):
        if la.get("mlp") and la["mlp"]["kind"] == "moe":
            if la["mlp"]["router"]["top"] > 1:
                yield "one expert fewer", edit(lambda c: c["layers"][i]["mlp"]["router"].update(top=la["mlp"]["router"]["top"] - 1)), ts
            if la["mlp"].get("shared"):
                yield "no shared expert", edit(lambda c: c["layers"][i]["mlp"].pop("shared")), ts
                yield "shared expert not gated", cfg, {n: a * 0 if n.endswith(f"l{i}.mlp.shared.sg") else a for n, a in ts.items()}
    yield "heads not gated", cfg, {n: a * 0 if n.endswith("mix.g") else a for n, a in ts.items()}
    yield "no norm bias", cfg, {n: a * 0 if n.endswith(".b") else a for n, a in ts.items()}
    yield "latents not weighted", cfg, {n: a * 0 + 1 if n.endswith("dkv.norm") else a for n, a in ts.items()}
    if cfg["embedding"]["scale"] != 1.0:
        yield "embedding not scaled", edit(lambda c: c["embedding"].update(scale=1.0)), ts


@pytest.mark.parametrize("name", sorted(kc.CONFIGS))
def test_small_mistakes_show(name):
    cfg = kc.CONFIGS[name]
    ts, ids = kc.tensors(cfg, 5), kc.token_ids(cfg, 60, 6)
    want = ko.forward(cfg, ts, ids)
    for what, other, tensors in _mutations(cfg, ts):
        assert kc.error(ko.forward(other, tensors, ids), want) > 0.005, what


def test_oracle_is_causal():
    cfg = kc.CONFIGS["mixed"]
    ts, ids = kc.tensors(cfg, 5), kc.token_ids(cfg, 40, 6)
    assert np.allclose(ko.forward(cfg, ts, ids)[:25], ko.forward(cfg, ts, ids[:25]))


# ---------------------------------------------------------------------------------------------- configuration, cache, entry points
def test_configuration_errors():
    def bad(f):
        c = copy.deepcopy(kc.CONFIGS["mixed"])
        f(c["layers"])
        return c
    for match, f in (("no latents of its own", lambda la: la[4]["mixer"].update(kv_from=1)), ("no latents of its own", lambda la: la[1]["mixer"].update(kv_from=2)),
                     ("no latents of its own", lambda la: la[2]["mixer"].update(kv_from=2)), ("differ in size", lambda la: la[4]["mixer"].update(kv_from=2)),
                     ("differ in size", lambda la: la[1]["mixer"].update(rot=kc.rot(10, 77.0))), ("unknown mixer", lambda la: la[0].update(type="nothing")),
                     ("unknown feed-forward", lambda la: la[0]["mlp"].update(kind="nothing"))):
        with pytest.raises(ValueError, match=match):
            Config.from_dict(bad(f))
    cfg = Config.from_dict(kc.CONFIGS["mixed"], 77)
    assert (cfg.vocab, cfg.width, cfg.ctx, cfg.embed_scale, cfg.order) == (101, 72, 77, 3.5, [(i, False) for i in range(5)])


def test_cache_rows_are_written_by_position():
    c = SequenceCache("cpu")
    r = c.add_rows(10, 12, torch.bfloat16)
    assert r.shape == (10, 12) and not r.any() and c.nbytes() == 240
    c.length = 7
    c.begin(3)                                    # no state that could not move back
    c.begin(0)
    assert c.length == 0


def _latent(**kw):
    f = dict(norm_dev=16, cos_dev=16, sin_dev=16, heads=4, dim=16, rot_dim=8, vdim=16, rank=32, rank_pad=64, rot_pad=8, ctx=100, bf16=1, scale=1.0, eps=1e-5)
    f.update(kw)
    return _lib.Latent(**f)


def test_argument_validation_codes_without_gpu():
    L = _lib.mixer_lib()
    OK, DTYPE, SHAPE, ALIGN, NULL, WS, RANGE = 0, -1, -2, -3, -4, -5, -6
    assert ctypes.sizeof(_lib.DenseArgs) == 9 * 8 + 13 * 8 + 16 and ctypes.sizeof(_lib.Latent) == 3 * 8 + 12 * 4 and ctypes.sizeof(_lib.Moe) == 6 * 8 + 8 * 4

    def product(precision=0, **kw):
        f = dict(w_dev=16, x_dev=16, dst_dev=16, ldw=64, ldx=64, ldd=8, m=4, n=8, k=64, batch=1)
        f.update(kw)
        return L.cq_dense_product(precision, _lib.DenseArgs(**f), None, 0, None)
    assert product(m=0) == OK and product(2) == DTYPE and product(1, x_bf16=1) == DTYPE and product(act=3) == DTYPE
    assert product(batch=0) == SHAPE and product(n=7, ldd=7, act=2) == SHAPE and product(act=1, accumulate=1) == SHAPE and product(dst_bf16=1, accumulate=1) == SHAPE
    assert product(batch=2, accumulate=1) == SHAPE and product(x_bf16=1, ldx=68) == SHAPE
    assert product(tiles_dev=16, n_tiles_dev=16, max_tiles=0, tile_rows=64) == SHAPE and product(tiles_dev=16, n_tiles_dev=16, max_tiles=1, tile_rows=48) == SHAPE
    assert product(1, tiles_dev=16, n_tiles_dev=16, max_tiles=1, tile_rows=32) == SHAPE and product(tiles_dev=16, max_tiles=1, tile_rows=64) == NULL
    assert product(w_dev=None) == NULL and product(x_dev=8) == ALIGN

    pack = lambda g, **kw: L.cq_mix_latent_pack(g, kw.get("row", 16), 200, kw.get("kv", 96), kw.get("cache", 16), None, 0, 16, kw.get("head", 24), 16, kw.get("pos", 0), 4, None)
    assert pack(_latent(heads=0)) == SHAPE and pack(_latent(rank_pad=48)) == SHAPE and pack(_latent(rot_dim=7)) == SHAPE and pack(_latent(rot_pad=12)) == SHAPE
    assert pack(_latent(cos_dev=None)) == NULL and pack(_latent(norm_dev=None)) == NULL and pack(_latent(), cache=None) == NULL
    assert pack(_latent(rank_pad=576)) == RANGE and pack(_latent(), pos=97) == RANGE and pack(_latent(), head=20) == SHAPE and pack(_latent(), kv=170) == SHAPE
    ex = lambda g, **kw: L.cq_mix_latent_expanded(g, 16, kw.get("dp", 16), 16, kw.get("row", 128), 64, 16, 16, 16, 4, kw.get("out", 16), 64, 0, kw.get("rows", 4), None)
    assert ex(_latent(), rows=0) == OK and ex(_latent(), dp=8) == SHAPE and ex(_latent(), row=120) == SHAPE and ex(_latent(), out=None) == NULL and ex(_latent(), rows=101) == RANGE
    assert ex(_latent(), out=8) == ALIGN
    g = _latent(ctx=5000)
    need = L.cq_mix_latent_absorbed_workspace_bytes(g, 1, 4000, 0)
    assert need > 0 and L.cq_mix_latent_absorbed(g, 16, 16, 16, 4, 16, 4000, 1, 16, need - 1, None) == WS
    assert L.cq_mix_latent_absorbed(g, 16, 16, 16, 4, 16, 5000, 1, None, 0, None) == RANGE
    need = L.cq_mix_latent_absorbed_workspace_bytes(g, 1, 0, 1)
    assert L.cq_mix_latent_step(g, 16, 96, 16, 16, 64, 16, 64, 136, 16, 16, None, 0, 16, need - 1, None) == WS
    assert L.cq_mix_latent_step(g, 16, 96, 16, 16, 64, 16, 32, 136, 16, 16, None, 0, 16, need, None) == SHAPE
    assert L.cq_mix_latent_step(g, 16, 96, 16, 16, 64, 16, 64, 136, 16, 16, None, 5000, 16, need, None) == RANGE

    sel = lambda E, top, ld=2000: L.cq_mix_moe_select(16, ld, 0, E, top, 16, 16, None, None)
    assert sel(8, 2) == OK and sel(8, 9) == SHAPE and sel(8, 2, 7) == SHAPE and sel(1025, 2) == RANGE and sel(100, 65) == RANGE
    assert L.cq_mix_moe_max_tiles(10, 4, 3, 8) == 3 + 4 and L.cq_mix_moe_max_tiles(1, 100, 3, 64) == 3
    f = dict(up_dev=16, down_dev=16, up_stride=2 * 40 * 64, down_stride=64 * 64, experts=4, top=2, kp=64, ff=40, ffp=64)
    assert L.cq_mix_moe_step_fits(_lib.Moe(**f)) == 1 and L.cq_mix_moe_step_fits(_lib.Moe(**{**f, "top": 5})) == 0
    assert L.cq_mix_moe_step_fits(_lib.Moe(**{**f, "kp": 65536, "up_stride": 2 * 40 * 65536})) == 0
    step = lambda norm=3, dim=64, **kw: L.cq_mix_moe_step(_lib.Moe(**{**f, **kw}), 16, norm, 16, 1e-5, dim, 16, 16, 16, None, None)
    assert step(0) == DTYPE and step(dim=65) == SHAPE and step(up_dev=None) == NULL and step(shared_ff=8, shared_ffp=64) == NULL and step(down_dev=8) == ALIGN
