"""CPU tests around the Venizen decoder: the oracle against independent formulations of its mechanisms, the sensitivity of the test
configurations to small mistakes, configuration and checkpoint reading, the sequence cache, argument checks of the mixer library."""
import copy
import json
import os

import numpy as np
import pytest
import torch

from candle_amd import _lib, registry
from candle_amd.cache import SequenceCache
from candle_amd.safetensors_file import SafetensorsError, SafetensorsFile
from candle_amd.venizen import Config
from oracle import venizen_oracle as vo
from tests import venizen_cases as vc


def rnd(seed, *shape):
    return np.random.Generator(np.random.PCG64(seed)).standard_normal(shape)


# ---------------------------------------------------------------------------------------------- oracle against other formulations
def test_retention_equals_its_decay_matrix_form():
    T, H, d, e = 13, 3, 5, 7
    q, k, v, g = rnd(1, T, H, d), rnd(2, T, H, d), rnd(3, T, H, e), np.array([0.5, 0.9, 1.0])
    i, j = np.arange(T)[:, None], np.arange(T)[None]
    want = np.stack([((q[:, h] @ k[:, h].T) * np.where(j <= i, g[h] ** (i - j).clip(0), 0.0)) @ v[:, h] for h in range(H)], axis=1)
    assert np.allclose(vo.retention(q, k, v, g), want)


def test_general_delta_equals_transition_matrices():
    T, H, d = 9, 2, 6
    r, k, v, w, a = rnd(1, T, H, d), rnd(2, T, H, d), rnd(3, T, H, d), vo.sigmoid(rnd(4, T, H, d)), vo.sigmoid(rnd(5, T, H, d))
    got = vo.general_delta(r, k, v, w, a)
    for h in range(H):
        S = np.zeros((d, d))
        for t in range(T):
            u = k[t, h] / np.sqrt(k[t, h] @ k[t, h] + 1e-6)
            S = (np.diag(w[t, h]) - np.outer(a[t, h] * u, u)) @ S + np.outer(k[t, h], v[t, h])
            assert np.allclose(got[t, h], S.T @ r[t, h])


def test_attention_without_mixing_and_window_is_causal_softmax():
    T, H, G, d, e = 7, 4, 2, 6, 3
    q, k, v = rnd(1, T, H, d), rnd(2, T, G, d), rnd(3, T, G, e)
    got = vo.talking_attention(q, k, v, np.eye(H), 0.3, vo.window_mask(T, T, 0))
    for h in range(H):
        for t in range(T):
            s = np.exp(0.3 * (k[:t + 1, h // 2] @ q[t, h]))
            assert np.allclose(got[t, h], s @ v[:t + 1, h // 2] / s.sum())


def test_window_mask_by_enumeration():
    m = vo.window_mask(12, 4, 2)
    for i in range(12):
        assert [j for j in range(12) if m[i, j]] == sorted({0, 1} & set(range(i + 1)) | set(range(max(0, i - 3), i + 1)))


def test_rotation_keeps_norms_and_depends_on_distance_only():
    z = np.repeat(rnd(1, 1, 1, 10), 20, axis=0)
    y = vo.rotate_half(z, 100.0, 6)
    assert np.allclose(y[..., 6:], z[..., 6:]) and np.allclose(np.linalg.norm(y, axis=-1), np.linalg.norm(z, axis=-1))
    dots = y[:, 0] @ y[:, 0].T
    assert np.allclose(dots[3, 1], dots[17, 15]) and np.allclose(dots[9, 2], dots[19, 12])
    assert np.allclose(y[1, 0, 0], z[1, 0, 0] * np.cos(1.0) - z[1, 0, 3] * np.sin(1.0))      # dimension 0 pairs with dimension 3


def test_poly_norm_known_values():
    z = np.array([[1.0, -1.0, 1.0, -1.0]])
    assert np.allclose(vo.poly_norm(z, (2.0, 3.0, 5.0, 7.0), 0.0), [[17.0, 3.0, 17.0, 3.0]])


# ---------------------------------------------------------------------------------------------- the configurations show small mistakes
def _mutations(cfg):
    """Configurations that a typical mistake would compute instead of cfg."""
    def edit(f):
        c = copy.deepcopy(cfg)
        f(c)
        return c

    def each_left(key, fn):
        def f(c):
            for la in c["layers"]:
                if la["type"] == "parallel":
                    m = la["mixer"]["left"]
                    m["mask"][key] = fn(m["mask"][key])
        return f

    yield "window one longer", edit(each_left("size", lambda x: x + 1))
    yield "one more kept token", edit(each_left("keep_first", lambda x: x + 1))
    if any(la["mixer"]["left"]["mask"]["size"] > 1 for la in cfg["layers"] if la["type"] == "parallel"):
        yield "window one shorter", edit(each_left("size", lambda x: max(1, x - 1)))
    if cfg["loop"]:
        yield "one pass fewer", edit(lambda c: c["loop"].update(times=c["loop"]["times"] - 1))


@pytest.mark.parametrize("name", sorted(vc.CONFIGS))
def test_small_mistakes_show(name):
    cfg = vc.CONFIGS[name]
    ts, ids = vc.tensors(cfg, 5), vc.token_ids(cfg, 90, 6)
    want = vo.forward(cfg, ts, ids)
    for what, other in _mutations(cfg):
        assert vc.error(vo.forward(other, ts, ids), want) > 0.02, what
    # token 0 read with and without the head mixing transposed
    t2 = {n: (a.T if n.endswith("talk") else a) for n, a in ts.items()}
    assert vc.error(vo.forward(cfg, t2, ids), want) > 0.02


def test_oracle_is_causal():
    cfg = vc.CONFIGS["mixed"]
    ts, ids = vc.tensors(cfg, 5), vc.token_ids(cfg, 40, 6)
    assert np.allclose(vo.forward(cfg, ts, ids)[:25], vo.forward(cfg, ts, ids[:25]))


# ---------------------------------------------------------------------------------------------- configuration, files, cache
@pytest.mark.parametrize("loop,n", [(None, 4), ({"start": 1, "stop": 3, "times": 3}, 4), ({"start": 0, "stop": 4, "times": 2}, 4), ({"start": 2, "stop": 3, "times": 1}, 3)])
def test_layer_runs(loop, n):
    d = vc.config(8, 8, [vc.delta(1, 8)] * n, loop)
    cfg = Config.from_dict(d)
    assert cfg.order == vo.layer_order(d)
    if loop and loop["times"] == 3:
        assert cfg.order == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]


def test_configuration_errors():
    with pytest.raises(ValueError, match="loop"):
        Config.from_dict(vc.config(8, 8, [vc.delta(1, 8)], {"start": 0, "stop": 2, "times": 2}))
    bad = vc.delta(1, 8)
    bad["type"] = "nothing"
    with pytest.raises(ValueError, match="unknown mixer"):
        Config.from_dict(vc.config(8, 8, [bad]))
    bad = vc.delta(1, 8, 16)
    bad["mlp"]["kind"] = "nothing"
    with pytest.raises(ValueError, match="unknown feed-forward"):
        Config.from_dict(vc.config(8, 8, [bad]))


def test_registry_refuses_unknown_architectures(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nothing"}))
    with pytest.raises(ValueError, match="unknown architecture 'Nothing'"):
        registry.load_model(str(tmp_path))


def test_safetensors_reader(tmp_path):
    cfg = vc.CONFIGS["one"]
    ts = vc.tensors(cfg, 3)
    vc.write_checkpoint(str(tmp_path), cfg, ts)
    f = SafetensorsFile(str(tmp_path / "model.safetensors"))
    assert sorted(f.names()) == sorted(ts) and "embed" in f and "nothing" not in f
    for n, a in ts.items():
        t = f.tensor(n)
        assert t.dtype == torch.bfloat16 and np.array_equal(t.float().numpy(), a)
    with pytest.raises(SafetensorsError, match="no tensor nothing"):
        f.tensor("nothing")
    data = (tmp_path / "model.safetensors").read_bytes()
    for cut in (4, 100, len(data) - 1):
        p = tmp_path / "cut.safetensors"
        p.write_bytes(data[:cut])
        with pytest.raises(SafetensorsError):
            SafetensorsFile(str(p))


def test_sequence_cache_keeps_states_in_order():
    c = SequenceCache("cpu")
    k, v = c.add_kv(2, 10, 4, 6)
    s = c.add_state(3, 5)
    assert k.shape == (2, 10, 4) and v.shape == (2, 10, 6) and c.nbytes() == 4 * (80 + 120 + 15)
    c.begin(0)
    s += 1
    c.length = 7
    c.begin(7)
    with pytest.raises(ValueError, match="does not continue"):
        c.begin(3)
    c.begin(0)                                   # starting over gives the old sequence back
    assert c.length == 0 and not s.any()
    only_kv = SequenceCache("cpu")
    only_kv.add_kv(1, 4, 2, 2)
    only_kv.length = 3
    only_kv.begin(1)                             # caches written by position may move back


def test_mixer_argument_validation_codes_without_gpu():
    L = _lib.mixer_lib()
    OK, DTYPE, SHAPE, ALIGN, NULL, WS, RANGE = 0, -1, -2, -3, -4, -5, -6
    mm = lambda *a: L.cq_dense_matmul(*a)
    assert mm(0, 16, 64, 16, 64, 16, 8, None, 0, 0, 0, 8, 64, None, 0, None) == OK
    assert mm(2, 16, 64, 16, 64, 16, 8, None, 0, 0, 4, 8, 64, None, 0, None) == DTYPE
    assert mm(0, 16, 64, 16, 64, 16, 8, None, 0, 0, 4, 8, 60, None, 0, None) == SHAPE
    assert mm(0, 16, 64, 16, 64, 16, 7, None, 0, 0, 4, 8, 64, None, 0, None) == SHAPE
    assert mm(0, None, 64, 16, 64, 16, 8, None, 0, 0, 4, 8, 64, None, 0, None) == NULL
    assert mm(0, 8, 64, 16, 64, 16, 8, None, 0, 0, 4, 8, 64, None, 0, None) == ALIGN
    need = L.cq_dense_matmul_workspace_bytes(0, 4, 8, 4096)
    assert need > 0 and mm(0, 16, 4096, 16, 4096, 16, 8, None, 0, 0, 4, 8, 4096, 16, need - 1, None) == WS
    assert L.cq_dense_matvec(16, 64, 16, 5, 16, 0.0, 64, 16, None, 0, 8, 64, None) == DTYPE
    assert L.cq_dense_matvec(16, 64, 16, 0, None, 0.0, 65, 16, None, 0, 8, 64, None) == SHAPE
    assert L.cq_dense_matvec(16, 64, 16, 1, None, 0.0, 64, 16, None, 0, 8, 64, None) == NULL
    assert L.cq_dense_matvec(16, 65536, 16, 0, None, 0.0, 64, 16, None, 0, 8, 65536, None) == RANGE
    assert [L.cq_mix_state_pad(d) for d in (1, 64, 65, 200, 256, 257)] == [64, 64, 128, 256, 256, -1]
    att = lambda H, G, dp, e, ep, w, k, pos, rows, ctx: L.cq_mix_talk_attention(16, 16, 16, 16, 1.0, w, k, 1.0, 16, H * e, pos, rows, H, G, dp, e, ep, ctx, None, 0, None)
    assert att(4, 3, 16, 16, 16, 4, 0, 0, 1, 8) == SHAPE          # heads not a multiple of kv heads
    assert att(4, 2, 16, 16, 16, 0, 0, 0, 1, 8) == SHAPE          # an empty window
    assert att(4, 2, 24, 16, 16, 4, 0, 0, 1, 8) == SHAPE
    assert att(4, 2, 16, 16, 16, 4, 0, 6, 3, 8) == RANGE          # beyond the cache
    assert att(128, 2, 16, 16, 16, 4, 0, 0, 1, 8) == RANGE
    assert L.cq_mix_delta_scan(16, 16, 64, 16, 16, 64, 1, 2, 300, None) == SHAPE
    assert L.cq_mix_delta_scan(16, 16, 600, 16, 16, 600, 1, 2, 300, None) == RANGE
    g = _lib.MixHeads(heads=2, dim=8, dim_pad=4, dst_dev=16)
    assert L.cq_mix_pack_heads(16, 64, g, 1, 1e-5, None, 0, 1, None) == SHAPE
    g = _lib.MixHeads(heads=2, dim=8, dim_pad=8, dst_dev=16, rot_dims=6)
    assert L.cq_mix_pack_heads(16, 64, g, 1, 1e-5, None, 0, 1, None) == NULL
    assert _lib.ctypes.sizeof(_lib.MixHeads) == 88


def test_trace_runner_is_an_executable_script():
    p = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "trace_run")
    assert os.access(p, os.X_OK) and open(p).readline().startswith("#!")
