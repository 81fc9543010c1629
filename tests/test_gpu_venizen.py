"""Venizen on the GPU: every mixer kernel and the whole decoder against the plain CPU implementation (oracle/venizen_oracle.py)."""
import io
import json

import numpy as np
import pytest
import torch

from candle_amd import _lib, mixers, registry
from candle_amd.cache import SequenceCache
from candle_amd.venizen import Config, Model
from oracle import venizen_oracle as vo
from tests import venizen_cases as vc

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
EPS = 1e-5


def rnd(seed, *shape, scale=1.0):
    return (np.random.Generator(np.random.PCG64(seed)).standard_normal(shape) * scale).astype(np.float32)


def up(a, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(a)).to(device=DEV, dtype=dtype)


_alive = []


def ptr(a):
    """Address of a device copy of a, kept alive until the test ends."""
    _alive.append(up(a))
    return _alive[-1].data_ptr()


@pytest.fixture(autouse=True)
def _release():
    yield
    torch.cuda.synchronize()
    _alive.clear()


def sp():
    return torch.cuda.current_stream().cuda_stream


def rel(got, want):
    got = got.double().cpu().numpy() if isinstance(got, torch.Tensor) else got
    return float(np.abs(got - want).max() / np.abs(want).max())


def padded(a, k):
    """Rows of a padded with zeros to k columns."""
    return np.pad(a, ((0, 0), (0, k - a.shape[1])))


# ---------------------------------------------------------------------------------------------- dense products
@pytest.mark.parametrize("m,n,k", [(1, 5, 24), (2, 33, 64), (7, 70, 200), (31, 64, 4100), (33, 130, 192), (64, 257, 1024), (65, 36, 77), (200, 129, 640), (1300, 2470, 64)])
@pytest.mark.parametrize("precision", [mixers.BF16, mixers.F32])
def test_dense_matmul(m, n, k, precision):
    x, w, r, add = rnd(1, m, k), vc.bf16(rnd(2, n, k, scale=k ** -0.5)), rnd(3, m, n), rnd(4, m, n)
    rt = mixers.Runtime(DEV, precision, 8)
    d = mixers.Dense(rt, [up(w, torch.bfloat16)])
    want = (vc.bf16(x) if precision == mixers.BF16 else x).astype(np.float64) @ w.T.astype(np.float64)
    xd, ld = up(padded(x, d.kp)), mixers.pad_to(n, 4)
    y = torch.full((m, ld), 7.0, device=DEV)
    d.rows(xd.data_ptr(), d.kp, y.data_ptr(), ld, m, sp())
    tol = 3e-6 if precision == mixers.F32 else 1e-5
    assert rel(y[:, :n], want) < tol and bool((y[:, n:] == 7.0).all())
    # the residual epilogue, with an addend, on rows that are not 16-byte aligned
    y = up(r)
    need = rt.L.cq_dense_matmul_workspace_bytes(precision, m, n, d.kp)
    ws = torch.empty(max(need, 4) // 4, device=DEV)
    _lib.check("mm", rt.L.cq_dense_matmul(precision, d.w.data_ptr(), d.kp, xd.data_ptr(), d.kp, y.data_ptr(), n, ptr(add), n, 1, m, n, d.kp, ws.data_ptr(), need, sp()))
    assert rel(y, want + r + add) < tol


@pytest.mark.parametrize("n,k", [(1, 8), (37, 72), (64, 2048), (530, 2100), (9000, 66), (21, 14336), (5, 30000)])
def test_dense_matvec_prologues(n, k):
    x, w = rnd(1, 1, k), vc.bf16(rnd(2, n, k, scale=k ** -0.5))
    g, r, add, coef = rnd(3, k), rnd(4, n), rnd(5, n), np.array([0.6, -0.4, 0.3, 0.15], dtype=np.float32)
    rt = mixers.Runtime(DEV, mixers.BF16, 8)
    d = mixers.Dense(rt, [up(w, torch.bfloat16)])
    xd = torch.full((1, d.kp), 3.0, device=DEV)          # what lies behind the row must not count
    xd[:, :k] = up(x)
    x64, w64 = x.astype(np.float64), w.astype(np.float64)
    for pro, vec, fx in ((mixers.PLAIN, None, x64), (mixers.NORM, g, vo.rms_norm(x64, g, EPS)), (mixers.POLY, coef, vo.poly_norm(x64, coef.astype(np.float64), EPS))):
        want = (fx @ w64.T)[0]
        y = torch.zeros(n, device=DEV)
        d.row(xd.data_ptr(), y.data_ptr(), sp(), pro, up(vec) if vec is not None else None, EPS)
        assert rel(y, want) < 4e-6, pro
        y = up(r)
        a = up(add)
        d.row(xd.data_ptr(), y.data_ptr(), sp(), pro, up(vec) if vec is not None else None, EPS, accumulate=True, add=a.data_ptr())
        assert rel(y, want + r + add) < 4e-6, pro


# ---------------------------------------------------------------------------------------------- row operations
@pytest.mark.parametrize("dim", [4, 7, 66, 1024, 5000])
def test_row_norms(dim):
    L, ld = _lib.mixer_lib(), mixers.pad_to(dim, 4) + 4
    x, w, dl = rnd(1, 9, dim), rnd(2, dim), rnd(3, 9, dim)
    xd, out = up(padded(x, ld)), torch.zeros((9, ld), device=DEV)
    _lib.check("n", L.cq_mix_rms_norm_rows(xd.data_ptr(), ld, None, ptr(padded(dl, ld)), ld, ptr(w), out.data_ptr(), ld, 9, dim, EPS, sp()))
    s = (x + dl).astype(np.float64)
    assert rel(xd[:, :dim], s) < 1e-6 and rel(out[:, :dim], vo.rms_norm(s, w, EPS)) < 2e-6
    index = torch.tensor([8, 0, 3], dtype=torch.int32, device=DEV)
    _lib.check("n", L.cq_mix_rms_norm_rows(xd.data_ptr(), ld, index.data_ptr(), None, 0, ptr(w), out.data_ptr(), ld, 3, dim, EPS, sp()))
    assert rel(out[:3, :dim], vo.rms_norm(s[[8, 0, 3]], w, EPS)) < 2e-6
    coef = np.array([0.5, -0.7, 0.9, -0.2], dtype=np.float32)
    _lib.check("p", L.cq_mix_poly_norm(xd.data_ptr(), ld, ptr(coef), out.data_ptr(), ld, 9, dim, EPS, sp()))
    assert rel(out[:, :dim], vo.poly_norm(s, coef.astype(np.float64), EPS)) < 3e-6
    _lib.check("t", L.cq_mix_tanh(xd.data_ptr(), ld, out.data_ptr(), ld, 9, dim, sp()))
    assert rel(out[:, :dim], np.tanh(s)) < 1e-6


@pytest.mark.parametrize("kind,weight", [(mixers.SILU, False), (mixers.SIGMOID, True)])
@pytest.mark.parametrize("heads,dim", [(1, 5), (3, 64), (5, 200)])
def test_head_norm_gate(heads, dim, kind, weight):
    L, n = _lib.mixer_lib(), heads * dim
    o, g, w = rnd(1, 6, n), rnd(2, 6, n, scale=3.0), rnd(3, n)
    out = torch.zeros((6, n), device=DEV)
    _lib.check("h", L.cq_mix_head_norm_gate(ptr(o), n, ptr(g), n, ptr(w) if weight else None, kind, 0.7, out.data_ptr(), n, 6, heads, dim, EPS, sp()))
    v = vo.over_rms(o.astype(np.float64).reshape(6, heads, dim), EPS).reshape(6, n)
    want = 0.7 * v * (w if weight else 1.0) * (vo.silu(g.astype(np.float64)) if kind == mixers.SILU else vo.sigmoid(g.astype(np.float64)))
    assert rel(out, want) < 3e-6


@pytest.mark.parametrize("dim,rot", [(6, 2), (40, 40), (64, 20), (200, 128), (256, 0)])
def test_pack_heads(dim, rot):
    """Norm, rotation and factor of two groups in one launch, one of them into a cache by position."""
    rt = mixers.Runtime(DEV, mixers.BF16, 50)
    rows, heads, pos, dp = 7, 3, 21, mixers.pad_to(dim, 16)
    src, w = rnd(1, rows, 2 * heads * dim), 1.0 + rnd(2, dim, scale=0.3)
    r = mixers.Rotation(rt, {"base": 300.0, "dims": rot})
    wd, cache, out = up(w), torch.full((heads, 50, dp), 5.0, device=DEV), torch.full((rows, heads, dp), 5.0, device=DEV)
    groups = mixers._group_array([
        mixers._heads(0, heads, dim, dim_pad=dp, dst=out.data_ptr(), row_stride=heads * dp, head_stride=dp, norm=wd, ctx=50, factor=0.5, **r.args()),
        mixers._heads(heads * dim, heads, dim, dim_pad=dp, dst=cache.data_ptr(), row_stride=dp, head_stride=50 * dp, by_position=True, ctx=50, **r.args())])
    _lib.check("p", rt.L.cq_mix_pack_heads(ptr(src), 2 * heads * dim, groups, 2, EPS, None, pos, rows, sp()))
    z = np.zeros((pos + rows, 2, heads, dim))
    z[pos:] = src.reshape(rows, 2, heads, dim)
    a, b = z[:, 0], z[:, 1]
    a = vo.rms_norm(a, w, EPS)
    if rot:
        a, b = vo.rotate_half(a, 300.0, rot), vo.rotate_half(b, 300.0, rot)
    assert rel(out[..., :dim], 0.5 * a[pos:]) < 2e-6 and not out[..., dim:].any()
    got = cache[:, pos:pos + rows].transpose(0, 1)
    assert rel(got[..., :dim], b[pos:]) < 2e-6 and not got[..., dim:].any()
    assert bool((cache[:, :pos] == 5.0).all()) and bool((cache[:, pos + rows:] == 5.0).all())


# ---------------------------------------------------------------------------------------------- attention
def attend(q, k, v, talk, scale, window, keep, pos, rows, out_scale=1.0):
    """cq_mix_talk_attention for the last `rows` of len(k) positions."""
    L = _lib.mixer_lib()
    T, G, d = k.shape
    H, e = q.shape[1], v.shape[2]
    dp, ep, ctx = mixers.pad_to(d, 16), mixers.pad_to(e, 16), T + 3
    kc, vc_, qd = torch.zeros((G, ctx, dp), device=DEV), torch.zeros((G, ctx, ep), device=DEV), torch.zeros((rows, H, dp), device=DEV)
    kc[:, :T, :d], vc_[:, :T, :e], qd[..., :d] = up(k.transpose(1, 0, 2)), up(v.transpose(1, 0, 2)), up(q[pos:pos + rows])
    kc[:, T:], vc_[:, T:] = float("nan"), float("nan")          # positions that do not exist yet
    out = torch.zeros((rows, H * e + 5), device=DEV)
    need = L.cq_mix_talk_attention_workspace_bytes(rows, H, e, window, keep, pos)
    ws = torch.full((max(need, 4) // 4,), float("nan"), device=DEV)
    _lib.check("a", L.cq_mix_talk_attention(qd.data_ptr(), kc.data_ptr(), vc_.data_ptr(), ptr(talk), scale, window, keep, out_scale, out.data_ptr(), H * e + 5, pos,
                                            rows, H, G, dp, e, ep, ctx, ws.data_ptr(), need, sp()))
    assert not out[:, H * e:].any()
    return out[:, :H * e].reshape(rows, H, e)


@pytest.mark.parametrize("H,G,d,e,window,keep,pos,rows", [
    (1, 1, 8, 8, 4, 0, 0, 1), (2, 1, 24, 40, 5, 2, 0, 37), (5, 1, 16, 16, 1, 3, 3, 20), (6, 6, 64, 48, 17, 0, 30, 33), (8, 2, 64, 64, 40, 9, 0, 100),
    (12, 4, 80, 24, 33, 40, 50, 70), (16, 4, 32, 128, 64, 4, 200, 2), (16, 16, 48, 20, 1000, 0, 0, 90), (20, 4, 128, 128, 50, 6, 0, 64), (24, 12, 40, 72, 100, 1, 60, 50),
    (32, 8, 64, 128, 96, 4, 150, 60), (30, 10, 16, 200, 31, 33, 0, 65), (36, 12, 32, 64, 48, 5, 20, 40), (64, 8, 64, 128, 70, 3, 100, 35), (4, 2, 256, 256, 20, 2, 0, 50),
    (6, 2, 32, 32, 300, 7, 700, 40)])
def test_talk_attention(H, G, d, e, window, keep, pos, rows):
    T = pos + rows
    q, k, v, talk = rnd(1, T, H, d), rnd(2, T, G, d), rnd(3, T, G, e), np.eye(H, dtype=np.float32) + rnd(4, H, H, scale=0.4)
    scale = 1.5 * d ** -0.5
    want = vo.talking_attention(q.astype(np.float64), k.astype(np.float64), v.astype(np.float64), talk.astype(np.float64), scale, vo.window_mask(T, window, keep))[pos:]
    assert rel(attend(q, k, v, talk, scale, window, keep, pos, rows, 0.6), 0.6 * want) < 5e-6


@pytest.mark.parametrize("window,keep,T", [(7, 0, 60), (32, 3, 150), (33, 32, 150), (64, 33, 300), (200, 1, 900)])
def test_talk_attention_edges_stand_out(window, keep, T):
    """One key whose score and value stand out, just inside and just outside the window and the kept first tokens: head 0 returns its value
    exactly where it is visible."""
    H, G, d, e = 4, 2, 32, 16
    q, k, v, talk = rnd(1, T, H, d), rnd(2, T, G, d, scale=0.1), rnd(3, T, G, e), np.eye(H, dtype=np.float32)
    i = T - 4
    keys = {j for j in (i, i - 1, i - window + 1, i - window, i - window - 1, keep - 1, keep, keep + 1, 0) if 0 <= j <= i}
    mask = vo.window_mask(T, window, keep)
    for j in sorted(keys):
        kk, vv = k.copy(), v.copy()
        kk[j, 0] = 12.0 * q[i, 0] / np.linalg.norm(q[i, 0])
        vv[j, 0] = 100.0
        want = vo.talking_attention(q.astype(np.float64), kk.astype(np.float64), vv.astype(np.float64), talk.astype(np.float64), 0.5, mask)
        assert (want[i, 0].min() > 60.0) == bool(mask[i, j]), (j, want[i, 0])
        for pos in (0, i - 1, i):
            got = attend(q, kk, vv, talk, 0.5, window, keep, pos, T - pos)
            assert rel(got, want[pos:]) < 5e-6, (j, pos)


class Side:
    """A Parallel mixer on random weights, for its single-token launches."""

    def __init__(self, left, right, ctx, seed=1):
        self.cfg = vc.parallel(left, right)["mixer"]
        rng = {}
        ts = vc.tensors(vc.config(8, 64, [vc.parallel(left, right)]), seed)
        for n, a in ts.items():
            if n.startswith("l0.mix."):
                name = n[len("l0.mix."):]
                rng[name] = up(a, torch.bfloat16 if a.ndim == 2 and not n.endswith("talk") else torch.float32)
        self.ts = {n[len("l0.mix."):]: a.astype(np.float64) for n, a in ts.items() if n.startswith("l0.mix.")}
        self.rt = mixers.Runtime(DEV, mixers.F32, ctx)
        self.m = mixers.Parallel(self.rt, self.cfg, lambda n: rng[n], EPS)
        self.cache = SequenceCache(DEV)
        self.kept = self.m.new_cache(self.cache)


@pytest.mark.parametrize("left,ctx,positions", [
    ((6, 2, 40, 24, 0.3, 9, 3, 1000.0, 20), 40, (0, 1, 2, 3, 8, 9, 10, 11, 12, 38, 39)),
    ((4, 4, 64, 64, 0.2, 1, 1, 1000.0, 64), 40, (0, 1, 2, 39)),
    ((16, 4, 128, 128, 0.1, 64, 20, 1000.0, 128), 300, (0, 15, 16, 63, 64, 84, 85, 299)),
    ((2, 1, 16, 16, 0.4, 5000, 8, 1000.0, 8), 6000, (4094, 4999, 5000, 5010, 5999)),
    ((40, 8, 200, 256, 0.08, 30, 0, 1000.0, 64), 64, (0, 29, 30, 63))])
def test_talk_decode_at_positions(left, ctx, positions):
    """One token at many positions over a full cache: in place of the new key and value lies NaN, and beyond them."""
    right = (2, 16, 24, (0.9, 0.99), 1000.0, 8)
    s = Side(left, right, ctx)
    lt, rg, L = s.m.left, s.m.right, s.rt.L
    H, G, d, e, scale, window, keep, base, dims = left
    full_k, full_v = rnd(5, ctx, G, d), rnd(6, ctx, G, e)
    for n, p in enumerate(positions):
        kv, state = s.kept
        kv[0].zero_(); kv[1].zero_(); state.zero_()
        kv[0][:, :ctx, :d], kv[1][:, :ctx, :e] = up(full_k.transpose(1, 0, 2)), up(full_v.transpose(1, 0, 2))
        kv[0][:, p:], kv[1][:, p:] = float("nan"), float("nan")
        row = rnd(20 + n, s.m.w_in.n)
        rowd, out = up(row), torch.zeros(s.m.w_out.kp, device=DEV)
        rec, nbytes = lt.records()
        pos_dev = torch.tensor([p - 1 if p else 0], dtype=torch.int32, device=DEV)      # host and device positions add up
        pos = p - int(pos_dev)
        _lib.check("d", L.cq_mix_talk_decode(rowd.data_ptr(), mixers._group_array(lt.groups(kv, 0, None)), EPS, lt.talk.data_ptr(), lt.scale, lt.window, lt.keep_first,
                                             pos_dev.data_ptr(), pos, rec, nbytes, sp()))
        v_off, g_off = rg.offsets(s.m.off)
        _lib.check("m", L.cq_mix_talk_merge_retention_step(rec, H, e, lt.window, lt.keep_first, ctx, 0.8, out.data_ptr(), rowd.data_ptr(),
                                                           mixers._group_array(rg.groups(s.m.off, None, None)), v_off, g_off, rg.decay.data_ptr(), state.data_ptr(), rg.heads,
                                                           rg.vdim, EPS, 1.25, out.data_ptr() + 4 * lt.width_out(), pos_dev.data_ptr(), pos, sp()))
        r64 = row.astype(np.float64)
        q = np.zeros((p + 1, H, d)); q[p] = r64[:H * d].reshape(H, d)
        kn = np.zeros((p + 1, G, d)); kn[p] = r64[H * d:(H + G) * d].reshape(G, d)
        vn = r64[(H + G) * d:(H + G) * d + G * e].reshape(G, e)
        q = vo.rotate_half(vo.rms_norm(q, s.ts["left.q.norm"], EPS), base, dims)[p:]
        kn = vo.rotate_half(vo.rms_norm(kn, s.ts["left.k.norm"], EPS), base, dims)[p]
        k, v = full_k[:p + 1].astype(np.float64), full_v[:p + 1].astype(np.float64)
        k[p], v[p] = kn, vn
        seen = vo.window_mask(p + 1, window, keep)[p] if p < 500 else np.array([p - j < window or j < keep for j in range(p + 1)])
        # one query row of the oracle's attention
        sc = np.einsum("hg,gj->hj", s.ts["left.talk"], np.stack([k[:, h // (H // G)] @ q[0, h] for h in range(H)]) * scale)
        sc = np.where(seen[None], sc, -np.inf)
        w = np.exp(sc - sc.max(axis=-1, keepdims=True))
        w /= w.sum(axis=-1, keepdims=True)
        want = np.stack([w[h] @ v[:, h // (H // G)] for h in range(H)])
        assert rel(out[:H * e].reshape(H, e), 0.8 * want) < 1e-5, p
        assert rel(kv[0][:, p, :d], kn) < 2e-6 and rel(kv[1][:, p, :e], vn) < 1e-7 and not kv[0][:, p, d:].any() and not kv[1][:, p, e:].any()
        if p + 1 < ctx:
            assert bool(kv[0][:, p + 1:].isnan().all()) and bool(kv[1][:, p + 1:].isnan().all())
        # the retention step beside it: a first token from a zero state
        m = s.cfg["right"]
        off = s.m.off
        rq, rk = np.zeros((p + 1, 2, 16)), np.zeros((p + 1, 2, 16))
        rq[p], rk[p] = r64[off:off + 32].reshape(2, 16), r64[off + 32:off + 64].reshape(2, 16)
        rq, rk = vo.rotate_half(rq, m["rot"]["base"], 8)[p:], vo.rotate_half(rk, m["rot"]["base"], 8)[p:] / 4.0
        rv, rgate = r64[v_off:v_off + 48].reshape(1, 2, 24), r64[g_off:g_off + 48]
        o = vo.over_rms(vo.retention(rq, rk, rv, np.array([0.9, 0.99])), EPS).reshape(48)
        assert rel(out[H * e:H * e + 48], 1.25 * o * vo.silu(rgate)) < 2e-5, p
        assert rel(state[:, :, :16], np.einsum("hd,he->hed", rk[0], rv[0])) < 1e-6 and not state[:, :, 16:].any()


# ---------------------------------------------------------------------------------------------- retention
@pytest.mark.parametrize("H,d,e", [(1, 8, 8), (3, 24, 40), (2, 64, 130), (4, 128, 64), (2, 256, 96), (9, 40, 16)])
@pytest.mark.parametrize("cuts", [(1, 1, 2, 3), (64, 1, 63, 65), (200,), (2, 700), (130, 500, 33)])
def test_retention_portions(H, d, e, cuts):
    L, T, dp = _lib.mixer_lib(), sum(cuts), mixers.pad_to(d, 16)
    decay = np.linspace(0.6, 1.0, H)
    q, k, v = rnd(1, T, H, d), rnd(2, T, H, d, scale=d ** -0.5), rnd(3, T, H * e)
    want = vo.retention(q.astype(np.float64), k.astype(np.float64), v.astype(np.float64).reshape(T, H, e), decay)
    state = torch.zeros((H, e, L.cq_mix_state_pad(d)), device=DEV)
    l2, at, got = up(np.log2(decay)), 0, []
    for n in cuts:
        qd, kd = torch.zeros((n, H, dp), device=DEV), torch.zeros((n, H, dp), device=DEV)
        qd[..., :d], kd[..., :d] = up(q[at:at + n]), up(k[at:at + n])
        out = torch.zeros((n, H * e + 3), device=DEV)
        need = L.cq_mix_retention_workspace_bytes(n, H, d, e)
        ws = torch.full((max(need, 4) // 4,), float("nan"), device=DEV)
        vd = up(v[at:at + n])
        _lib.check("r", L.cq_mix_retention(qd.data_ptr(), kd.data_ptr(), vd.data_ptr(), H * e, l2.data_ptr(), state.data_ptr(), out.data_ptr(), H * e + 3, n, H, d, dp, e,
                                           ws.data_ptr(), need, sp()))
        got.append(out[:, :H * e].reshape(n, H, e))
        at += n
    got = torch.cat(got).double().cpu().numpy()
    for h in range(H):                               # heads of very different size: each against its own scale
        assert rel(got[:, h], want[:, h]) < 1e-5, h
    S = np.zeros((H, d, e))
    for t in range(T):
        S = decay[:, None, None] * S + k[t].astype(np.float64)[:, :, None] * v[t].astype(np.float64).reshape(H, 1, e)
    assert rel(state[:, :, :d], S.transpose(0, 2, 1)) < 1e-5 and not state[:, :, d:].any()


def test_retention_remembers_a_far_token():
    """A single value written hundreds of tokens ago, everything since orthogonal to it, read back at its decayed size."""
    L, H, d, e, T = _lib.mixer_lib(), 2, 16, 16, 900
    decay = np.array([0.999, 0.99])
    q, k, v = np.zeros((T, H, d), np.float32), rnd(1, T, H, d, scale=0.1), rnd(2, T, H, e)
    k[..., 0] = 0.0
    k[3, :, :], k[3, :, 0], v[3] = 0.0, 1.0, 50.0
    q[-1, :, 0] = 1.0
    state, out = torch.zeros((H, e, 64), device=DEV), torch.zeros((T, H * e), device=DEV)
    need = L.cq_mix_retention_workspace_bytes(T, H, d, e)
    ws = torch.empty(max(need, 4) // 4, device=DEV)
    _lib.check("r", L.cq_mix_retention(ptr(q), ptr(k), ptr(v.reshape(T, -1)), H * e, ptr(np.log2(decay)), state.data_ptr(), out.data_ptr(),
                                       H * e, T, H, d, 16, e, ws.data_ptr(), need, sp()))
    want = 50.0 * decay ** (T - 1 - 3)
    assert np.allclose(out[-1].reshape(H, e).cpu().numpy(), want[:, None], rtol=2e-4)


# ---------------------------------------------------------------------------------------------- generalized delta rule
@pytest.mark.parametrize("H,d", [(1, 8), (3, 20), (9, 48), (2, 64), (3, 100), (2, 200)])
@pytest.mark.parametrize("cuts", [(1, 2, 3), (16, 17, 31, 1), (150,)])
def test_general_delta_portions(H, d, cuts):
    """Packing and scan over portions, and a last token through the single-token kernel."""
    L, W, rank, ldw2 = _lib.mixer_lib(), H * d, 11, 64
    T = sum(cuts) + 1
    rows = rnd(1, T, 5 * W + 12)
    w2, w0, ab, weight = vc.bf16(rnd(2, W, rank, scale=0.7)), rnd(3, W, scale=1.5), rnd(4, W), 1.0 + rnd(5, W, scale=0.2)
    r64 = rows.astype(np.float64)
    part = lambda i: r64[:, i * W:(i + 1) * W].reshape(T, H, d)
    low = np.tanh(r64[:, 5 * W:5 * W + rank])
    wl = low @ w2.T.astype(np.float64)
    w = np.exp(-np.exp(-0.5) * vo.sigmoid(wl + w0)).reshape(T, H, d)
    a = vo.sigmoid(part(4) + ab.astype(np.float64).reshape(H, d))
    want = vo.general_delta(part(0), part(1), part(2), w, a)
    spd = L.cq_mix_state_pad(d)
    state, rd, wld = torch.zeros((H, d, spd), device=DEV), up(rows), up(wl)
    w0d, abd, ld, at = up(w0), up(ab), rows.shape[1], 0
    for n in cuts:
        packed = torch.full((n * H * (4 * spd + 1),), float("nan"), device=DEV)
        out = torch.zeros((n, W + 1), device=DEV)
        src = rd.data_ptr() + 4 * at * ld
        _lib.check("p", L.cq_mix_delta_prep(src, ld, 0, W, 4 * W, wld.data_ptr() + 4 * at * W, W, w0d.data_ptr(), abd.data_ptr(), packed.data_ptr(), n, H, d, sp()))
        _lib.check("s", L.cq_mix_delta_scan(packed.data_ptr(), src + 8 * W, ld, state.data_ptr(), out.data_ptr(), W + 1, n, H, d, sp()))
        assert rel(out[:, :W].reshape(n, H, d), want[at:at + n]) < 1e-5, at
        at += n
    w2d = torch.zeros((W, ldw2), dtype=torch.bfloat16, device=DEV)
    w2d[:, :rank] = up(w2, torch.bfloat16)
    out = torch.zeros(W, device=DEV)
    _lib.check("d", L.cq_mix_delta_step(rd.data_ptr() + 4 * at * ld, 0, W, 2 * W, 3 * W, 4 * W, 5 * W, w2d.data_ptr(), ldw2, rank, w0d.data_ptr(), abd.data_ptr(),
                                        ptr(weight), state.data_ptr(), out.data_ptr(), H, d, EPS, sp()))
    o = vo.over_rms(want[at], EPS).reshape(W) * weight * vo.sigmoid(r64[at, 3 * W:4 * W])
    assert rel(out, o) < 2e-5 and not state[:, :, d:].any()


# ---------------------------------------------------------------------------------------------- the decoder
LIMIT = {"float32": 2e-5, "bfloat16": 2e-2}
_built = {}


def model_of(name, dtype, ctx=400, seed=5):
    key = (name, dtype, ctx, seed)
    if key not in _built:
        cfg = vc.CONFIGS[name]
        ts = vc.tensors(cfg, seed)
        _built[key] = (cfg, ts, Model(Config.from_dict(cfg, ctx), lambda n: torch.from_numpy(ts[n]).to(torch.bfloat16), DEV, dtype))
    cfg, ts, m = _built[key]
    m.reset()
    return cfg, ts, m


def run(m, ids, cuts):
    """Logits at every position, the tokens brought in portions of the given sizes (the last one repeats)."""
    out, at, i = [], 0, 0
    while at < len(ids):
        n = min(cuts[min(i, len(cuts) - 1)], len(ids) - at)
        out.append(m.step(ids[at:at + n], range(n)).cpu().numpy())
        at, i = at + n, i + 1
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(vc.CONFIGS))
def test_prompt_portions_and_decoding_equal_the_oracle(name, dtype):
    cfg, ts, m = model_of(name, dtype)
    ids = vc.token_ids(cfg, 150, 6)
    want, runs_want = vo.forward(cfg, ts, ids, True)
    runs = []
    m.tap = lambda r, x: runs.append(x.double().cpu().numpy())
    whole = run(m, ids, [len(ids)])
    m.tap = None
    assert vc.error(whole, want) < LIMIT[dtype]
    assert len(runs) == len(m.cfg.order) and all(vc.error(a, b) < LIMIT[dtype] for a, b in zip(runs, runs_want))
    for cuts in ([1], [2], [3, 1, 7, 2], [100, 2, 3, 1], [64, 65], [149, 1]):
        m.reset()
        got = run(m, ids, cuts)
        assert vc.error(got, want) < LIMIT[dtype], cuts
        assert vc.error(got, whole) < LIMIT[dtype], cuts


def test_a_sequence_does_not_depend_on_the_one_before():
    cfg, ts, m = model_of("mixed", "float32")
    a, b = vc.token_ids(cfg, 60, 1), vc.token_ids(cfg, 33, 2)
    alone = run(m, b, [20, 1])
    m.reset()
    run(m, a, [40, 1, 5])
    m.reset()
    assert np.array_equal(run(m, b, [20, 1]), alone)
    # position 0 starts over by itself; any other position must continue
    m.step(a[:9], [])
    first = m.step(b[:20], [19], pos=0).cpu().numpy()
    assert vc.error(first, alone[19:20]) < 1e-6
    with pytest.raises(ValueError, match="does not continue"):
        m.step(b[:3], [0], pos=7)


def test_steps_want_any_places_and_check_their_arguments():
    cfg, ts, m = model_of("one", "float32", ctx=30)
    ids = vc.token_ids(cfg, 30, 3)
    want = vo.forward(cfg, ts, ids)
    assert vc.error(m.step(ids[:12], [11, 0, 5, 5]).cpu().numpy(), want[[11, 0, 5, 5]]) < 2e-5
    assert m.step(ids[12:20], []).shape == (0, cfg["vocab"])
    assert vc.error(m.step(ids[20:21], [0, 0]).cpu().numpy(), want[[20, 20]]) < 2e-5
    for tokens, places in (([], []), (ids[:10], [0]), (ids[:2], [2]), ([cfg["vocab"]], [0]), ([-1], [0])):
        with pytest.raises(ValueError):
            m.step(tokens, places)
    assert vc.error(m.step(ids[21:], range(9)).cpu().numpy(), want[21:]) < 2e-5
    with pytest.raises(ValueError, match="outside the context"):
        m.step([1], [0])


def test_long_calls_run_as_several_passes(monkeypatch):
    cfg, ts, m = model_of("plain", "float32")
    ids = vc.token_ids(cfg, 130, 4)
    monkeypatch.setattr(Model, "MAX_ROWS", 43)
    places = [0, 42, 43, 85, 86, 128, 129]
    assert vc.error(m.step(ids, places).cpu().numpy(), vo.forward(cfg, ts, ids)[places]) < 2e-5


def test_long_decoding_stays_on_the_oracle():
    cfg, ts, m = model_of("mixed", "float32")
    ids = vc.token_ids(cfg, 380, 8)
    want = vo.forward(cfg, ts, ids)
    assert vc.error(run(m, ids, [5, 1]), want) < 2e-5


def test_a_far_kept_token_decides_a_decoded_logit():
    """Token 0's key is made to stand out for every later query by its own weights: with the kept tokens left out the logits differ."""
    cfg = json.loads(json.dumps(vc.CONFIGS["one"]))
    cfg["layers"][0]["mixer"]["left"]["mask"] = {"size": 20, "keep_first": 1}
    ts = vc.tensors(cfg, 9)
    left = cfg["layers"][0]["mixer"]["left"]
    left["rot"]["base"] = 1e9                                        # almost no rotation beyond the first pair
    ids = [1] + [2 + t % 60 for t in range(299)]
    ts["embed"][1] *= 0.0
    ts["embed"][1][:8] = 4.0                                         # token 0's own direction
    without = json.loads(json.dumps(cfg))
    without["layers"][0]["mixer"]["left"]["mask"]["keep_first"] = 0
    want = vo.forward(cfg, ts, ids)
    assert vc.error(vo.forward(without, ts, ids)[250:], want[250:]) > 0.02
    m = Model(Config.from_dict(cfg, 300), lambda n: torch.from_numpy(ts[n]).to(torch.bfloat16), DEV, "float32")
    assert vc.error(run(m, ids, [100, 1]), want) < 2e-5


def oracle_greedy(cfg, ts, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(np.argmax(vo.forward(cfg, ts, ids)[-1])))
    return ids[len(prompt):]


def test_greedy_generation_with_and_without_a_graph():
    cfg, ts, m = model_of("mixed", "float32")
    p1, p2 = vc.token_ids(cfg, 21, 10), vc.token_ids(cfg, 40, 11)
    w1, w2 = oracle_greedy(cfg, ts, p1, 24), oracle_greedy(cfg, ts, p2, 30)
    assert m.generate_greedy(p1, 24, use_graph=False)["tokens"] == w1
    for _ in range(3):                                               # capture, then replays between eager work
        assert m.generate_greedy(p1, 24)["tokens"] == w1
        assert m.generate_greedy(p2, 30)["tokens"] == w2
    # the sequence can be continued by hand from where the generation stopped
    last = m.step([w2[-1]], [0]).cpu().numpy()
    assert m.cache.length == 40 + 30 and vc.error(last, vo.forward(cfg, ts, p2 + w2)[-1:]) < 2e-5
    assert m.generate_greedy(p1, 1)["tokens"] == w1[:1]


def test_bfloat16_greedy_graph_equals_eager():
    cfg, ts, m = model_of("wide", "bfloat16")
    p = vc.token_ids(cfg, 50, 12)
    eager = m.generate_greedy(p, 40, use_graph=False)["tokens"]
    assert all(m.generate_greedy(p, 40)["tokens"] == eager for _ in range(2))


def test_checkpoint_folder_through_the_registry_and_command_line(tmp_path, capsys):
    from candle_amd import generate
    cfg = vc.CONFIGS["wide"]
    ts = vc.tensors(cfg, 5)
    vc.write_checkpoint(str(tmp_path), cfg, ts)
    m = registry.load_model(str(tmp_path), dtype="float32", ctx=64)
    ids = vc.token_ids(cfg, 30, 6)
    assert isinstance(m, Model) and vc.error(m.step(ids, range(30)).cpu().numpy(), vo.forward(cfg, ts, ids)) < 2e-5
    generate.main(["--model", str(tmp_path), "--tokens", ",".join(map(str, ids)), "--new", "5", "--dtype", "float32", "--ctx", "64"])
    assert capsys.readouterr().out.splitlines()[0] == ",".join(map(str, oracle_greedy(cfg, ts, ids, 5)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay(tmp_path, capsys, monkeypatch, dtype):
    from candle_amd import trace_run
    cfg = vc.CONFIGS["mixed"]
    ts = vc.tensors(cfg, 5)
    vc.write_checkpoint(str(tmp_path / "m"), cfg, ts)
    (tmp_path / "out").mkdir()
    a, b = vc.token_ids(cfg, 50, 6), vc.token_ids(cfg, 9, 7)
    steps = [("a", a[:30], [0, 29], []), ("a", a[30:32], [], []), ("a", a[32:], [17], ["a"]), ("b", b[:8], [7], []), ("b", b[8:], [0], ["b"])]
    lines = [json.dumps({"step": i, "entries": [{"id": n, "tokens": t, "want": w}], "end": e}) for i, (n, t, w, e) in enumerate(steps)]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(lines) + "\n"))
    trace_run.main(["--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(tmp_path / "out"), "--max-tokens", "64"])
    assert capsys.readouterr().out.split("\n")[:5] == [f"done {i}" for i in range(5)]
    assert sorted(p.name for p in (tmp_path / "out").iterdir()) == ["0.f32", "2.f32", "3.f32", "4.f32"]
    wa, wb = vo.forward(cfg, ts, a), vo.forward(cfg, ts, b)
    for step, want in ((0, wa[[0, 29]]), (2, wa[[49]]), (3, wb[[7]]), (4, wb[[8]])):
        got = np.fromfile(tmp_path / "out" / f"{step}.f32", dtype="<f4").reshape(len(want), cfg["vocab"])
        assert vc.error(got, want) < LIMIT[dtype], step
