"""Kudurax on the GPU: its kernels and the whole decoder against the plain CPU implementation (oracle/kudurax_oracle.py)."""
import io
import json

import numpy as np
import pytest
import torch

from candle_amd import _lib, mixers, registry
from candle_amd.cache import SequenceCache
from candle_amd.kudurax import Config, Model
from oracle import kudurax_oracle as ko
from tests import kudurax_cases as kc

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
EPS = 1e-5
TYPES = [(mixers.F32, 3e-6), (mixers.BF16, 1.2e-2)]


def rnd(seed, *shape, scale=1.0):
    return (np.random.Generator(np.random.PCG64(seed)).standard_normal(shape) * scale).astype(np.float32)


def up(a, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(a)).to(device=DEV, dtype=dtype)


_alive = []


def ptr(a, dtype=torch.float32):
    """Address of a device copy of a, kept alive until the test ends."""
    _alive.append(up(a, dtype))
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
    """The last axis of a padded with zeros to k."""
    return np.pad(a, [(0, 0)] * (a.ndim - 1) + [(0, k - a.shape[-1])])


# ---------------------------------------------------------------------------------------------- norms and activations
@pytest.mark.parametrize("dim", [1, 7, 66, 1024, 5000])
def test_layer_norm_rows(dim):
    L, ld = _lib.mixer_lib(), dim + 3
    x, w, b = rnd(1, 9, dim) + 2.0, rnd(2, dim), rnd(3, dim)
    xd, vec, out = up(padded(x, ld)), up(np.concatenate([w, b])), torch.full((9, ld), 7.0, device=DEV)
    want = ko.layer_norm(x.astype(np.float64), w, b, EPS)
    _lib.check("n", L.cq_mix_layer_norm_rows(xd.data_ptr(), ld, None, vec.data_ptr(), out.data_ptr(), None, ld, 9, dim, EPS, sp()))
    assert rel(out[:, :dim], want) < 3e-6 and bool((out[:, dim:] == 7.0).all())
    index = torch.tensor([8, 0, 3], dtype=torch.int32, device=DEV)
    _lib.check("n", L.cq_mix_layer_norm_rows(xd.data_ptr(), ld, index.data_ptr(), vec.data_ptr(), out.data_ptr(), None, ld, 3, dim, EPS, sp()))
    assert rel(out[:3, :dim], want[[8, 0, 3]]) < 3e-6
    for also in (True, False):
        out, out16 = torch.full((9, ld), 7.0, device=DEV), torch.full((9, ld), 7.0, device=DEV, dtype=torch.bfloat16)
        _lib.check("n", L.cq_mix_layer_norm_rows(xd.data_ptr(), ld, None, vec.data_ptr(), out.data_ptr() if also else None, out16.data_ptr(), ld, 9, dim, EPS, sp()))
        assert rel(out16[:, :dim], want) < 5e-3 and bool((out16[:, dim:] == 7.0).all()) and (rel(out[:, :dim], want) < 3e-6 if also else bool((out == 7.0).all()))


@pytest.mark.parametrize("n,k", [(1, 8), (37, 72), (530, 2100), (21, 14336)])
def test_matvec_prologues(n, k):
    x, w, r = rnd(1, k) + 0.5, kc.bf16(rnd(2, n, k, scale=k ** -0.5)), rnd(4, n)
    g, b = rnd(5, k), rnd(6, k)
    rt = mixers.Runtime(DEV, mixers.BF16, 8)
    d = mixers.Dense(rt, [up(w, torch.bfloat16)])
    xd = torch.full((d.kp,), 3.0, device=DEV)            # what lies behind the row must not count
    xd[:k] = up(x)
    x64 = x.astype(np.float64)
    for pro, vec, fx in ((mixers.LAYER_NORM, up(np.concatenate([g, b])), ko.layer_norm(x64, g, b, EPS)), (mixers.RELU2, None, ko.relu_squared(x64))):
        y = up(r)
        d.row(xd.data_ptr(), y.data_ptr(), sp(), pro, vec, EPS, accumulate=True)
        assert rel(y, w.astype(np.float64) @ fx + r) < 5e-6, pro


# ---------------------------------------------------------------------------------------------- dense products with options
@pytest.mark.parametrize("m,n,k", [(1, 6, 24), (7, 70, 200), (33, 130, 1100), (65, 36, 77), (300, 514, 640)])
@pytest.mark.parametrize("precision,tol", [(mixers.F32, 4e-6), (mixers.BF16, 1e-2)])
def test_product_activations_and_types(m, n, k, precision, tol):
    rt = mixers.Runtime(DEV, precision, 8)
    bf = int(rt.t_bf16)
    x, w, scale = kc.bf16(rnd(1, m, k)), kc.bf16(rnd(2, n, k, scale=k ** -0.5)), rnd(3, m)
    d = mixers.Dense(rt, [up(w, torch.bfloat16)])
    kind = torch.bfloat16 if bf else torch.float32
    xd = up(padded(x, d.kp), kind)
    z = x.astype(np.float64) @ w.T.astype(np.float64)
    for act, want, cols in ((mixers.ACT_NONE, z * scale[:, None], n), (mixers.ACT_RELU2, ko.relu_squared(z) * scale[:, None], n),
                            (mixers.ACT_SWIGLU, ko.silu(z[:, 0::2]) * z[:, 1::2] * scale[:, None], n // 2)):
        for ld in (cols, mixers.pad_to(cols, 8) + 8):
            y = torch.full((m, ld), 7.0, device=DEV, dtype=kind)
            d.rows(xd.data_ptr(), d.kp, y.data_ptr(), ld, m, sp(), act=act, row_scale_dev=ptr(scale), x_bf16=bf, dst_bf16=bf)
            assert rel(y[:, :cols], want) < tol and bool((y[:, cols:] == 7.0).all()), (act, ld)


@pytest.mark.parametrize("precision,tol", [(mixers.F32, 3e-6), (mixers.BF16, 1e-5)])
def test_product_batches(precision, tol):
    rt = mixers.Runtime(DEV, precision, 8)
    B, m, n, k = 5, 37, 75, 128
    x, w = kc.bf16(rnd(1, m, B, k)), kc.bf16(rnd(2, B, n, k, scale=k ** -0.5))
    xd, wd, y = up(x), up(w, torch.bfloat16), torch.zeros((m, B, n + 1), device=DEV)
    mixers.dense_product(rt, precision, sp(), w_dev=wd.data_ptr(), ldw=k, w_batch=n * k, x_dev=xd.data_ptr(), ldx=B * k, x_batch=k, dst_dev=y.data_ptr(), ldd=B * (n + 1),
                         dst_batch=n + 1, m=m, n=n, k=k, batch=B)
    want = np.stack([x[:, b].astype(np.float64) @ w[b].T for b in range(B)], axis=1)
    assert rel(y[..., :n], want) < tol and not y[..., n:].any()


@pytest.mark.parametrize("rows,experts,top,tile", [(1, 5, 2, 64), (40, 3, 3, 64), (300, 7, 2, 32), (300, 7, 2, 128), (130, 300, 4, 64), (4096, 2, 1, 128), (4096, 40, 5, 64)])
@pytest.mark.parametrize("precision", [mixers.F32, mixers.BF16])
def test_grouped_product_over_a_plan(rows, experts, top, tile, precision):
    if precision == mixers.F32 and tile != 64:
        pytest.skip("f32 tiles hold 64 rows")
    rt = mixers.Runtime(DEV, precision, 8)
    L, pairs, n, k = rt.L, rows * top, 36, 64
    rng = np.random.Generator(np.random.PCG64(3))
    ids = np.stack([rng.permutation(experts)[:top] for _ in range(rows)]).astype(np.int32)
    if rows == 300:
        ids[:, 0] = np.where(np.arange(rows) < 290, 1, ids[:, 0])                # one busy expert, some possibly idle
    weights, x, w = rnd(4, rows, top), kc.bf16(rnd(1, rows, k)), kc.bf16(rnd(2, experts, n, k))
    i32 = dict(dtype=torch.int32, device=DEV)
    most = L.cq_mix_moe_max_tiles(rows, experts, top, tile)
    src, dst, n_tiles, tiles, scale = torch.zeros(pairs, **i32), torch.zeros(pairs, **i32), torch.zeros(1, **i32), torch.zeros((most, 4), **i32), torch.zeros(pairs, device=DEV)
    _lib.check("plan", L.cq_mix_moe_plan(ptr(ids, torch.int32), ptr(weights), rows, experts, top, tile, src.data_ptr(), dst.data_ptr(), scale.data_ptr(), tiles.data_ptr(),
                                         n_tiles.data_ptr(), sp()))
    t = tiles[:int(n_tiles)].cpu().numpy()
    order = dst.cpu().numpy()
    assert len(t) <= most and sorted(order.tolist()) == list(range(pairs)) and np.array_equal(src.cpu().numpy(), order // top)
    assert np.array_equal(scale.cpu().numpy(), weights.reshape(-1)[order]) and t[:, 2].sum() == pairs and (t[:, 2] <= tile).all() and (t[:, 2] > 0).all()
    for group, first, count, _ in t:
        assert (ids.reshape(-1)[order[first:first + count]] == group).all()
    xd, wd, y = up(x), up(w, torch.bfloat16), torch.zeros((pairs, n), device=DEV)
    mixers.dense_product(rt, precision, sp(), w_dev=wd.data_ptr(), ldw=k, w_batch=n * k, x_dev=xd.data_ptr(), ldx=k, dst_dev=y.data_ptr(), ldd=n, m=pairs, n=n, k=k, batch=1,
                         tiles_dev=tiles.data_ptr(), n_tiles_dev=n_tiles.data_ptr(), max_tiles=most, tile_rows=tile, src_rows_dev=src.data_ptr(), dst_rows_dev=dst.data_ptr(),
                         row_scale_dev=scale.data_ptr())
    want = np.stack([weights[r, j] * (w[ids[r, j]].astype(np.float64) @ x[r]) for r in range(rows) for j in range(top)])
    assert rel(y, want) < 4e-6
    acc = up(rnd(5, rows, n))
    before = acc.double().cpu().numpy()
    _lib.check("add", L.cq_mix_moe_add(y.data_ptr(), n, top, acc.data_ptr(), n, rows, n - 1, sp()))
    after = before.copy()
    after[:, :n - 1] += want.reshape(rows, top, n).sum(axis=1)[:, :n - 1]
    assert rel(acc, after) < 4e-6


@pytest.mark.parametrize("experts,top", [(1, 1), (5, 5), (64, 8), (65, 3), (200, 64), (1000, 7)])
def test_expert_choice(experts, top):
    rows = 11
    z = rnd(1, rows, experts + 2)
    z[3, :experts] = np.round(z[3, :experts])                                    # equals: the lower expert first
    L, ids, w, s = _lib.mixer_lib(), torch.zeros((rows, top), dtype=torch.int32, device=DEV), torch.zeros((rows, top), device=DEV), torch.zeros(rows, device=DEV)
    _lib.check("s", L.cq_mix_moe_select(ptr(z), experts + 2, rows, experts, top, ids.data_ptr(), w.data_ptr(), s.data_ptr(), sp()))
    want_ids, want_w = ko.route(z[:, :experts].astype(np.float64), top)
    assert np.array_equal(ids.cpu().numpy(), want_ids) and rel(w, want_w) < 2e-6 and rel(s, ko.sigmoid(z[:, experts].astype(np.float64))) < 1e-6


class Feed:
    """A mixture on random weights."""

    def __init__(self, width, mlp, precision, seed=1):
        cfg = kc.config(8, width, [kc.latent(1, 8, 2, 8, 8, 1.0, kc.rot(2), mlp)])
        ts = {n[len("l0.mlp."):]: a for n, a in kc.tensors(cfg, seed).items() if n.startswith("l0.mlp.")}
        self.ts = {n: a.astype(np.float64) for n, a in ts.items()}
        self.rt = mixers.Runtime(DEV, precision, 8)
        self.m = mixers.GatedExperts(self.rt, mlp, lambda n: up(ts[n], torch.bfloat16), EPS)
        vec = {"n": 1.0 + rnd(7, width, scale=0.2), "n.b": rnd(8, width, scale=0.2)}
        self.norm = mixers.LayerNorm(self.rt, lambda n: torch.from_numpy(vec[n]), "n", EPS)
        self.rms = mixers.RmsNorm(self.rt, lambda n: torch.from_numpy(vec[n]), "n", EPS)
        self.normed = lambda x: ko.layer_norm(x, vec["n"], vec["n.b"], EPS)
        self.rms_normed = lambda x: ko.rms_norm(x, vec["n"], EPS)


@pytest.mark.parametrize("width,mlp", [(40, kc.moe(1, 1, 8)), (72, kc.moe(6, 2, 24, 40)), (2100, kc.moe(9, 3, 70, 10)), (136, kc.moe(130, 9, 65)), (64, kc.moe(5, 4, 520, 1030))])
def test_experts_single_token_and_rows(width, mlp):
    for precision, tol in ((mixers.F32, 2e-5), (mixers.BF16, 2e-2)):
        f = Feed(width, mlp, precision)
        ld = mixers.pad_to(width, 64)
        x = rnd(2, 40, width)
        x64 = x.astype(np.float64)
        want = x + ko.mixture(f.normed(x64), f.ts, "", mlp)
        assert f.rt.L.cq_mix_moe_step_fits(f.m.sizes)
        for fused in (True, False):
            f.m.fused = fused
            xd = up(padded(x[:1], ld))
            f.m.step(xd.data_ptr(), f.norm, None, sp())
            assert rel(xd[:, :width], want[:1]) < (2e-5 if fused else tol), fused
        f.m.fused = True
        xd = up(padded(x[:1], ld))
        f.m.step(xd.data_ptr(), f.rms, ptr(np.full((1, width), 0.25, np.float32)), sp())
        assert rel(xd[:, :width], x[:1] + ko.mixture(f.rms_normed(x64[:1]), f.ts, "", mlp) + 0.25) < 2e-5
        xd, h = up(padded(x, ld)), f.rt.normed(f.m.INPUT, 40 * ld)
        f.norm.rows(xd.data_ptr(), ld, h, ld, 40, sp())
        f.m.prefill(h, ld, xd.data_ptr(), ld, 40, sp())
        assert rel(xd[:, :width], want) < tol and not xd[:, width:].any()


# ---------------------------------------------------------------------------------------------- latent attention
class Attention:
    """The attention of a latent mixer on given latents and queries: both forms and the single-token step, the cache filled with NaN where nothing may be read."""

    def __init__(self, H, d, r, e, rank, T, precision, seed=1, scale=0.2, eps=EPS):
        self.H, self.d, self.r, self.e, self.rank, self.T = H, d, r, e, rank, T
        m = {"heads": H, "dim": d, "rot_dim": r, "vdim": e, "kv_rank": rank, "scale": scale, "rot": kc.rot(r, 1000.0, (2.0, 8.0, 1.0, 32))}
        self.m, w = m, 8
        self.ts = {"q": np.zeros((H * (d + r), w), np.float32), "dkv": np.zeros((rank + r, w), np.float32), "dkv.norm": 1.0 + rnd(seed + 5, rank, scale=0.2),
                   "uk": kc.bf16(rnd(seed + 1, H * d, rank, scale=rank ** -0.5)), "uv": kc.bf16(rnd(seed + 2, H * e, rank, scale=rank ** -0.5)),
                   "g": np.zeros((H, w), np.float32), "o": np.zeros((w, H * e), np.float32)}
        self.rt = mixers.Runtime(DEV, precision, T + 3)
        self.la = mixers.LatentAttention(self.rt, m, lambda n: up(self.ts[n], torch.float32 if n == "dkv.norm" else torch.bfloat16), eps)
        self.kept = self.la.new_cache(SequenceCache(DEV))
        n = H * (d + r)
        self.rows = rnd(seed + 3, T, n + rank + r + H)                           # projection rows: queries, latent, rotated key part, gates
        self.g_off = n + rank + r

    def want(self):
        z = self.rows.astype(np.float64)
        H, d, r, e, T = self.H, self.d, self.r, self.e, self.T
        n = H * (d + r)
        c = ko.rms_norm(z[:, n:n + self.rank], self.ts["dkv.norm"], EPS)
        kr = ko.rotate_pairs(z[:, None, n + self.rank:n + self.rank + r], self.m["rot"])[:, 0]
        q = z[:, :n].reshape(T, H, d + r)
        q = np.concatenate([q[..., :d], ko.rotate_pairs(q[..., d:], self.m["rot"])], axis=-1)
        k = np.concatenate([(c @ self.ts["uk"].T).reshape(T, H, d), np.repeat(kr[:, None], H, axis=1)], axis=-1)
        v = (c @ self.ts["uv"].T).reshape(T, H, e)
        o = ko.causal_attention(q, k, v, self.m["scale"]) * ko.sigmoid(z[:, self.g_off:])[..., None]
        return o.reshape(T, H * e)

    def run(self, cuts, form):
        """Head outputs of all rows brought in the given portions; form: expanded, absorbed or step (portions of one)."""
        la, rt, L, H = self.la, self.rt, self.rt.L, self.H
        self.kept[self.T:] = float("nan")
        self.kept[:self.T].fill_(float("nan"))
        self.kept[:, la.rank:la.rank_pad] = 0
        self.kept[:, la.rank_pad + la.rot_dim:] = 0
        kind = torch.bfloat16 if rt.t_bf16 else torch.float32
        rowd = up(np.pad(self.rows, ((0, 0), (0, -self.rows.shape[1] % 4))))
        ldp, at, out = rowd.shape[1], 0, []
        bf = int(rt.t_bf16)
        for n in cuts:
            row, gate = rowd[at:].data_ptr(), rowd[at:].data_ptr() + 4 * self.g_off
            o = torch.zeros((n, H * self.e), device=DEV)
            if form == "step":
                need = L.cq_mix_latent_absorbed_workspace_bytes(la.shape, 1, 0, 1)
                ws, q = torch.full((need // 4,), float("nan"), device=DEV), torch.zeros((H, la.ld), device=DEV, dtype=kind)
                pos_dev = torch.tensor([at - 1 if at else 0], dtype=torch.int32, device=DEV)       # host and device positions add up
                _lib.check("s", L.cq_mix_latent_step(la.shape, row, la.kv_off, self.kept.data_ptr(), la.ukt.data_ptr(), la.ukt.shape[2], la.uv.w.data_ptr(), la.uv.kp,
                                                     self.g_off, q.data_ptr(), o.data_ptr(), pos_dev.data_ptr(), at - int(pos_dev), ws.data_ptr(), need, sp()))
            elif form == "expanded":
                head = la.dim_pad + la.rot_pad
                o = o.to(kind)
                q, kv = torch.full((n, H, head), float("nan"), device=DEV, dtype=kind), torch.full((at + n, la.expand.n), float("nan"), device=DEV, dtype=kind)
                _lib.check("p", L.cq_mix_latent_pack(la.shape, row, ldp, la.kv_off, self.kept.data_ptr(), None, 0, q.data_ptr(), head, la.dim_pad, at, n, sp()))
                # the product reads whole steps of 64 columns of finite values; copy the rows that exist
                src = torch.zeros((at + n, mixers.pad_to(la.ld, 64)), device=DEV, dtype=kind)
                src[:, :la.ld] = self.kept[:at + n]
                la.expand.rows(src.data_ptr(), src.shape[1], kv.data_ptr(), la.expand.n, at + n, sp(), x_bf16=bf, dst_bf16=bf)
                _lib.check("e", L.cq_mix_latent_expanded(la.shape, q.data_ptr(), la.dim_pad, kv.data_ptr(), la.expand.n, H * la.dim_pad, la.v_pad, self.kept.data_ptr(), gate, ldp,
                                                         o.data_ptr(), H * self.e, at, n, sp()))
            else:
                kp = la.ukt.shape[2]
                plain, q = torch.zeros((n, H, kp), device=DEV), torch.zeros((n, H, la.ld), device=DEV, dtype=kind)
                lat = torch.full((n, H, la.rank_pad), float("nan"), device=DEV)
                _lib.check("p", L.cq_mix_latent_pack(la.shape, row, ldp, la.kv_off, self.kept.data_ptr(), plain.data_ptr(), kp, q.data_ptr(), la.ld, la.rank_pad, at, n, sp()))
                mixers.dense_product(rt, rt.precision, sp(), w_dev=la.ukt.data_ptr(), ldw=kp, w_batch=la.rank * kp, x_dev=plain.data_ptr(), ldx=H * kp, x_batch=kp,
                                     dst_dev=q.data_ptr(), ldd=H * la.ld, dst_batch=la.ld, dst_bf16=bf, m=n, n=la.rank, k=kp, batch=H)
                need = L.cq_mix_latent_absorbed_workspace_bytes(la.shape, n, at, 0)
                ws = torch.full((max(need, 4) // 4,), float("nan"), device=DEV)
                _lib.check("a", L.cq_mix_latent_absorbed(la.shape, q.data_ptr(), self.kept.data_ptr(), gate, ldp, lat.data_ptr(), at, n, ws.data_ptr(), need, sp()))
                uv = torch.from_numpy(self.ts["uv"].reshape(H, self.e, self.rank)).to(DEV)
                o = torch.einsum("nhr,her->nhe", lat[..., :self.rank].float(), uv).reshape(n, H * self.e)
            out.append(o.float())
            at += n
        assert bool(self.kept[at:, :la.rank].isnan().all())                      # nothing written beyond
        return torch.cat(out)


SHAPES = [(1, 8, 2, 8, 8, 70), (3, 24, 10, 40, 36, 140), (16, 72, 24, 56, 112, 150), (5, 128, 64, 128, 512, 130), (18, 40, 16, 20, 130, 90), (33, 16, 8, 12, 256, 70), (2, 250, 64, 250, 200, 80), (3, 32, 150, 24, 90, 100)]


@pytest.mark.parametrize("precision,tol", TYPES)
@pytest.mark.parametrize("H,d,r,e,rank,T", SHAPES)
def test_latent_attention_forms_and_portions(H, d, r, e, rank, T, precision, tol):
    a = Attention(H, d, r, e, rank, T, precision)
    want = a.want()
    for form, cuts in (("expanded", [T]), ("expanded", [1, 2, 63, T - 66]), ("absorbed", [T]), ("absorbed", [2, 1, 30, 31, T - 64]), ("step", [1] * T)):
        assert rel(a.run(cuts, form), want) < tol, (form, cuts)


@pytest.mark.parametrize("precision,tol", TYPES)
@pytest.mark.parametrize("T", [66, 130, 700])
def test_one_key_stands_out(T, precision, tol):
    """One position whose score for the last query and whose value stand out, at the first tokens, around the borders of key tiles and splits, at the query
    itself and right behind an earlier query: its value decides the output exactly where it is visible."""
    H, d, r, e, rank = 4, 32, 8, 16, 48
    i = T - 2
    for j in sorted({x for x in (0, 1, 15, 16, 31, 32, 33, 63, 64, 65, 127, 128, i - 1, i, i + 1) if x < T}):
        a = Attention(H, d, r, e, rank, T, precision, scale=1.0)
        a.rows *= 0.3
        n = H * (d + r)
        a.rows[:, n:n + rank] = rnd(9, T, rank) * [0.2] * rank
        a.rows[:, n:n + 4] = 0.0
        a.rows[:, n + 4] = 1.0                       # keeps the other latents' norm away from zero
        a.rows[j, n:n + rank] = 0.0
        a.rows[j, n] = 5.0                           # the latent of j: only its first value
        a.ts["uk"][:, 0] = 0.0
        for h in range(H):
            a.ts["uk"][h * d, 0] = 1.0               # it is the first unrotated key dimension of every head
            a.rows[i:, h * (d + r)] = 6.0            # which the last queries ask for
        a.ts["uv"][:, 0] = 3.0
        a.la = mixers.LatentAttention(a.rt, a.m, lambda x: up(a.ts[x], torch.float32 if x == "dkv.norm" else torch.bfloat16), EPS)
        want = a.want()
        gated = want[i] / np.repeat(ko.sigmoid(a.rows[i, a.g_off:].astype(np.float64)), e)
        assert (gated.min() > 10.0) == (j <= i), (j, gated)
        for form, cuts in (("expanded", [T]), ("absorbed", [T]), ("absorbed", [T - 2, 2]), ("expanded", [T - 3, 3]), ("step", [1] * T)):
            if form == "step" and T > 200 and j not in (0, 64, i):
                continue
            got = a.run(cuts, form)
            assert rel(got[i:], want[i:]) < tol, (j, form, cuts)


# ---------------------------------------------------------------------------------------------- the decoder
LIMIT = {"float32": 2e-5, "bfloat16": 3e-2}
_built = {}


def model_of(name, dtype, ctx=400, seed=5):
    key = (name, dtype, ctx, seed)
    if key not in _built:
        cfg = kc.CONFIGS[name]
        ts = kc.tensors(cfg, seed)
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


def error(got, want, dtype):
    """bfloat16: a position whose router decides between two nearly equal experts may go the other way; the median position stands for all."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    e = np.sqrt(((got - want) ** 2).mean(axis=-1)) / np.sqrt((want ** 2).mean())
    return float(e.max() if dtype == "float32" else np.median(e))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(kc.CONFIGS))
def test_prompt_portions_and_decoding_equal_the_oracle(name, dtype):
    cfg, ts, m = model_of(name, dtype)
    ids = kc.token_ids(cfg, 230, 6)
    want, runs_want = ko.forward(cfg, ts, ids, True)
    runs = []
    m.tap = lambda r, x: runs.append(x.double().cpu().numpy())
    whole = run(m, ids, [len(ids)])
    m.tap = None
    assert error(whole, want, dtype) < LIMIT[dtype]
    assert len(runs) == len(cfg["layers"]) and all(error(a, b, dtype) < LIMIT[dtype] for a, b in zip(runs, runs_want))
    for cuts in ([1], [2], [3, 1, 7, 2], [100, 2, 3, 1], [64, 65], [229, 1]):
        m.reset()
        got = run(m, ids, cuts)
        assert error(got, want, dtype) < LIMIT[dtype], cuts
        assert error(got, whole, dtype) < LIMIT[dtype], cuts


def test_large_prompts_expand_and_small_portions_absorb():
    """Full-size latents: a prompt that is long enough for keys and values per head, then portions and tokens over the latents themselves."""
    cfg, ts, m = model_of("large", "float32")
    ids = kc.token_ids(cfg, 300, 4)
    assert m.layers[0].mixer.expands(200) and not m.layers[0].mixer.expands(60)
    want = ko.forward(cfg, ts, ids)
    for cuts in ([280, 5, 1], [3, 270, 2], [300]):
        m.reset()
        assert error(run(m, ids, cuts), want, "float32") < 2e-5, cuts


def test_a_sequence_does_not_depend_on_the_one_before():
    cfg, ts, m = model_of("mixed", "float32")
    a, b = kc.token_ids(cfg, 90, 1), kc.token_ids(cfg, 33, 2)
    alone = run(m, b, [20, 1])
    m.reset()
    run(m, a, [40, 1, 5])
    m.reset()
    assert np.array_equal(run(m, b, [20, 1]), alone)
    for t in m.cache.rows:                               # what an earlier sequence left behind is never read
        t[len(b):] = float("nan")
    m.reset()
    assert np.array_equal(run(m, b, [20, 1]), alone)
    for t in m.cache.rows:
        t[len(b):] = 0
    # caches by position: a sequence may be continued from an earlier place
    m.step(b[:30], [])
    again = m.step(b[20:], range(13), pos=20).cpu().numpy()
    assert error(again, alone[20:], "float32") < 1e-5


def test_layers_share_the_cache_they_attend_to():
    cfg, ts, m = model_of("mixed", "float32")
    assert len(m.cache.rows) == 2 and m.kept[1] is m.kept[0] and m.kept[4] is m.kept[0] and m.kept[3] is m.kept[2]


def test_steps_want_any_places_and_check_their_arguments():
    cfg, ts, m = model_of("one", "float32", ctx=30)
    ids = kc.token_ids(cfg, 30, 3)
    want = ko.forward(cfg, ts, ids)
    assert kc.error(m.step(ids[:12], [11, 0, 5, 5]).cpu().numpy(), want[[11, 0, 5, 5]]) < 2e-5
    assert m.step(ids[12:20], []).shape == (0, cfg["vocab"])
    assert kc.error(m.step(ids[20:21], [0, 0]).cpu().numpy(), want[[20, 20]]) < 2e-5
    assert kc.error(m.step(ids[21:], range(9)).cpu().numpy(), want[21:]) < 2e-5
    with pytest.raises(ValueError, match="outside the context"):
        m.step([1], [0])


def test_long_calls_run_as_several_passes(monkeypatch):
    cfg, ts, m = model_of("plain", "float32")
    ids = kc.token_ids(cfg, 130, 4)
    monkeypatch.setattr(Model, "MAX_ROWS", 43)
    places = [0, 42, 43, 85, 86, 128, 129]
    assert kc.error(m.step(ids, places).cpu().numpy(), ko.forward(cfg, ts, ids)[places]) < 2e-5


def test_long_decoding_stays_on_the_oracle():
    cfg, ts, m = model_of("mixed", "float32")
    ids = kc.token_ids(cfg, 390, 8)
    assert kc.error(run(m, ids, [5, 1]), ko.forward(cfg, ts, ids)) < 2e-5


def oracle_greedy(cfg, ts, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(np.argmax(ko.forward(cfg, ts, ids)[-1])))
    return ids[len(prompt):]


def test_greedy_generation_with_and_without_a_graph():
    cfg, ts, m = model_of("mixed", "float32")
    p1, p2 = kc.token_ids(cfg, 21, 10), kc.token_ids(cfg, 40, 11)
    w1, w2 = oracle_greedy(cfg, ts, p1, 24), oracle_greedy(cfg, ts, p2, 30)
    assert m.generate_greedy(p1, 24, use_graph=False)["tokens"] == w1
    for _ in range(3):                                               # capture, then replays between eager work
        assert m.generate_greedy(p1, 24)["tokens"] == w1
        assert m.generate_greedy(p2, 30)["tokens"] == w2
    # the sequence can be continued by hand from where the generation stopped
    last = m.step([w2[-1]], [0]).cpu().numpy()
    assert m.cache.length == 40 + 30 and kc.error(last, ko.forward(cfg, ts, p2 + w2)[-1:]) < 2e-5
    # experts too large for the two launches of a token: the same tokens from the several-row path, captured as well
    for la in m.layers:
        if isinstance(la.mlp, mixers.GatedExperts):
            la.mlp.fused = False
    m._graph = None
    try:
        assert all(m.generate_greedy(p1, 24)["tokens"] == w1 for _ in range(2))
    finally:
        for la in m.layers:
            if isinstance(la.mlp, mixers.GatedExperts):
                la.mlp.fused = True
        m._graph = None


def test_bfloat16_greedy_graph_equals_eager():
    cfg, ts, m = model_of("wide", "bfloat16")
    p = kc.token_ids(cfg, 50, 12)
    eager = m.generate_greedy(p, 40, use_graph=False)["tokens"]
    assert all(m.generate_greedy(p, 40)["tokens"] == eager for _ in range(2))


def test_checkpoint_folder_through_the_registry_and_command_line(tmp_path, capsys):
    from candle_amd import generate
    cfg = kc.CONFIGS["mixed"]
    ts = kc.tensors(cfg, 5)
    kc.write_checkpoint(str(tmp_path), cfg, ts)
    m = registry.load_model(str(tmp_path), dtype="float32", ctx=64)
    ids = kc.token_ids(cfg, 30, 6)
    assert isinstance(m, Model) and kc.error(m.step(ids, range(30)).cpu().numpy(), ko.forward(cfg, ts, ids)) < 2e-5
    generate.main(["--model", str(tmp_path), "--tokens", ",".join(map(str, ids)), "--new", "5", "--dtype", "float32", "--ctx", "64"])
    assert capsys.readouterr().out.splitlines()[0] == ",".join(map(str, oracle_greedy(cfg, ts, ids, 5)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay(tmp_path, capsys, monkeypatch, dtype):
    from candle_amd import trace_run
    cfg = kc.CONFIGS["plain"]
    ts = kc.tensors(cfg, 5)
    kc.write_checkpoint(str(tmp_path / "m"), cfg, ts)
    (tmp_path / "out").mkdir()
    a, b = kc.token_ids(cfg, 50, 6), kc.token_ids(cfg, 9, 7)
    steps = [("a", a[:30], [0, 29], []), ("a", a[30:32], [], []), ("a", a[32:], [17], ["a"]), ("b", b[:8], [7], []), ("b", b[8:], [0], ["b"])]
    lines = [json.dumps({"step": i, "entries": [{"id": n, "tokens": t, "want": w}], "end": e}) for i, (n, t, w, e) in enumerate(steps)]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(lines) + "\n"))
    trace_run.main(["--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(tmp_path / "out"), "--max-tokens", "64"])
    assert capsys.readouterr().out.split("\n")[:5] == [f"done {i}" for i in range(5)]
    wa, wb = ko.forward(cfg, ts, a), ko.forward(cfg, ts, b)
    for step, want in ((0, wa[[0, 29]]), (2, wa[[49]]), (3, wb[[7]]), (4, wb[[8]])):
        got = np.fromfile(tmp_path / "out" / f"{step}.f32", dtype="<f4").reshape(len(want), cfg["vocab"])
        assert kc.error(got, want) < LIMIT[dtype] * (1 if dtype == "float32" else 4), step
