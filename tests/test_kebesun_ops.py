"""Each mechanism of the Kebesun design alone: ``kserve_amd.ops`` (and the
mixture of experts) against the float64 functions of kebesun_oracle.py.

Parametrised over the CPU forms (always) and the HIP kernels in both
activation dtypes (marked gpu). Inputs are rounded to the activation dtype
first, so the oracle and the op see the same numbers.
"""

import os
import sys

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import kebesun_oracle as O  # noqa: E402

from kserve_amd import ops  # noqa: E402
from kserve_amd.engine.config import SoftmaxMoESpec  # noqa: E402
from kserve_amd.models.mixers import SoftmaxRoutedMoE  # noqa: E402
from kserve_amd.ops.torch_ref import scaled_inv_freq  # noqa: E402

BACKENDS = [
    pytest.param(("cpu", torch.float32), id="cpu-f32"),
    pytest.param(("cuda", torch.float32), id="gpu-f32", marks=pytest.mark.gpu),
    pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=pytest.mark.gpu),
]


@pytest.fixture(params=BACKENDS)
def be(request):
    if request.param[0] == "cuda":
        assert ops.has_native_seq(), "kserve_amd_seq_C must be built on a GPU box"
    return request.param


def rnd(*shape, seed=0, scale=1.0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype).float()


def act(x, be):
    return x.to(be[1]).to(be[0])


def f32(x, be):
    return x.float().to(be[0])


def i32(v, be):
    return torch.as_tensor(v, dtype=torch.int32).to(be[0])


def i64(v, be):
    return torch.as_tensor(v, dtype=torch.int64).to(be[0])


def np64(x):
    return x.double().cpu().numpy()


def close(got, want, be, f32_tol=2e-5, bf16_tol=2e-2):
    tol = bf16_tol if be[1] == torch.bfloat16 else f32_tol
    got = np64(got)
    scale = max(np.abs(want).max(), 1e-6)
    err = np.abs(got - want).max() / scale
    assert err < tol, f"relative error {err:.3g} (tolerance {tol})"


class TestScaledResidualNorm:
    @pytest.mark.parametrize("width", [16, 50, 192, 2048, 8204])
    @pytest.mark.parametrize("rows", ["plain", "gathered"])
    def test_two_scaled_deltas(self, be, width, rows):
        eps, T, top = 1e-5, 6, 3
        x = rnd(T, width, seed=1, scale=2.0)
        d0 = rnd(T, width + 8, seed=2, dtype=be[1])[:, :width]
        c0, c1 = rnd(width, seed=3), rnd(width, seed=4)
        w = rnd(width, seed=5) * 0.2
        kw = {}
        if rows == "plain":
            d1 = rnd(T, width, seed=6, dtype=be[1])
            summed = np64(d1)
        else:
            d1 = rnd(T * top + 2, width, seed=6, dtype=be[1])
            index = torch.randperm(T * top, generator=torch.Generator().manual_seed(7))
            rw = rnd(T * top, seed=8).abs()
            summed = (np64(d1)[index] * np64(rw)[:, None]).reshape(T, top, width).sum(1)
            kw = dict(d1_index=i32(index, be), d1_weights=f32(rw, be), d1_top=top)
        new_x = np64(x) + np64(c0) * np64(d0) + np64(c1) * summed
        xr = f32(x, be).clone()
        dd = act(torch.cat([d0, d0[:, :8]], dim=1), be)[:, :width]  # strided rows
        got = ops.add_rms_norm_f32res(
            xr, f32(w, be), eps, 1.0, be[1], d0=dd, c0=f32(c0, be), d1=act(d1, be),
            c1=f32(c1, be), **kw,
        )
        assert got.dtype == be[1]
        close(xr, new_x, be, bf16_tol=1e-5)
        close(got, O.norm(new_x, np64(w), eps), be)

    @pytest.mark.parametrize("width", [24, 50, 1024])
    def test_without_norm_and_without_output(self, be, width):
        T = 4
        x = rnd(T, width, seed=11)
        d = rnd(T, width, seed=12, dtype=be[1])
        c = rnd(width, seed=13)
        want = np64(x) + np64(c) * np64(d)
        xr = f32(x, be).clone()
        got = ops.add_rms_norm_f32res(xr, None, 1e-5, 1.0, be[1], d0=act(d, be), c0=f32(c, be))
        close(xr, want, be, bf16_tol=1e-5)
        close(got, want, be, bf16_tol=5e-3)
        xr = f32(x, be).clone()
        assert ops.add_rms_norm_f32res(
            xr, None, 1e-5, 1.0, be[1], d1=act(d, be), c1=f32(c, be), want_out=False
        ) is None
        close(xr, want, be, bf16_tol=1e-5)
        # nothing to add: a rounded copy, the stream untouched
        got = ops.add_rms_norm_f32res(xr, None, 1e-5, 1.0, be[1])
        assert torch.equal(got, xr.to(be[1]))
        # an fp32 delta without a factor beside an output of either dtype
        e = rnd(T, width, seed=14)
        xr = f32(x, be).clone()
        ops.add_rms_norm_f32res(xr, f32(c, be), 1e-5, 1.0, be[1], d0=f32(e, be))
        close(xr, np64(x) + np64(e), be, bf16_tol=1e-5)

    @pytest.mark.parametrize("T,N,K", [(1, 24, 16), (33, 40, 56), (5, 7, 9)])
    def test_product_with_fp32_result(self, be, T, N, K):
        x, w = rnd(T, K, seed=15, dtype=be[1]), rnd(N, K, seed=16, dtype=be[1])
        got = ops.linear_f32out(act(x, be), act(w, be))
        assert got.dtype == torch.float32
        close(got, np64(x) @ np64(w).T, be, bf16_tol=2e-5)


class TestChannelDecays:
    @pytest.mark.parametrize("T,r,n,tau", [(1, 1, 8, 1.0), (17, 5, 24, 16.0), (40, 16, 300, 4.0),
                                           (16, 64, 256, 0.5), (3, 20, 1, 100.0)])
    def test_against_oracle(self, be, T, r, n, tau):
        low = rnd(T, r + 4, seed=21, scale=2.0, dtype=be[1])[:, :r]
        w2, b = rnd(n, r, seed=22), rnd(n, seed=23, scale=3.0)
        wide = act(torch.cat([low, low[:, :1].expand(-1, 4)], dim=1), be)
        got = ops.lowrank_channel_decay(wide[:, :r], f32(w2, be), f32(b, be), tau)
        assert got.dtype == torch.float32
        want = O.sigmoid(np64(low) @ np64(w2).T + np64(b)) ** (1.0 / tau)
        close(got, want, be, bf16_tol=2e-5)

    def test_extreme_logits(self, be):
        """Decays next to 0 and next to 1: the logarithm of the sigmoid must
        neither overflow nor lose the distance from 1."""
        low = torch.zeros(1, 4)
        b = torch.tensor([-200.0, -80.0, -30.0, 0.0, 8.0, 30.0, 200.0])
        w2 = torch.zeros(7, 4)
        got = np64(ops.lowrank_channel_decay(act(low, be), f32(w2, be), f32(b, be), 16.0))[0]
        want = np.exp(-np.logaddexp(0.0, -np64(b)) / 16.0)
        assert np.all(np.isfinite(got)) and np.abs(got - want).max() < 1e-6
        assert np.abs((1 - got[4]) / (1 - want[4]) - 1) < 5e-3


class TestGatedLinearScan:
    def _inputs(self, T, H, K, V, be, seed):
        q, k = (rnd(T, H * K, seed=seed + i, dtype=be[1]) for i in range(2))
        v = rnd(T, H * V, seed=seed + 2, dtype=be[1])
        a = torch.sigmoid(rnd(T, H * K, seed=seed + 3, scale=2.0)) ** 0.25
        return q, k, v, a

    def _oracle(self, q, k, v, a, H, scale):
        T = q.shape[0]
        r = lambda x: np64(x).reshape(T, H, -1)  # noqa: E731
        return O.gla_recurrence(r(q) * scale, r(k), r(v), r(a)).reshape(T, -1)

    def _run(self, be, parts, state):
        """parts: [(tensors of one sequence, first row, rows, slot)]; q, k and
        v are column slices of wider rows."""
        rows = [torch.cat([s[j][lo : lo + n] for s, lo, n, _ in parts]) for j in range(4)]
        wide = act(torch.cat([rows[0], rows[1], rows[2], rows[0][:, :1]], dim=1), be)
        c = np.cumsum([0] + [t.shape[1] for t in rows[:3]])
        pos = torch.cat([torch.arange(lo, lo + n) for _, lo, n, _ in parts])
        cu = np.cumsum([0] + [n for _, _, n, _ in parts])
        H, K = state.shape[1], state.shape[3]
        return ops.linear_scan(
            wide[:, c[0] : c[1]], wide[:, c[1] : c[2]], wide[:, c[2] : c[3]], state,
            i64(pos, be), i32(cu, be), i32([s for *_, s in parts], be), H,
            channel_decay=f32(rows[3], be), q_scale=K ** -0.5,
        )

    @pytest.mark.parametrize("H,K,V", [(2, 8, 12), (3, 33, 70), (1, 1, 1), (2, 130, 40),
                                       (2, 200, 9), (4, 16, 16)])
    def test_portions(self, be, H, K, V):
        T = 45
        s = self._inputs(T, H, K, V, be, seed=31)
        want = self._oracle(*s, H, K ** -0.5)
        # junk in every slot: a portion at position 0 must not read it
        state = torch.full((3, H, V, K), 1e6).to(be[0])
        for cuts in ([T], [1] * T, [2, 17, 16, 1, 9], [16, 16, 13]):
            got, at = [], 0
            for n in cuts:
                got.append(self._run(be, [(s, at, n, 2)], state))
                at += n
            close(torch.cat(got), want, be, f32_tol=1e-5, bf16_tol=1e-5)

    @pytest.mark.parametrize("H,K,V", [(2, 16, 20), (1, 100, 64), (2, 130, 66)])
    def test_decays_of_any_size(self, be, H, K, V):
        """Decays from 1 down to 0, changing from token to token: stretches in
        which a channel's product falls below anything a quotient of products
        could bear, next to ordinary ones."""
        T = 100
        q, k, v, a = self._inputs(T, H, K, V, be, seed=33)
        z = rnd(T, H * K, seed=37, scale=4.0)
        z[20:30] = 9.0            # no decay at all
        z[40:44, ::3] = -60.0
        z[70, 1] = -300.0         # one channel forgets everything at one token
        a = torch.sigmoid(z.double()).float()
        a[75, 0] = 0.0
        want = self._oracle(q, k, v, a, H, K ** -0.5)
        state = torch.full((2, H, V, K), 1e6).to(be[0])
        for cuts in ([T], [1] * T, [3, 60, 2, 35]):
            got, at = [], 0
            for n in cuts:
                got.append(self._run(be, [((q, k, v, a), at, n, 1)], state))
                at += n
            close(torch.cat(got), want, be, f32_tol=1e-5, bf16_tol=1e-5)

    def test_unequal_batch_and_slot_reuse(self, be):
        H, K, V = 2, 16, 8
        seqs = [self._inputs(n, H, K, V, be, seed=40 + 5 * i) for i, n in enumerate((30, 12, 21))]
        wants = [self._oracle(*s, H, K ** -0.5) for s in seqs]
        state = torch.full((5, H, V, K), 7.0).to(be[0])
        slot, got = [3, 1, 4], [[], [], []]

        def step(parts):
            o = self._run(be, [(seqs[i], lo, hi - lo, slot[i]) for i, lo, hi in parts], state)
            at = 0
            for i, lo, hi in parts:
                got[i].append(o[at : at + hi - lo].cpu())
                at += hi - lo

        step([(0, 0, 17), (1, 0, 11)])
        step([(1, 11, 12), (0, 17, 18), (2, 0, 2)])
        step([(2, 2, 21), (0, 18, 30)])
        for i in range(3):
            close(torch.cat(got[i]), wants[i], be, bf16_tol=2e-5)
        slot[1], got[1] = 3, []   # a finished sequence's slot for a new one
        step([(1, 0, 12)])
        close(torch.cat(got[1]), wants[1], be, bf16_tol=2e-5)

    def test_channels_decay_apart(self, be):
        """One early write into two key channels, 700 empty tokens after it: the
        channel whose decay is close to one keeps it, the other one loses it."""
        T, K, V = 720, 8, 4
        q, k, v = torch.zeros(T, K), torch.zeros(T, K), rnd(T, V, seed=51, dtype=be[1])
        q[:, 0] = q[:, 1] = 1.0
        k[3, 0] = k[3, 1] = 4.0
        a = torch.ones(T, K)
        a[:, 0], a[:, 1] = 0.9999, 0.9
        want = self._oracle(q, k, v, a, 1, K ** -0.5)
        assert 0.8 < want[-1].max() / (np64(v)[3].max() * 4.0 * K ** -0.5) < 1.0
        state = torch.zeros(2, 1, V, K).to(be[0])
        got, at = [], 0
        for n in [300, 37, 363] + [1] * 20:
            got.append(self._run(be, [((q, k, v, a), at, n, 1)], state))
            at += n
        close(torch.cat(got), want, be, f32_tol=1e-4, bf16_tol=1e-4)


class TestRotation:
    @pytest.mark.parametrize("n,scaling", [
        (8, None), (12, {"factor": 2.5}), (16, {"factor": 1.0}),
        (8, {"factor": 3.0, "original": 40, "fast": 4.0, "slow": 0.5}),
        (32, {"factor": 8.0, "original": 300, "fast": 32.0, "slow": 1.0}),
    ])
    def test_frequencies(self, n, scaling):
        f, m = scaled_inv_freq(n, 777.0, scaling)
        want, want_m = O.frequencies({"dims": n, "base": 777.0, "scaling": scaling})
        assert np.abs(np64(f) / want - 1).max() < 1e-6 and abs(m - want_m) < 1e-12

    @pytest.mark.parametrize("D,V,rot,factor", [(12, 20, 8, 2.0), (16, 8, 16, 3.0), (9, 5, 2, 1.0),
                                                (64, 64, 64, 4.0), (10, 10, 0, 1.0)])
    def test_unnormed_heads_to_pages(self, be, D, V, rot, factor):
        """q and k turned and otherwise untouched, v as it is; positions in the
        hundreds; a token that is not cached."""
        H, G, bs, T = 4, 2, 8, 5
        pos, slots = [0, 1, 317, 5, 900], [9, 17, -1, 3, 30]
        widths = [H * D, G * D, G * V]
        x = rnd(T, sum(widths), seed=61, scale=2.0, dtype=be[1])
        q, k, v = x.split(widths, dim=1)
        r = {"dims": rot, "base": 50.0, "scaling": {"factor": factor}} if rot else None
        full = np.zeros((901, H + G, D))
        full[pos] = np.concatenate([np64(q).reshape(T, H, D), np64(k).reshape(T, G, D)], axis=1)
        turned = O.turn(full, r)[pos]
        inv = scaled_inv_freq(rot, 50.0, {"factor": factor})[0].to(be[0]) if rot else None
        kc = torch.full((5, G, bs, D), 7.0, dtype=be[1], device=be[0])
        vc = torch.full((5, G, bs, V), 7.0, dtype=be[1], device=be[0])
        xa = act(x, be)
        a, b = widths[0], widths[0] + widths[1]
        got = ops.qk_headnorm_rope_cache(
            xa[:, :a], xa[:, a:b], xa[:, b:], None, None, i64(pos, be), i32(slots, be),
            kc, vc, 1e-5, H, inv, qk_norm=False,
        )
        close(got, turned[:, :H].reshape(T, -1), be, f32_tol=1e-4, bf16_tol=1e-4)
        for t, s in enumerate(slots):
            if s >= 0:
                close(kc[s // bs, :, s % bs], turned[t, H:], be, f32_tol=1e-4)
                close(vc[s // bs, :, s % bs], np64(v)[t].reshape(G, V), be)
        untouched = [s for s in range(5 * bs) if s not in slots]
        assert all((kc[s // bs, :, s % bs] == 7.0).all() for s in untouched)


class TestLatentRows:
    YARN = {"factor": 3.0, "original": 40, "fast": 4.0, "slow": 0.5}

    @pytest.mark.parametrize("kv_rank,rot,extra", [(16, 8, 3), (72, 20, 0), (260, 64, 8), (8, 2, 1)])
    def test_norm_turn_and_scatter(self, be, kv_rank, rot, extra):
        eps, bs, T = 1e-5, 8, 6
        row = rnd(T, 24 + kv_rank + rot + extra, seed=71, scale=2.0, dtype=be[1])
        kw = rnd(kv_rank, seed=72) + 1.0
        pos, slots = [0, 1, 2, 500, 31, 7], [9, 17, -1, 3, 40, 8]
        inv, m = scaled_inv_freq(rot, 777.0, self.YARN)
        cache = torch.full((6, 1, bs, kv_rank + rot), 7.0, dtype=be[1], device=be[0])
        out = ops.latent_norm_rope_cache(
            act(row, be)[:, 24:], 0, kv_rank, rot, None, f32(kw, be), i64(pos, be),
            i32(slots, be), cache, eps, inv.to(be[0]), pairs=False, rot_mult=m,
        )
        assert out is None
        c = O.rms(np64(row)[:, 24 : 24 + kv_rank], eps) * np64(kw)
        full = np.zeros((501, rot))
        full[pos] = np64(row)[:, 24 + kv_rank : 24 + kv_rank + rot]
        kr = O.turn(full, {"dims": rot, "base": 777.0, "scaling": self.YARN})[pos]
        flat = cache.view(-1, kv_rank + rot)
        for t, s in enumerate(slots):
            if s >= 0:
                close(flat[s, :kv_rank], c[t], be)
                close(flat[s, kv_rank:], kr[t], be, f32_tol=1e-4)
        assert (flat[[s for s in range(48) if s not in slots]] == 7.0).all()

    @pytest.mark.parametrize("T,H,K,N,tail", [(5, 3, 16, 24, 8), (70, 2, 40, 300, 4), (1, 4, 24, 70, 10),
                                              (2100, 2, 128, 192, 64), (130, 2, 20, 36, 6)])
    def test_folded_queries(self, be, T, H, K, N, tail):
        """Per-head product with the turned tail, queries being a column slice
        of a wider projection."""
        x = rnd(T, H * (K + tail) + 8, seed=73, dtype=be[1])
        w = rnd(H, N, K, seed=74, scale=K ** -0.5, dtype=be[1])
        inv, m = scaled_inv_freq(tail, 777.0, self.YARN)
        xh = np64(x)[:, : H * (K + tail)].reshape(T, H, K + tail)
        tl = O.turn(xh[..., K:], {"dims": tail, "base": 777.0, "scaling": self.YARN})
        want = np.concatenate([np.einsum("thk,hnk->thn", xh[..., :K], np64(w)), tl], axis=-1)
        got = ops.head_matmul_rope(
            act(x, be)[:, : H * (K + tail)], act(w, be), H, tail, i64(torch.arange(T), be),
            inv.to(be[0]), torch.float32, pairs=False, rot_mult=m,
        )
        close(got, want.reshape(T, -1), be, f32_tol=3e-4, bf16_tol=3e-4)


def paged(rows_per_seq, bs, be, seed=0):
    """Scatter each sequence's [ctx, G, cols] rows over shuffled pages of one
    pool that is full of junk."""
    nb = [-(-r.shape[0] // bs) for r in rows_per_seq]
    total = sum(nb) + 3
    _, G, cols = rows_per_seq[0].shape
    perm = (torch.randperm(total - 1, generator=torch.Generator().manual_seed(seed)) + 1).tolist()
    cache = torch.full((total, G, bs, cols), 3.0)
    tables = torch.zeros(len(rows_per_seq), max(nb), dtype=torch.int32)
    for s, r in enumerate(rows_per_seq):
        for b in range(nb[s]):
            tables[s, b] = perm.pop()
            part = r[b * bs : (b + 1) * bs]
            cache[tables[s, b], :, : part.shape[0]] = part.transpose(0, 1)
    return cache.to(be[1]).to(be[0]), tables.to(be[0])


class TestKeptFirstPositions:
    """ctx_attention_f32 with a window and kept first positions."""

    def run(self, be, qs, ks, vs, scale, window, keep, bs):
        """qs [n, H, D] (the last n positions), ks [ctx, G, D], vs [ctx, G, V]
        per sequence."""
        H = qs[0].shape[1]
        kc, tables = paged(ks, bs, be, seed=1)
        vc, _ = paged(vs, bs, be, seed=1)
        cu = np.cumsum([0] + [q.shape[0] for q in qs])
        got = ops.ctx_attention_f32(
            f32(torch.cat([q.reshape(q.shape[0], -1) for q in qs]), be), kc, vc, tables,
            i32(cu, be), i32([k.shape[0] for k in ks], be), scale,
            max(q.shape[0] for q in qs), H, out_dtype=be[1], window=window, keep_first=keep,
        )
        want = []
        for q, k, v in zip(qs, ks, vs):
            n, ctx, G = q.shape[0], k.shape[0], k.shape[1]
            ok = O.visible(ctx, {"size": window, "keep_first": keep} if window else None)[ctx - n :]
            k, v = np64(k.to(be[1])), np64(v.to(be[1]))
            o = np.zeros((n, H, v.shape[-1]))
            for h in range(H):
                g = h // (H // G)
                s = np.where(ok, np64(q)[:, h] @ k[:, g].T * scale, -np.inf)
                o[:, h] = O.softmax(s) @ v[:, g]
            want.append(o.reshape(n, -1))
        return got, np.concatenate(want)

    @pytest.mark.parametrize("H,G,D,V,window,keep,bs", [
        (4, 2, 12, 20, 9, 3, 16), (6, 3, 64, 64, 40, 70, 16), (2, 1, 8, 8, 1, 1, 8),
        (8, 1, 40, 24, 64, 64, 16), (3, 3, 100, 130, 130, 5, 64), (2, 2, 16, 16, 33, 300, 16),
        (4, 4, 32, 32, 20, 0, 16), (4, 2, 16, 16, 0, 6, 16), (16, 1, 128, 128, 70, 130, 32),
    ])
    def test_portions_and_decode_batched(self, be, H, G, D, V, window, keep, bs):
        ctxs, nqs = [260, 70, 1, 33, 400], [260, 5, 1, 1, 37]
        ks = [rnd(c, G, D, seed=81 + i) for i, c in enumerate(ctxs)]
        vs = [rnd(c, G, V, seed=91 + i) for i, c in enumerate(ctxs)]
        qs = [rnd(n, H, D, seed=101 + i) for i, n in enumerate(nqs)]
        got, want = self.run(be, qs, ks, vs, 1.5 * D ** -0.5, window, keep, bs)
        close(got, want, be)
        # decode only: one token per sequence
        got, want = self.run(be, [q[-1:] for q in qs], ks, vs, 1.5 * D ** -0.5, window, keep, bs)
        close(got, want, be)

    @pytest.mark.parametrize("decode", [False, True])
    @pytest.mark.parametrize("window,keep,bs", [(40, 20, 16), (16, 16, 16), (33, 64, 16), (64, 65, 8),
                                                (130, 1, 64), (20, 130, 16)])
    def test_needles(self, be, window, keep, bs, decode):
        """One key stands out by its score and its value: at the kept range's
        last position and the first behind it, at the window's last position
        and the first outside, at position 0 — far from and close to the
        query."""
        H, G, D = 4, 2, 16
        n = 1 if decode else 5
        for ctx in (keep + window + 1, keep + window + 200, window + keep // 2 + 1):
            for needle in {0, keep - 1, keep, ctx - window, ctx - window - 1, ctx - 1}:
                if not 0 <= needle < ctx:
                    continue
                k, v = rnd(ctx, G, D, seed=111, scale=0.1), rnd(ctx, G, 8, seed=112, scale=0.1)
                k[needle] = 0.0
                k[needle, :, 2] = 5.0
                v[needle] = 6.0
                q = rnd(n, H, D, seed=113, scale=0.1)
                q[:, :, 2] = 4.0
                got, want = self.run(be, [q], [k], [v], 1.0, window, keep, bs)
                close(got, want, be)
                seen = got.float().cpu().view(n, H, 8)[-1]
                if needle < keep or needle >= ctx - window:
                    assert (seen > 5.0).all(), (ctx, needle)
                else:
                    assert (seen.abs() < 1.0).all(), (ctx, needle)


class TestRouter:
    @pytest.mark.parametrize("E,top,W", [(5, 2, 32), (18, 3, 100), (70, 4, 64), (3, 3, 16), (5, 1, 48),
                                         (1, 1, 8), (130, 64, 24)])
    def test_softmax_over_the_chosen(self, be, E, top, W):
        T = 9
        h = rnd(T, W, seed=121, dtype=be[1])
        r, b = rnd(E, W, seed=122, scale=W ** -0.5), rnd(E, seed=123, scale=0.7)
        z = np64(h) @ np64(r).T + np64(b)
        want = O.routing(z, top)
        idx, w, dense, lg = ops.route_tokens(
            act(h, be), f32(r, be), top, dense=True, want_logits=True, over_chosen=True,
            bias=f32(b, be),
        )
        close(lg, z, be, bf16_tol=2e-5)
        close(dense, want, be, bf16_tol=2e-5)
        got = np.zeros_like(want)
        np.put_along_axis(got, np64(idx).astype(np.int64), np64(w), axis=1)
        close(torch.from_numpy(got), want, be, bf16_tol=2e-5)
        # the same choice on given logits
        i2, w2, d2 = ops.router_topk(f32(torch.from_numpy(z), be), top, dense=True, over_chosen=True)
        close(d2, want, be, bf16_tol=2e-5)

    def test_logits_far_apart(self, be):
        """Scores of all experts together would underflow; the choice and the
        second weight must not depend on them. The bias alone decides."""
        h, r = torch.zeros(2, 8), torch.zeros(4, 8)
        b = torch.tensor([-300.0, 250.0, -290.0, -299.0])
        idx, w, dense, _ = ops.route_tokens(act(h, be), f32(r, be), 3, dense=True,
                                            over_chosen=True, bias=f32(b, be))
        assert idx[0].tolist() == [1, 2, 3]
        assert torch.allclose(w[0].cpu(), torch.tensor([1.0, 0.0, 0.0]))
        b = torch.tensor([-300.0, -299.0, -390.0, -600.0])
        idx, w, dense, _ = ops.route_tokens(act(h, be), f32(r, be), 2, dense=True,
                                            over_chosen=True, bias=f32(b, be))
        assert idx[0].tolist() == [1, 0]
        close(w, np.repeat(O.softmax(np.array([[-299.0, -300.0]])), 2, axis=0), be)

    @pytest.mark.parametrize("E,top", [(5, 2), (3, 3), (1, 1), (6, 1)])
    @pytest.mark.parametrize("T", [3, 1500])
    def test_experts_in_both_forms(self, be, E, top, T):
        """The all-experts form (few tokens) and the sorted form (many), summed
        by the mixture itself and left as rows for the residual kernel."""
        W, ff = 24, 16
        cfg = O.make_config([O.attention_layer(mlp=O.moe(E, top, ff))], width=W)
        sd = O.random_weights(cfg, seed=131, dtype=be[1])
        mod = SoftmaxRoutedMoE(
            W, SoftmaxMoESpec(experts=E, top=top, ff=ff, over_chosen=True, router_bias=True), be[1]
        )
        mod.load(lambda n: sd[n], "l0.mlp.")
        mod.to(be[0])
        h = rnd(T, W, seed=132, dtype=be[1])
        want = O.experts(np64(h), {k: np64(v) for k, v in sd.items()}, "l0.mlp.",
                         cfg["layers"][0]["mlp"])
        close(mod(act(h, be)), want, be, f32_tol=1e-4)
        y = mod.rows(act(h, be))
        assert (y.index is None) == (T <= mod.dense_max_tokens)
        x = torch.zeros(T, W, device=be[0])
        ops.add_rms_norm_f32res(
            x, None, 1e-5, 1.0, be[1], d1=y.y, d1_index=y.index, d1_weights=y.weights,
            d1_top=y.top, want_out=False,
        )
        close(x, want, be, f32_tol=1e-4)
