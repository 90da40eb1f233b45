"""The mechanisms of the Mededra design one at a time, against the float64
functions in mededra_oracle.py: the plain torch form of every op on the CPU,
the HIP kernel under ``-m gpu``.
"""

import math
import os
import sys

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import mededra_oracle as O  # noqa: E402

from kserve_amd import ops  # noqa: E402
from kserve_amd.ops import torch_ref  # noqa: E402

DEVICES = [
    pytest.param("cpu", id="cpu"),
    pytest.param("cuda", id="gpu", marks=pytest.mark.gpu),
]
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(params=DEVICES)
def dev(request):
    if request.param == "cuda":
        assert ops.has_native_seq(), "kserve_amd_seq_C must be built on a GPU box"
    return request.param


def rnd(*shape, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g) * scale


def np64(t):
    return t.detach().double().cpu().numpy()


def maxdiff(got, want):
    return float(np.abs(np64(got) - want).max())


class Meta:
    def __init__(self, **kw):
        self.__dict__.update(kw)


class Pages:
    """Scattered pages and state slots for a few sequences; ``meta`` describes
    one step's portions [(sequence, start, length)]."""

    def __init__(self, totals, bs, dev, seed=1):
        self.bs, self.dev = bs, dev
        need = [-(-n // bs) for n in totals]
        perm = torch.randperm(sum(need) + 3, generator=torch.Generator().manual_seed(seed)) + 1
        self.num_blocks = sum(need) + 5
        self.tables, at = [], 0
        for n in need:
            self.tables.append(perm[at : at + n])
            at += n
        self.width = max(need)

    def meta(self, parts):
        pos, seq, cu, slots, ctx, slot_of = [], [], [0], [], [], []
        bt = torch.zeros(len(parts), self.width, dtype=torch.int32)
        for i, (s, a, n) in enumerate(parts):
            p = torch.arange(a, a + n)
            pos.append(p)
            seq += [i] * n
            cu.append(cu[-1] + n)
            slots.append(self.tables[s][p // self.bs] * self.bs + p % self.bs)
            bt[i, : len(self.tables[s])] = self.tables[s]
            ctx.append(a + n)
            slot_of.append(s + 1)
        i32 = dict(dtype=torch.int32, device=self.dev)
        return torch.cat(pos).to(self.dev), Meta(
            slot_mapping=torch.cat(slots).to(torch.int32).to(self.dev),
            seq_of_token=torch.tensor(seq, **i32), cu_seqlens=torch.tensor(cu, **i32),
            block_tables=bt.to(self.dev), context_lens=torch.tensor(ctx, **i32),
            max_seqlen=max(n for _, _, n in parts),
            state_slots=torch.tensor(slot_of, **i32),
        )


def layer_cache(mod, pages, dtype, dev, junk=True):
    """The caches the model runner would allocate for one mixer, full of
    large numbers where nothing may be read before it is written."""
    from kserve_amd.models.mixers import LayerCache

    def alloc(shape, dt):
        return torch.full(shape, 1e4 if junk else 0.0, dtype=dt, device=dev)

    k = v = ks = conv = ssm = None
    st = mod.state_shapes()
    if hasattr(mod, "kv_shape"):
        g, d, dv = mod.kv_shape()
        k = alloc((pages.num_blocks, g, pages.bs, d), dtype)
        v = alloc((pages.num_blocks, g, pages.bs, dv), dtype) if dv else None
        if st.get("k_scale"):
            ks = alloc((pages.num_blocks, pages.bs), torch.float32)
    slots = len(pages.tables) + 1
    if st.get("conv"):
        conv = alloc((slots, *st["conv"][0]), st["conv"][1])
    if st.get("ssm"):
        ssm = alloc((slots, *st["ssm"][0]), torch.float32)
    return LayerCache(k, v, conv, ssm, ks)


def run_mixer(mod, hs, bs, dtype, dev, schedule):
    """hs: input rows per sequence; schedule: steps of (sequence, count).
    Returns the outputs per sequence."""
    pages = Pages([h.shape[0] for h in hs], bs, dev)
    cache = layer_cache(mod, pages, dtype, dev)
    at = [0] * len(hs)
    out = [[] for _ in hs]
    for step in schedule:
        parts = [(s, at[s], n) for s, n in step]
        pos, meta = pages.meta(parts)
        x = torch.cat([hs[s][a : a + n] for s, a, n in parts]).to(dev)
        y = mod(x, pos, cache, meta).float().cpu()
        off = 0
        for s, a, n in parts:
            out[s].append(y[off : off + n])
            off += n
            at[s] += n
    assert at == [h.shape[0] for h in hs]
    return [torch.cat(o) for o in out]


class TestYarn:
    @pytest.mark.parametrize("dims,base,scaling", [
        (16, 100.0, None), (16, 100.0, O.yarn()), (48, 5e4, O.yarn(8.0, 4096, 32.0, 1.0)),
        (8, 10.0, O.yarn(2.0, 10, 30.0, 20.0)),   # both ends clipped to 0
        (2, 50.0, O.yarn(4.0, 1000, 1.5, 1.2)),
    ])
    def test_frequencies(self, dims, base, scaling):
        f, m = torch_ref.yarn_inv_freq(dims, base, scaling)
        wf, wm = O.rotary_frequencies(O.rot(dims, base, scaling))
        assert np.abs(np64(f) / wf - 1).max() < 1e-6 and abs(m - wm) < 1e-12
        if scaling is None:
            assert m == 1.0


class TestBuckets:
    @pytest.mark.parametrize("B,D", [(8, 30), (32, 100), (2, 5), (6, 1000), (16, 9)])
    def test_every_distance(self, B, D):
        got = torch_ref.distance_buckets(3 * D, B, float(D)).tolist()
        assert got == [O.bucket(n, B, D) for n in range(3 * D)]
        assert got[-1] == B - 1 and got[D] == B - 1


class TestConvNoActivation:
    @pytest.mark.parametrize("dtype", DTYPES)
    @pytest.mark.parametrize("taps,channels", [(2, 8), (4, 64), (6, 5)])
    def test_portions(self, dev, dtype, taps, channels):
        T = 23
        x = rnd(T, channels, seed=4).to(dtype)
        w = rnd(channels, taps, seed=5, scale=0.5)
        want = O.conv(np64(x), np64(w))
        state = torch.full((3, taps - 1, channels), 50.0, dtype=dtype).to(dev)
        i32 = dict(dtype=torch.int32, device=dev)
        for cuts in ([T], [1] * T, [2, 2, 1, 9, 9]):
            outs, at = [], 0
            for n in cuts:
                outs.append(ops.causal_conv_silu(
                    x[at : at + n].to(dev), w.to(dev), None, state,
                    torch.arange(at, at + n, device=dev), torch.zeros(n, **i32),
                    torch.tensor([0, n], **i32), torch.tensor([2], **i32), silu=False))
                at += n
            assert maxdiff(torch.cat(outs), want) < 1e-5, cuts


class TestHeadNormRotatePairs:
    @pytest.mark.parametrize("in_dtype,cache_dtype", [
        (torch.float32, torch.float32), (torch.float32, torch.bfloat16),
        (torch.bfloat16, torch.bfloat16)])
    @pytest.mark.parametrize("H,G,D,V,rot", [(4, 2, 12, 20, 8), (2, 1, 7, 5, 6),
                                             (3, 3, 64, 128, 64), (2, 2, 8, 8, 0)])
    def test_against_oracle(self, dev, in_dtype, cache_dtype, H, G, D, V, rot):
        T, bs = 9, 4
        wide = rnd(T, 2 * H * D + 2 * G * D + G * V, seed=2).to(in_dtype)
        a, b = 2 * H * D, 2 * H * D + 2 * G * D
        qw, kw = 1 + 0.2 * rnd(D, seed=3), 1 + 0.2 * rnd(D, seed=4)
        r = O.rot(rot, 40.0, O.yarn()) if rot else None
        inv, mult = (torch_ref.yarn_inv_freq(rot, 40.0, O.yarn()) if rot else (None, 1.0))
        pages = Pages([T], bs, dev)
        pos, meta = pages.meta([(0, 0, T)])
        kc = torch.zeros(pages.num_blocks, G, bs, 2 * D, dtype=cache_dtype, device=dev)
        vc = torch.zeros(pages.num_blocks, G, bs, V, dtype=cache_dtype, device=dev)
        x = wide.to(dev)
        q = ops.qk_headnorm_rope_cache(
            x[:, :a], x[:, a:b], x[:, b:], qw.to(dev), kw.to(dev), pos,
            meta.slot_mapping, kc, vc, 1e-5, 2 * H,
            inv.to(dev) if inv is not None else None, pairs=True, rot_mult=mult, maps=2)
        n = np64(wide)
        wq = O.rotate_pairs(O.rms(n[:, :a].reshape(T, H, 2, D), 1e-5) * np64(qw), r)
        wk = O.rotate_pairs(O.rms(n[:, a:b].reshape(T, G, 2, D), 1e-5) * np64(kw), r)
        assert maxdiff(q, wq.reshape(T, -1)) < 2e-5
        tol = 3e-2 if cache_dtype == torch.bfloat16 else 2e-5
        t = pages.tables[0]
        for p in range(T):
            assert maxdiff(kc[t[p // bs], :, p % bs], wk[p].reshape(G, 2 * D)) < tol
            assert maxdiff(vc[t[p // bs], :, p % bs], n[p, b:].reshape(G, V)) < tol


class TestDiffCombine:
    @pytest.mark.parametrize("dtype", DTYPES)
    @pytest.mark.parametrize("H,V", [(1, 1), (3, 20), (4, 96), (2, 256)])
    def test_against_oracle(self, dev, dtype, H, V):
        T = 7
        o = rnd(T, H * 2 * V, seed=6)
        lam = torch.tensor([0.37])
        a = np64(o).reshape(T, H, 2, V)
        want = O.rms(a[:, :, 0] - 0.37 * a[:, :, 1], 1e-5) * 0.8
        got = ops.diff_combine(o.to(dev), lam.to(dev), H, 1e-5, 0.8, dtype)
        assert got.dtype == dtype
        assert maxdiff(got, want.reshape(T, -1)) < (2e-2 if dtype == torch.bfloat16 else 2e-5)


class TestPostGroupNorm:
    @pytest.mark.parametrize("dtype", DTYPES)
    @pytest.mark.parametrize("width,groups", [(24, 1), (24, 2), (24, 3), (30, 5), (40, 8),
                                              (2048, 4), (35, 7), (1024, 2), (64, 64)])
    @pytest.mark.parametrize("form", ["one", "two", "none"])
    def test_against_oracle(self, dev, dtype, width, groups, form):
        T, eps = 5, 1e-5
        x = rnd(T, width, seed=1)
        d = rnd(T, width + 8, seed=2, scale=0.01).to(dtype)[:, :width]
        d2 = rnd(T, width, seed=3, scale=7.0).to(dtype)
        w, pw, pw2, nw = (1 + 0.2 * rnd(width, seed=4 + i) for i in range(4))
        if form == "none":
            new = np64(x)
        else:
            y = np64(d)
            if form == "two":
                y = 0.5 * (O.rms(y, eps) * np64(pw) + O.rms(np64(d2), eps) * np64(pw2))
            new = np64(x) + O.group_rms(y, groups, eps) * np64(w)
        kw = {}
        if form == "two":
            kw = dict(delta2=d2.to(dev), pre_w=pw.to(dev), pre_w2=pw2.to(dev))
        for nxt in (None, nw):
            res = x.clone().to(dev)
            got = ops.post_group_norm_add(
                res, None if form == "none" else d.to(dev), w.to(dev), groups, eps,
                dtype, next_weight=nxt.to(dev) if nxt is not None else None, **kw)
            assert maxdiff(res, new) < 2e-5
            want = new if nxt is None else O.group_rms(new, groups, eps) * np64(nw)
            assert got.dtype == dtype
            assert maxdiff(got, want) < (4e-2 if dtype == torch.bfloat16 else 3e-5)
        res = x.clone().to(dev)
        assert ops.post_group_norm_add(
            res, None if form == "none" else d.to(dev), w.to(dev), groups, eps, dtype,
            want_out=False, **kw) is None
        assert maxdiff(res, new) < 2e-5

    def test_groups_are_separate(self, dev):
        """One huge group does not shrink the others."""
        x = torch.zeros(1, 16)
        d = torch.ones(1, 16)
        d[0, :4] = 1e4
        res = x.clone().to(dev)
        ops.post_group_norm_add(res, d.to(dev), torch.ones(16).to(dev), 4, 1e-5, torch.float32)
        assert (res.cpu() - 1).abs().max() < 1e-3


class TestSigmoidGateNorm:
    @pytest.mark.parametrize("dtype", DTYPES)
    @pytest.mark.parametrize("groups,size", [(2, 12), (3, 5), (4, 64), (1, 1100)])
    def test_against_oracle(self, dev, dtype, groups, size):
        T, inner = 6, groups * size
        y = rnd(T, inner, seed=8, scale=3.0)
        z = rnd(T, inner + 4, seed=9, scale=2.0).to(dtype)[:, 4:]
        w = 1 + 0.1 * rnd(size, seed=10)
        want = O.rms(np64(y).reshape(T, groups, size), 1e-5) * np64(w)
        want = want.reshape(T, inner) * O.sigmoid(np64(z))
        got = ops.gated_group_rms_norm(y.to(dev), z.to(dev), w.to(dev), 1e-5, groups, dtype,
                                       gate_after=True, gate_sigmoid=True)
        assert maxdiff(got, want) < (3e-2 if dtype == torch.bfloat16 else 1e-5)


class TestChannelDelta:
    def _rows(self, T, H, G, K, V, seed):
        qkv = rnd(T, 2 * G * K + H * V, seed=seed)
        a = rnd(T, H * K + 5, seed=seed + 1, scale=2.0)
        b = rnd(T, H + 3, seed=seed + 2, scale=2.0)
        a_log = torch.linspace(-2.0, 0.7, H)
        dt = torch.linspace(-2.0, 1.0, H * K)
        return qkv, a, b, a_log, dt

    @pytest.mark.parametrize("dtype", DTYPES)
    @pytest.mark.parametrize("H,G,K,V", [(2, 2, 8, 12), (4, 2, 16, 5), (3, 1, 33, 70),
                                         (1, 1, 1, 1), (2, 1, 130, 40), (2, 2, 200, 9)])
    def test_recurrence_in_portions(self, dev, dtype, H, G, K, V):
        """Unit norms, per-channel decays and the scan, fed whole, token by
        token and in uneven portions into slots full of junk."""
        T = 45
        qkv, a, b, a_log, dt = self._rows(T, H, G, K, V, 3)
        a, b = a.to(dtype)[:, 5:], b.to(dtype)[:, 2 : 2 + H]
        n = np64(qkv)
        q = O.unit(n[:, : G * K].reshape(T, G, K)) * K ** -0.5
        k = O.unit(n[:, G * K : 2 * G * K].reshape(T, G, K))
        v = n[:, 2 * G * K :].reshape(T, H, V)
        g = np.exp(-np.exp(np64(a_log))[None, :, None]
                   * O.softplus(np64(a) + np64(dt)).reshape(T, H, K))
        want = O.delta_rule(q, k, v, g, O.sigmoid(np64(b))).reshape(T, -1)
        state = torch.full((3, H, V, K), 1e6).to(dev)
        i32 = dict(dtype=torch.int32, device=dev)
        for cuts in ([T], [1] * T, [2, 17, 16, 1, 9], [16, 16, 13]):
            outs, at = [], 0
            for c in cuts:
                rows = qkv[at : at + c].clone().to(dev)
                gg = ops.delta_unit_decay(rows, G, K, K ** -0.5, 1e-6,
                                          a[at : at + c].to(dev), a_log.to(dev), dt.to(dev))
                assert maxdiff(gg, g[at : at + c].reshape(c, -1)) < 1e-5
                outs.append(ops.linear_scan(
                    rows[:, : G * K], rows[:, G * K : 2 * G * K], rows[:, 2 * G * K :],
                    state, torch.arange(at, at + c, device=dev),
                    torch.tensor([0, c], **i32), torch.tensor([2], **i32), G,
                    b_raw=b[at : at + c].to(dev), channel_decay=gg))
                at += c
            assert maxdiff(torch.cat(outs), want) < 1e-4 * max(1.0, np.abs(want).max()), cuts

    def test_channels_decay_apart(self, dev):
        """Two key channels written once, then one is forgotten at once and
        the other kept for 600 tokens."""
        K, V, T = 4, 3, 640
        q, k, v = torch.zeros(T, K), torch.zeros(T, K), torch.zeros(T, V)
        k[2, 0], v[2] = 1.0, torch.tensor([1.0, 2.0, 3.0])
        k[3, 1], v[3] = 1.0, torch.tensor([-5.0, 4.0, 0.5])
        q[:, 0] = 1.0
        q[1::2, 0], q[1::2, 1] = 0.0, 1.0
        g = torch.ones(T, K)
        g[:, 1] = 0.1
        beta = torch.full((T, 1), 40.0)      # sigmoid = 1
        want = O.delta_rule(np64(q)[:, None], np64(k)[:, None], np64(v)[:, None],
                            np64(g)[:, None], O.sigmoid(np64(beta))).reshape(T, V)
        assert abs(want[-2] - [1, 2, 3]).max() < 1e-9 and abs(want[-1]).max() < 1e-9
        state = torch.full((2, 1, V, K), 9.0).to(dev)
        i32 = dict(dtype=torch.int32, device=dev)
        outs, at = [], 0
        for c in [300, 2, 318] + [1] * 20:
            sl = slice(at, at + c)
            outs.append(ops.linear_scan(
                q[sl].to(dev), k[sl].to(dev), v[sl].to(dev), state,
                torch.arange(at, at + c, device=dev), torch.tensor([0, c], **i32),
                torch.tensor([1], **i32), 1, b_raw=beta[sl].to(dev),
                channel_decay=g[sl].to(dev)))
            at += c
        assert maxdiff(torch.cat(outs), want) < 1e-5

    @pytest.mark.parametrize("dtype", DTYPES)
    @pytest.mark.parametrize("conv", [1, 4])
    def test_mixer(self, dev, dtype, conv):
        """The whole sublayer in two sequences that share steps."""
        from kserve_amd.engine.config import DeltaMixerSpec
        from kserve_amd.models.mixers import ChannelDeltaMixer

        W = 24
        layer = O.parallel_layer(d_heads=4, d_kv_heads=2, d_dim=12, d_vdim=20, conv=conv,
                                 a_rank=3, g_rank=9)
        sd = O.random_weights(O.make_config([layer], width=W), seed=5, dtype=dtype)
        m = layer["mixer"]["right"]
        mod = ChannelDeltaMixer(W, DeltaMixerSpec.from_dict(m, channel_decay=True), 1e-5, dtype)
        mod.load(lambda n: sd[n], "l0.mix.right.")
        mod.to(dev)
        hs = [rnd(n, W, seed=n).to(dtype) for n in (41, 18)]
        sched = [[(0, 20), (1, 2)], [(0, 1), (1, 9)], [(1, 1), (0, 2)]] + \
                [[(0, 1), (1, 1)]] * 6 + [[(0, 12)]]
        outs = run_mixer(mod, hs, 16, dtype, dev, sched)
        Wn = {k: np64(v) for k, v in sd.items()}
        for h, o in zip(hs, outs):
            want = O.delta(np64(h), Wn, "l0.mix.right.", m, 1e-5)
            tol = 6e-2 if dtype == torch.bfloat16 else 1e-4
            assert maxdiff(o, want) < tol * np.abs(want).max()


class TestDifferential:
    @pytest.mark.parametrize("dtype", DTYPES)
    @pytest.mark.parametrize("H,G,D,V,window,bs,conv,cap", [
        (4, 2, 12, 20, 9, 16, 3, 5.0), (2, 2, 8, 16, 16, 8, 4, 2.0),
        (3, 1, 7, 5, 17, 4, 2, 30.0), (1, 1, 4, 4, 1, 16, 1, 1.0),
        (20, 1, 16, 32, 40, 16, 2, 3.0), (2, 1, 64, 128, 50, 16, 4, 8.0),
        (2, 1, 136, 40, 30, 16, 2, 4.0), (4, 4, 8, 8, 0, 16, 0, 0.0)])
    def test_mixer(self, dev, dtype, H, G, D, V, window, bs, conv, cap):
        """Prompt portions, tokens decoded alone and both in one step;
        windows below, at and off the page size; more than 16 query heads per
        group; a key row too wide for the decode form; no window, no
        convolution, no cap."""
        from kserve_amd.engine.config import DifferentialMixerSpec
        from kserve_amd.models.mixers import DifferentialAttention

        W = 24
        layer = O.attention_layer(H, G, D, V, conv or 1, 0.25, 0.7, cap, window,
                                  rotation=O.rot(2 * (D // 4), 60.0, O.yarn()))
        layer["mixer"]["conv"] = conv
        if not window:
            layer["mixer"].pop("mask")
        sd = O.random_weights(O.make_config([layer], width=W), seed=7, dtype=dtype) if conv \
            else self._no_conv_weights(layer, W, dtype)
        spec = DifferentialMixerSpec.from_dict(layer["mixer"])
        assert spec.window == window
        mod = DifferentialAttention(W, spec, 1e-5, dtype)
        mod.load(lambda n: sd[n], "l0.mix.")
        mod.to(dev)
        hs = [rnd(n, W, seed=n).to(dtype) for n in (75, 33)]
        sched = [[(0, 31), (1, 2)], [(0, 1), (1, 17)], [(0, 2), (1, 1)]] + \
                [[(0, 1), (1, 1)]] * 13 + [[(0, 16)], [(0, 1)], [(0, 11)]]
        outs = run_mixer(mod, hs, bs, dtype, dev, sched)
        Wn = {k: np64(v) for k, v in sd.items()}
        for h, o in zip(hs, outs):
            want = O.differential(np64(h), Wn, "l0.mix.", layer["mixer"], 1e-5)
            if dtype == torch.float32:
                assert maxdiff(o, want) < 2e-4 * np.abs(want).max()
            else:
                # the difference of the maps is divided by its own RMS, which
                # amplifies rounding where they nearly cancel
                err = np.abs(np64(o) - want).max(axis=1) / np.abs(want).max()
                assert np.mean(err < 6e-2) > 0.9 and np.median(err) < 3e-2

    def _no_conv_weights(self, layer, W, dtype):
        layer["mixer"]["conv"] = 1
        sd = O.random_weights(O.make_config([layer], width=W), seed=7, dtype=dtype)
        layer["mixer"]["conv"] = 0
        return {k: v for k, v in sd.items() if not k.endswith(".conv")}

    def test_lambda(self):
        from kserve_amd.engine.config import DifferentialMixerSpec
        from kserve_amd.models.mixers import DifferentialAttention

        layer = O.attention_layer()
        sd = O.random_weights(O.make_config([layer]), seed=8)
        mod = DifferentialAttention(32, DifferentialMixerSpec.from_dict(layer["mixer"]), 1e-5,
                                    torch.float32)
        mod.load(lambda n: sd[n], "l0.mix.")
        want = O.lam({k: np64(v) for k, v in sd.items()}, "l0.mix.", 0.2)
        assert abs(float(mod.lam) - want) < 1e-5
        assert abs(want - 0.2) > 1e-3


class TestTalkingHeads:
    @pytest.mark.parametrize("dtype", DTYPES)
    @pytest.mark.parametrize("H,G,D,window,bs,bias_max,buckets", [
        (4, 2, 8, 9, 16, 30, 8), (8, 4, 64, 16, 8, 20, 32), (1, 1, 4, 1, 16, 20, 4),
        (6, 3, 20, 33, 4, 25, 6), (12, 6, 128, 40, 16, 60, 16), (18, 1, 16, 70, 16, 50, 8),
        (20, 20, 32, 21, 16, 64, 8), (32, 8, 128, 50, 16, 45, 32), (40, 10, 8, 30, 16, 33, 8),
        (3, 3, 200, 0, 16, 40, 8), (16, 4, 64, 64, 16, 100, 32), (36, 36, 70, 25, 16, 30, 8)])
    def test_mixer(self, dev, dtype, H, G, D, window, bs, bias_max, buckets):
        """Prompt portions, tokens decoded alone and both in one step, for
        head counts from 1 to 40 in key groups of 1 to 18, head sizes from 4
        to 200, windows below and above the bias's last distance."""
        from kserve_amd.engine.config import TalkingMixerSpec
        from kserve_amd.models.mixers import TalkingHeadsAttention

        W = 24
        layer = O.parallel_layer(heads=H, kv_heads=G, dim=D, scale=1.5 * D ** -0.5,
                                 window=window, bias_max=bias_max, buckets=buckets)
        if not window:
            layer["mixer"]["left"].pop("mask")
        sd = O.random_weights(O.make_config([layer], width=W), seed=9, dtype=dtype)
        m = layer["mixer"]["left"]
        mod = TalkingHeadsAttention(W, TalkingMixerSpec.from_dict(m), 1e-5, dtype)
        mod.load(lambda n: sd[n], "l0.mix.left.")
        mod.to(dev)
        hs = [rnd(n, W, seed=n).to(dtype) for n in (75, 33)]
        sched = [[(0, 31), (1, 2)], [(0, 1), (1, 17)], [(0, 2), (1, 1)]] + \
                [[(0, 1), (1, 1)]] * 13 + [[(0, 16)], [(0, 1)], [(0, 11)]]
        outs = run_mixer(mod, hs, bs, dtype, dev, sched)
        Wn = {k: np64(v) for k, v in sd.items()}
        for h, o in zip(hs, outs):
            want = O.talking(np64(h), Wn, "l0.mix.left.", m, 1e-5)
            tol = 6e-2 if dtype == torch.bfloat16 else 1e-4
            assert maxdiff(o, want) < tol * np.abs(want).max()

    def test_far_key_stands_out_through_a_split_decode(self, dev):
        """500 tokens of which one key far back carries every head's score,
        one position inside and outside the window, decoded with the keys
        split over blocks and in a prompt portion; the oracle's own output
        changes where the key is visible."""
        from kserve_amd.engine.config import TalkingMixerSpec
        from kserve_amd.models.mixers import TalkingHeadsAttention

        W, T, window, needle = 16, 500, 300, 100
        layer = O.parallel_layer(heads=4, kv_heads=2, dim=8, scale=4.0, window=window,
                                 bias_max=200, buckets=16)
        sd = O.random_weights(O.make_config([layer], width=W), seed=10)
        p = "l0.mix.left."
        sd[p + "talk"] = torch.eye(4) + 0.05 * rnd(4, 4, seed=3)
        sd[p + "k"][:, 0] = 0.0
        sd[p + "k"][0, 0] = sd[p + "k"][8, 0] = 30.0     # one channel per key head
        sd[p + "q"][:, 1] = 0.0
        sd[p + "q"][::8, 1] = 30.0
        sd[p + "k.norm"].fill_(1.0)
        sd[p + "q.norm"].fill_(1.0)
        h = rnd(T, W, seed=11)
        h[:, 0], h[:, 1] = 0.0, 2.0
        h[needle, 0] = 3.0
        m = layer["mixer"]["left"]
        Wn = {k: np64(v) for k, v in sd.items()}
        want = O.talking(np64(h), Wn, p, m, 1e-5)
        h2 = np64(h).copy()
        h2[needle, 0] = 0.0
        diff = np.abs(want - O.talking(h2, Wn, p, m, 1e-5)).max(axis=1)
        last = needle + window - 1
        assert diff[needle:last + 1].min() > 0.05 * np.abs(want).max()
        assert diff[last + 1 :].max() == 0.0
        mod = TalkingHeadsAttention(W, TalkingMixerSpec.from_dict(m), 1e-5, torch.float32)
        mod.load(lambda n: sd[n], p)
        mod.to(dev)
        for sched in ([[(0, last - 5)]] + [[(0, 1)]] * 12 + [[(0, T - last - 7)]],
                      [[(0, 200)], [(0, last - 201)], [(0, 2)], [(0, 2)], [(0, T - last - 3)]]):
            (o,) = run_mixer(mod, [h], 16, torch.float32, dev, sched)
            assert maxdiff(o, want) < 2e-4 * np.abs(want).max()

    def test_bias_needs_its_place(self):
        """The mixed bias per distance, and the constant tail past the last
        distance (a window wider than ``bias_max``)."""
        from kserve_amd.engine.config import TalkingMixerSpec
        from kserve_amd.models.mixers import TalkingHeadsAttention

        layer = O.parallel_layer(heads=3, kv_heads=3, window=500, bias_max=40, buckets=10)
        sd = O.random_weights(O.make_config([layer]), seed=12)
        mod = TalkingHeadsAttention(32, TalkingMixerSpec.from_dict(layer["mixer"]["left"]),
                                    1e-5, torch.float32)
        mod.load(lambda n: sd[n], "l0.mix.left.")
        assert mod.bias.shape == (3, 41)
        rel, talk = np64(sd["l0.mix.left.rel"]), np64(sd["l0.mix.left.talk"])
        for n in (0, 1, 4, 5, 20, 39, 40, 499):
            want = talk @ rel[O.bucket(n, 10, 40)]
            assert maxdiff(mod.bias[:, min(n, 40)], want) < 1e-5

    def test_sink_and_gate(self, dev):
        """With every score far below zero the 1 in the denominator takes
        the weight; the gate scales single elements."""
        H, D, bs = 2, 4, 16
        kc = torch.ones(2, 1, bs, D).to(dev)
        ks = torch.ones(2, bs).to(dev)
        i32 = dict(dtype=torch.int32, device=dev)
        for n in (1, 3):
            q = torch.full((n, H * D), -1.0).to(dev)
            gate = torch.zeros(n, H * D)
            gate[:, 0] = 30.0
            out = ops.talk_attention(
                q, kc, ks, torch.ones(1, 1, **i32), torch.tensor([0, n], **i32),
                torch.tensor([n], **i32), 0.5, n, H, torch.eye(H).to(dev),
                torch.zeros(H, 1).to(dev), 0, gate=gate.to(dev))
            for i in range(n):
                k = i + 1
                w = k * math.exp(-2.0) / (1 + k * math.exp(-2.0))
                assert abs(float(out[i, 0]) - w) < 1e-6
                assert abs(float(out[i, 5]) - w / 2) < 1e-6


class TestGreedyFp32:
    @pytest.mark.parametrize("V", [1, 61, 256, 4097, 40000])
    def test_every_bit_and_ties(self, dev, V):
        """fp32 logits that differ below the bf16 step; ties go to the lower
        index; masked (-inf) entries."""
        x = 1.0 + 1e-4 * rnd(9, V, seed=20).to(dev)
        assert (ops.greedy_sample(x).cpu() == x.cpu().argmax(-1)).all()
        x = torch.full((3, V), -math.inf)
        x[:, V // 2 :] = 2.5
        assert (ops.greedy_sample(x.to(dev)).cpu() == V // 2).all()
