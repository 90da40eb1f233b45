"""The Kebesun decoder (gated linear attention, latent attention and windowed
attention with kept first positions beside dense or routed feed-forwards; a
looped span of layers) through the engine, against the float64 oracle in
kebesun_oracle.py.

Every test builds its own small config and random checkpoint. The same tests
run on the CPU (plain torch forms of the ops, the engine's scheduling, page and
slot logic) and — marked gpu — on the HIP kernels in both activation dtypes.
"""

import json
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import kebesun_oracle as O  # noqa: E402

from kserve_amd.engine.config import (  # noqa: E402
    CacheConfig,
    EngineConfig,
    HybridModelConfig,
    SchedulerConfig,
)
from kserve_amd.engine.engine import LLMEngine  # noqa: E402
from kserve_amd.engine.replay import TraceReplayer  # noqa: E402
from kserve_amd.engine.sampling_params import SamplingParams  # noqa: E402
from kserve_amd.models.registry import build_model  # noqa: E402

BACKENDS = [
    pytest.param(("cpu", "float32"), id="cpu-f32"),
    pytest.param(("cuda", "float32"), id="gpu-f32", marks=pytest.mark.gpu),
    pytest.param(("cuda", "bfloat16"), id="gpu-bf16", marks=pytest.mark.gpu),
]


def all_kinds_config(backend=None, **kw):
    """Every mixer twice with different sizes, both feed-forwards and none, a
    loop over layers of all three kinds. In bf16 every expert is chosen: a
    near-tie in a discrete choice changes every later position of a recurrent
    model; the choice itself is tested in fp32 and, per block, in both."""
    all_chosen = backend is not None and backend[1] == "bfloat16"

    def moe(n, top, ff):
        return O.moe(n, n if all_chosen else top, ff)

    kw.setdefault("loop", (1, 4, 2))
    return O.make_config(
        layers=[
            O.attention_layer(heads=4, kv_heads=2, dim=12, vdim=20, window=9, keep=3,
                              mlp=O.dense(24)),
            O.gla_layer(heads=2, dim=12, vdim=20, tau=8.0, rank=5, mlp=moe(5, 2, 16)),
            O.latent_layer(heads=3, dim=12, rot_dim=8, vdim=20, kv_rank=28, mlp=O.dense(40)),
            O.attention_layer(heads=3, kv_heads=1, dim=16, vdim=8, window=26, keep=18,
                              scale=0.2, rot=O.linear_rot(10, 50.0, 3.0), mlp=moe(3, 1, 24)),
            O.latent_layer(heads=5, dim=8, rot_dim=4, vdim=12, kv_rank=20, scale=0.4,
                           rot=O.yarn_rot(4, 200.0, 2.0, 30, 8.0, 1.0)),
            O.gla_layer(heads=3, dim=20, vdim=8, tau=2.0, rank=2, mlp=moe(4, 3, 8)),
        ],
        **kw,
    )


def checkpoint(cfg, backend, seed=0):
    dt = torch.bfloat16 if backend[1] == "bfloat16" else torch.float32
    return O.random_weights(cfg, seed=seed, dtype=dt)


def make_engine(cfg, sd, backend, num_blocks=64, block_size=16, max_seqs=4,
                eager=False, multi_step=1, max_len=1024, batched_tokens=None,
                mixed=False):
    device, dtype = backend
    mc = HybridModelConfig.from_dict(cfg)
    mc.dtype = dtype
    model = build_model(mc, device=device)
    model.load_hf_state_dict(sd)
    ec = EngineConfig(
        model=mc,
        cache=CacheConfig(block_size=block_size, num_gpu_blocks=num_blocks),
        scheduler=SchedulerConfig(
            max_num_seqs=max_seqs,
            max_num_batched_tokens=batched_tokens or max_len,
            max_model_len=max_len, enable_chunked_prefill=True,
            multi_step=multi_step, mixed_batches=mixed,
        ),
        device=device, eos_token_id=-1, enforce_eager=eager,
    )
    return LLMEngine(ec, model=model)


def row_err(got, want):
    """Per position: centered RMS difference over the vocabulary, relative to
    the RMS of the expected logits."""
    got, want = got.double().cpu(), want.double()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    scale = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    return d.pow(2).mean(-1).sqrt() / scale


def close(got, want, backend, factor=1.0):
    """fp32: every position inside the tolerance. bf16: the median well
    inside, nine positions in ten inside, none far outside (head outputs of
    the recurrent layers are divided by their own RMS, so rounding is amplified
    where they happen to be small)."""
    e = row_err(got, want)
    if backend[1] == "bfloat16":
        ok = bool(
            e.median() < 4e-2 * factor
            and (e < 8e-2 * factor).float().mean() >= 0.9
            and e.max() < 0.4 * factor
        )
    else:
        ok = bool(e.max() < 2e-4 * factor)
    if not ok:
        print("row errors: median %.3g, 90%% %.3g, max %.3g at %d of %d" % (
            e.median(), e.quantile(0.9), e.max(), e.argmax(), e.numel()))
    return ok


def run_schedule(engine, prompts, schedule):
    """schedule: list of steps, each a list of (request index, count); every
    token's logits are collected. Returns {index: [T, vocab]}."""
    rp = TraceReplayer(engine)
    at = {i: 0 for i in range(len(prompts))}
    got = {i: [] for i in range(len(prompts))}
    for step in schedule:
        entries, end, order = [], [], []
        for i, n in step:
            lo = at[i]
            entries.append(
                {"id": f"r{i}", "tokens": prompts[i][lo : lo + n], "want": list(range(n))}
            )
            order.append((i, n))
            at[i] = lo + n
            if at[i] == len(prompts[i]):
                end.append(f"r{i}")
        logits = rp.step(entries, end)
        off = 0
        for i, n in order:
            got[i].append(logits[off : off + n].float().cpu())
            off += n
    return {i: torch.cat(v) for i, v in got.items() if v}


def random_prompt(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


@pytest.fixture(scope="module", params=BACKENDS)
def backend(request):
    if request.param[0] == "cuda":
        from kserve_amd import ops

        assert ops.has_native_seq(), "kserve_amd_seq_C must be built on a GPU box"
    return request.param


class TestWholePrompts:
    def test_logits_and_residual_stream(self, backend):
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(60, cfg["vocab"], 1)
        res = []
        want = O.forward(cfg, sd, toks, res)
        eng.model.debug_residuals = []
        got = run_schedule(eng, [toks], [[(0, len(toks))]])[0]
        streams = eng.model.debug_residuals
        eng.model.debug_residuals = None
        assert close(got, want, backend)
        assert len(streams) == len(res) == 9
        if backend[1] == "float32":
            for mine, ref in zip(streams, res):
                scale = ref.abs().max().item()
                assert (mine.double().cpu() - ref).abs().max().item() < 1e-3 * scale

    def test_first_tokens(self, backend):
        """Prompts of 1, 2 and 3 tokens: no more than the kept positions."""
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=3)
        eng = make_engine(cfg, sd, backend)
        for n in (1, 2, 3):
            toks = random_prompt(n, cfg["vocab"], 10 + n)
            got = run_schedule(eng, [toks], [[(0, n)]])[0]
            assert close(got, O.forward(cfg, sd, toks), backend)

    @pytest.mark.parametrize("loop", [(0, 4, 1), (0, 4, 3), (3, 4, 4), (0, 1, 2), None])
    def test_loops(self, backend, loop):
        """A span that is the whole model, its end, its start, run once or
        several times, and no loop at all; sizes of one and absent parts: single
        heads, a window of one with and without kept positions, one expert, one
        latent coordinate pair, a low rank of one, no rotation, no mask."""
        cfg = O.make_config(
            vocab=31, width=24, loop=loop,
            layers=[
                O.attention_layer(heads=1, kv_heads=1, dim=8, vdim=8, scale=1.0, window=1,
                                  keep=0, rot=None, mlp=O.moe(1, 1, 8)),
                O.gla_layer(heads=1, dim=8, vdim=8, tau=1.0, rank=1),
                O.latent_layer(heads=1, dim=5, rot_dim=2, vdim=3, kv_rank=7, scale=1.0,
                               rot=O.yarn_rot(2, 10.0, 1.0, 12, 2.0, 0.1), mlp=O.dense(8)),
                O.attention_layer(heads=2, kv_heads=2, dim=6, vdim=5, window=loop and 1, keep=1,
                                  rot=O.linear_rot(2, 10.0, 1.0), mlp=O.moe(3, 3, 5)),
            ],
        )
        sd = checkpoint(cfg, backend, seed=4)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(23, cfg["vocab"], 5)
        got = run_schedule(eng, [toks], [[(0, 12)]] + [[(0, 1)]] * 11)[0]
        if backend[1] == "float32":
            assert close(got, O.forward(cfg, sd, toks), backend)
        else:
            # heads of a few columns are divided by their own RMS: rounding is
            # amplified more often than in heads of a usual size
            e = row_err(got, O.forward(cfg, sd, toks))
            assert e.median() < 0.1 and e.max() < 1.0

    def test_more_heads_and_wider(self, backend):
        """Latent rows of 272 columns (the expanded form), 70 experts (64 when all
        are chosen), heads of 72 and 130 columns, kept positions that outnumber
        the window."""
        n, top = (64, 64) if backend[1] == "bfloat16" else (70, 4)
        cfg = O.make_config(
            vocab=40, width=48, loop=(0, 2, 2),
            layers=[
                O.latent_layer(heads=12, dim=24, rot_dim=16, vdim=40, kv_rank=256, scale=0.15),
                O.attention_layer(heads=12, kv_heads=3, dim=72, vdim=40, window=10, keep=24,
                                  scale=0.1, rot=O.linear_rot(30, 100.0, 2.0)),
                O.gla_layer(heads=2, dim=130, vdim=72, tau=16.0, rank=16, mlp=O.moe(n, top, 8)),
            ],
        )
        sd = checkpoint(cfg, backend, seed=21)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(60, cfg["vocab"], 22)
        got = run_schedule(eng, [toks], [[(0, 40)], [(0, 9)]] + [[(0, 1)]] * 11)[0]
        assert close(got, O.forward(cfg, sd, toks), backend)


class TestSchedules:
    def test_prefill_then_decode(self, backend):
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=5)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(75, cfg["vocab"], 6)
        sched = [[(0, 30)]] + [[(0, 1)] for _ in range(45)]
        got = run_schedule(eng, [toks], sched)[0]
        assert close(got, O.forward(cfg, sd, toks), backend)

    def test_graphs_equal_eager(self, backend):
        if backend[0] != "cuda":
            pytest.skip("captured graphs are a GPU path")
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=15)
        toks = random_prompt(50, cfg["vocab"], 16)
        sched = [[(0, 20)]] + [[(0, 1)] for _ in range(30)]
        outs = []
        for eager in (False, True):
            eng = make_engine(cfg, sd, backend, eager=eager)
            outs.append(run_schedule(eng, [toks], sched)[0])
        assert row_err(outs[0], outs[1].double()).max() < 1e-5

    def test_token_by_token_from_the_start(self, backend):
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=6)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(40, cfg["vocab"], 7)
        got = run_schedule(eng, [toks], [[(0, 1)] for _ in toks])[0]
        assert close(got, O.forward(cfg, sd, toks), backend)

    @pytest.mark.parametrize("sizes", [[2] * 20, [3, 17, 2, 16, 1, 5, 2, 2, 31],
                                       [16, 16, 16, 1, 15, 2, 14], [9, 9, 21, 21, 1, 8]])
    def test_portions(self, backend, sizes):
        """Portions down to two tokens, cut inside pages, windows, the kept
        positions and scan chunks."""
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=7)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(sum(sizes), cfg["vocab"], 8)
        got = run_schedule(eng, [toks], [[(0, n)] for n in sizes])[0]
        assert close(got, O.forward(cfg, sd, toks), backend)

    def test_mixed_batches_and_reuse(self, backend):
        """Unequal requests side by side — portions next to decode tokens,
        requests skipped for a step — in a pool too small for all of them at
        once, so pages and state slots are handed out again."""
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=8)
        # 9 usable pages of 16 and 3 slots; six requests
        eng = make_engine(cfg, sd, backend, num_blocks=10, max_seqs=3)
        lens = [40, 23, 9, 33, 17, 48]
        prompts = [random_prompt(n, cfg["vocab"], 20 + i) for i, n in enumerate(lens)]
        sched = [
            [(0, 19), (1, 5)],
            [(0, 1), (1, 16), (2, 2)],
            [(0, 1), (2, 1)],
            [(1, 1), (2, 1), (0, 19)],      # request 0 done
            [(1, 1), (2, 5)],               # requests 1, 2 done
            [(3, 33), (4, 3)],              # request 3 done
            [(4, 1), (5, 20)],
            [(4, 1)],
            [(5, 1), (4, 12)],              # request 4 done
        ] + [[(5, 1)] for _ in range(27)]
        got = run_schedule(eng, prompts, sched)
        for i, toks in enumerate(prompts):
            assert got[i].shape[0] == len(toks)
            assert close(got[i], O.forward(cfg, sd, toks), backend), i
        bm = eng.scheduler.block_manager
        assert bm.num_free_blocks == 9
        assert eng.scheduler.state_slots.num_free == 3

    def test_alone_equals_batched(self, backend):
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=9)
        prompts = [random_prompt(n, cfg["vocab"], 40 + n) for n in (26, 7, 18)]
        eng = make_engine(cfg, sd, backend)
        together = run_schedule(
            eng, prompts,
            [[(0, 20), (1, 7), (2, 3)], [(0, 1), (2, 15)]] + [[(0, 1)]] * 5,
        )
        for i, toks in enumerate(prompts):
            alone = run_schedule(eng, [toks], [[(0, len(toks))]])[0]
            # same kernels, other batch composition: rounding only
            assert close(together[i], alone.double(), backend, factor=0.5)

    def test_long_decode(self, backend):
        cfg = O.make_config(
            vocab=50, width=32, loop=(1, 3, 2),
            layers=[
                O.latent_layer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=24),
                O.gla_layer(heads=2, dim=8, vdim=16, tau=16.0),
                O.attention_layer(heads=2, kv_heads=1, dim=8, vdim=16, window=70, keep=20),
            ],
        )
        sd = checkpoint(cfg, backend, seed=10)
        eng = make_engine(cfg, sd, backend, num_blocks=32)
        toks = random_prompt(300, cfg["vocab"], 11)
        got = run_schedule(eng, [toks], [[(0, 4)]] + [[(0, 1)]] * 296)[0]
        assert close(got, O.forward(cfg, sd, toks), backend)


class TestNeedles:
    """One layer whose weights make a single early token decide the output,
    so that a key lost at a page border, one position off a window's or the
    kept range's edge, or dropped from a carried state shows at once.

    Token 1 is the needle. Every other embedding has no component along
    coordinate 0, and all embeddings share a large coordinate 1. One key
    channel reads coordinate 0 (non-zero for the needle only), the query
    channel beside it reads coordinate 1 (the same for every token); the
    needle's value is far from the others'. Rotation is kept off that
    channel."""

    def _setup(self, kind, backend, window=40, keep=0):
        if kind == "attention":
            layer = O.attention_layer(heads=2, kv_heads=1, dim=8, vdim=8, scale=1.5,
                                      window=window, keep=keep, rot=O.linear_rot(4, 50.0))
        elif kind == "latent_attention":
            layer = O.latent_layer(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=12, scale=1.0)
        else:
            layer = O.gla_layer(heads=2, dim=8, vdim=8, tau=16.0)
        cfg = O.make_config(vocab=40, width=16, layers=[layer])
        sd = checkpoint(cfg, backend, seed=12)

        def edit(name, fn):
            w = sd[name].float()
            fn(w)
            sd[name] = w.to(sd[name].dtype)

        def embed(w):
            w[:, 0] = 0.0
            w[1, 0] = 8.0
            w[:, 1] = 4.0

        edit("embed", embed)
        # small additions would drown in the stream: make the mixer's large
        edit("l0.ls1", lambda w: w.fill_(4.0))
        edit("l0.norm1", lambda w: w.zero_())
        p = "l0.mix."

        def channel(per_head, at, col, gain):
            """Channel ``at`` of every head reads one coordinate; no other
            channel reads coordinates 0 and 1."""
            def fn(w):
                w[:, :2] = 0.0
                for r in range(at, w.shape[0], per_head):
                    w[r] = 0.0
                    w[r, col] = gain
            return fn

        if kind == "attention":
            edit(p + "q", channel(8, 7, 1, 3.0))
            edit(p + "k", channel(8, 7, 0, 3.0))
            edit(p + "v", lambda w: w[:, 0].fill_(2.0))
        elif kind == "latent_attention":
            edit(p + "q", channel(12, 7, 1, 3.0))
            # latent coordinate 0 belongs to the needle; it decides the key
            # channel that the queries look at, and the value
            edit(p + "dkv", channel(99, 0, 0, 6.0))
            edit(p + "dkv.norm", lambda w: w.fill_(1.0))
            edit(p + "uk", channel(8, 7, 0, 3.0))
            edit(p + "uv", lambda w: w[:, 0].fill_(2.0))
        else:
            # queries read the needle's channel only: the read-out is the
            # needle's row of the state
            def only_needle(w):
                w.zero_()
                w[7::8, 1] = 3.0
            edit(p + "q", only_needle)
            edit(p + "k", channel(8, 7, 0, 3.0))
            edit(p + "v", lambda w: w[:, 0].fill_(2.0))
            edit(p + "a2.b", lambda w: w.fill_(6.0))
        return cfg, sd

    def _prompt(self, total, needle_at, vocab, seed):
        toks = [2 + t for t in random_prompt(total, vocab - 2, seed)]
        toks[needle_at] = 1
        return toks

    def _without(self, cfg, sd, toks):
        other = list(toks)
        other[toks.index(1)] = 2
        return O.forward(cfg, sd, other)

    def _tol(self, backend):
        return 8e-2 if backend[1] == "bfloat16" else 2e-4

    @pytest.mark.parametrize("keep", [0, 3, 5])
    @pytest.mark.parametrize("window", [33, 48, 64])
    @pytest.mark.parametrize("cut", ["whole", "decode", "portions"])
    def test_window_edges(self, backend, keep, window, cut):
        """The needle just inside and just outside the window and never among
        the kept positions, for queries in a prompt portion and decoded alone;
        windows smaller than, equal to and no multiple of the 16-token page."""
        cfg, sd = self._setup("attention", backend, window, keep)
        needle, total = 5, 5 + window + 6
        toks = self._prompt(total, needle, cfg["vocab"], 13)
        want = O.forward(cfg, sd, toks)
        gone = self._without(cfg, sd, toks)
        last_in = needle + window - 1
        # the test would see the needle missing, or staying too long
        assert row_err(want, gone)[[last_in - 1, last_in]].min() > 0.1
        assert row_err(want[last_in + 1 :], gone[last_in + 1 :]).max() < 1e-9
        eng = make_engine(cfg, sd, backend)
        if cut == "whole":
            sched = [[(0, total)]]
        elif cut == "decode":
            sched = [[(0, last_in - 2)]] + [[(0, 1)]] * (total - last_in + 2)
        else:
            sched = [[(0, last_in)], [(0, 2)], [(0, total - last_in - 2)]]
        got = run_schedule(eng, [toks], sched)[0]
        e = row_err(got, want)
        assert e.max() < self._tol(backend), e.argmax()

    @pytest.mark.parametrize("window,keep", [(20, 17), (33, 16), (7, 40), (64, 1)])
    @pytest.mark.parametrize("cut", ["whole", "decode", "portions"])
    def test_kept_positions(self, backend, window, keep, cut):
        """The needle as the last kept position, seen from everywhere after
        it, and as the first one that is not kept."""
        for needle in (keep - 1, keep):
            cfg, sd = self._setup("attention", backend, window, keep)
            total = keep + 2 * window + 70
            toks = self._prompt(total, needle, cfg["vocab"], 17)
            want = O.forward(cfg, sd, toks)
            e = row_err(want, self._without(cfg, sd, toks))
            if needle < keep:
                assert e[needle:].min() > 0.1
            else:
                assert e[needle + window :].max() < 1e-9
            eng = make_engine(cfg, sd, backend)
            if cut == "whole":
                sched = [[(0, total)]]
            elif cut == "decode":
                sched = [[(0, keep + 2)]] + [[(0, 1)]] * (total - keep - 2)
            else:
                sched = [[(0, keep)], [(0, 2)], [(0, window)], [(0, 3)],
                         [(0, total - keep - window - 5)]]
                sched = [p for p in sched if p[0][1] > 0]
            got = run_schedule(eng, [toks], sched)[0]
            e = row_err(got, want)
            assert e.max() < self._tol(backend), (needle, e.argmax())

    @pytest.mark.parametrize("kind", ["attention", "latent_attention", "gla"])
    @pytest.mark.parametrize("needle_at", [0, 15, 16, 31])
    def test_far_token_at_page_borders(self, backend, kind, needle_at):
        """The needle 300+ positions back, first and last in a page, read by
        prompt portions and by tokens decoded alone."""
        cfg, sd = self._setup(kind, backend, window=400)
        total = 350
        toks = self._prompt(total, needle_at, cfg["vocab"], 14)
        want = O.forward(cfg, sd, toks)
        assert row_err(want, self._without(cfg, sd, toks))[[total - 20, total - 1]].min() > 0.1
        eng = make_engine(cfg, sd, backend)
        sched = [[(0, 100)], [(0, 37)], [(0, 163)], [(0, 2)], [(0, 16)]] + [[(0, 1)]] * 32
        got = run_schedule(eng, [toks], sched)[0]
        e = row_err(got, want)
        assert e.max() < self._tol(backend), e.argmax()


class TestGeneration:
    def test_greedy_through_the_engine(self, backend):
        """LLMEngine.generate with its own scheduler, multi-step decode
        windows, mixed batches and a pool that forces preemption equals
        step-by-step argmax of the oracle for every request."""
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=30)
        sd["head"] = sd["head"] * 4
        prompts = [random_prompt(n, cfg["vocab"], 60 + n) for n in (12, 5, 19, 8)]
        new = 12

        def follows_oracle(prompt, out):
            """Every generated token is the oracle's argmax given what was
            generated before it (or within a hair of it: near-ties)."""
            logits = O.forward(cfg, sd, list(prompt) + [int(t) for t in out])
            for i, t in enumerate(out):
                row = logits[len(prompt) + i - 1]
                if (row.max() - row[int(t)]).item() > 1e-3:
                    return False
            return True

        for kw in (
            dict(multi_step=4),
            dict(multi_step=1, mixed=True, batched_tokens=16),
            dict(multi_step=4, num_blocks=6, max_seqs=2),
        ):
            eng = make_engine(cfg, sd, backend, **kw)
            outs = eng.generate(
                prompts,
                SamplingParams(max_tokens=new, temperature=0.0, ignore_eos=True),
            )
            assert len(outs) == len(prompts)
            got = [list(o.output_token_ids) for o in outs.values()]
            assert all(len(g) == new for g in got)
            if backend[1] == "float32":
                assert all(follows_oracle(p, g) for p, g in zip(prompts, got)), kw
            bm = eng.scheduler.block_manager
            assert bm.num_free_blocks == kw.get("num_blocks", 64) - 1
            assert eng.scheduler.state_slots.num_free == kw.get("max_seqs", 4)

    def test_sampled_generation(self, backend):
        """Temperature sampling through the engine's samplers (on the GPU the
        fused sampler inside captured multi-step windows)."""
        cfg = all_kinds_config(backend)
        sd = checkpoint(cfg, backend, seed=31)
        prompts = [random_prompt(n, cfg["vocab"], 80 + n) for n in (9, 4, 15)]
        eng = make_engine(cfg, sd, backend, multi_step=4)
        outs = eng.generate(
            prompts,
            SamplingParams(max_tokens=10, temperature=0.8, top_k=20, top_p=0.9,
                           ignore_eos=True, seed=5),
        )
        assert len(outs) == 3
        for o in outs.values():
            assert len(o.output_token_ids) == 10
            assert all(0 <= t < cfg["vocab"] for t in o.output_token_ids)


def write_model(d, cfg, sd):
    from safetensors.torch import save_file

    d.mkdir()
    (d / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(d / "model.safetensors"))


class TestPlumbing:
    def test_registry_config_layout_and_loading(self, tmp_path):
        from kserve_amd.models.registry import load_model_config, native_modules_for

        cfg = all_kinds_config()
        sd = O.random_weights(cfg, seed=2, dtype=torch.bfloat16)
        d = tmp_path / "model"
        write_model(d, cfg, sd)
        mc = load_model_config(str(d))
        assert mc.architecture == "Kebesun"
        assert native_modules_for(str(d)) == ("kserve_amd_seq_C",)
        assert mc.has_recurrent_state
        a = mc.layers[3].attention
        assert (a.window, a.keep_first, a.chunk, a.rot_dims) == (26, 18, 0, 10)
        assert a.rot_scaling == {"factor": 3.0}
        lt = mc.layers[4].latent
        assert (lt.q_rank, lt.rot_pairs, lt.cache_dim, lt.rot_dims) == (0, False, 24, 4)
        assert lt.rot_scaling["original"] == 30.0 and not lt.sink and not lt.gate
        assert mc.layers[5].gated_linear.tau == 2.0
        assert mc.layers[4].mlp is None and mc.layers[0].mlp.ff == 24
        m = mc.layers[1].mlp
        assert (m.experts, m.top, m.ff) == (5, 2, 16) and m.over_chosen and m.router_bias
        assert mc.layer_runs() == [(0, None), (1, 0), (2, 0), (3, 0), (1, 1), (2, 1), (3, 1),
                                   (4, None), (5, None)]
        mc.dtype = "bfloat16"
        model = build_model(mc, device="cpu")
        layout = model.cache_layout()
        # every pass of the looped span has pages and state of its own
        assert len(layout) == 9 and layout[1:4] == layout[4:7]
        assert layout[0] == ((2, 12, 20), {})
        assert layout[1] == (None, {"ssm": ((2, 20, 12), torch.float32)})
        assert layout[2] == ((1, 36, 0), {})
        per_token = 2 * (2 * (12 + 20) + 2 * 36 + 2 * (16 + 8) + 24)
        assert mc.kv_bytes_per_block(16, 2) == 16 * per_token
        # a size that only tensors carry
        model.load_hf_state_dict(sd)
        assert (model.layers[1].mix.a_rank, model.layers[5].mix.a_rank) == (5, 2)

    def test_no_state_slots_without_recurrent_layers(self):
        cfg = O.make_config([O.attention_layer(), O.latent_layer()], loop=(0, 1, 2))
        mc = HybridModelConfig.from_dict(cfg)
        assert not mc.has_recurrent_state
        backend = ("cpu", "float32")
        sd = checkpoint(cfg, backend)
        eng = make_engine(cfg, sd, backend)
        assert eng.runner.num_state_slots == 0
        toks = random_prompt(20, cfg["vocab"], 3)
        got = run_schedule(eng, [toks], [[(0, 11)], [(0, 9)]])[0]
        assert close(got, O.forward(cfg, sd, toks), backend)

    def test_server_cli_picks_the_engine(self, tmp_path):
        from kserve_amd.runtimes.huggingfaceserver import detect_backend

        (tmp_path / "config.json").write_text(json.dumps(all_kinds_config()))
        assert detect_backend(str(tmp_path)) == "engine"

    def test_unknown_parts_are_refused(self):
        for change in (
            lambda c: c["layers"][0].update(type="something-else"),
            lambda c: c["layers"][0]["mlp"].update(kind="another"),
        ):
            cfg = all_kinds_config()
            change(cfg)
            with pytest.raises(ValueError):
                HybridModelConfig.from_dict(cfg)

    def test_weights_can_be_loaded_again(self):
        cfg = all_kinds_config()
        mc = HybridModelConfig.from_dict(cfg)
        mc.dtype = "float32"
        model = build_model(mc)
        a, b = (O.random_weights(cfg, seed=s) for s in (1, 2))
        toks = random_prompt(20, cfg["vocab"], 3)
        model.load_hf_state_dict(a)
        model.load_hf_state_dict(b)
        eng = LLMEngine(EngineConfig(
            model=mc, cache=CacheConfig(num_gpu_blocks=8),
            scheduler=SchedulerConfig(max_num_seqs=2, max_model_len=64),
            device="cpu", eos_token_id=-1), model=model)
        got = run_schedule(eng, [toks], [[(0, 20)]])[0]
        assert close(got, O.forward(cfg, b, toks), ("cpu", "float32"))

    def test_engine_from_a_model_directory(self, tmp_path):
        from kserve_amd.engine.replay import engine_config_for_trace

        cfg = all_kinds_config()
        sd = O.random_weights(cfg, seed=2)
        d = tmp_path / "model"
        write_model(d, cfg, sd)
        ec = engine_config_for_trace(str(d), "float32", 128, "cpu", block_size=16)
        eng = LLMEngine(ec)
        toks = random_prompt(30, cfg["vocab"], 3)
        got = run_schedule(eng, [toks], [[(0, 17)], [(0, 13)]])[0]
        assert close(got, O.forward(cfg, sd, toks), ("cpu", "float32"))

    def test_random_init_runs(self):
        mc = HybridModelConfig.from_dict(all_kinds_config())
        mc.dtype = "float32"
        model = build_model(mc).random_init()
        assert all(torch.isfinite(p).all() for p in model.parameters())
