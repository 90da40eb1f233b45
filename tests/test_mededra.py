"""The Mededra decoder (differential attention; talking-heads attention beside
a channel-decay delta rule; grouped output norms) through the engine, against
the float64 oracle in mededra_oracle.py.

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
import mededra_oracle as O  # noqa: E402

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


def both_kinds_config(**kw):
    """Both layer types twice with different sizes; one layer has no
    feed-forward."""
    return O.make_config(
        layers=[
            O.attention_layer(heads=4, kv_heads=2, dim=12, vdim=20, conv=3, window=9,
                              mlp=O.mlp(24)),
            O.parallel_layer(heads=4, kv_heads=2, dim=8, window=21, bias_max=30,
                             d_heads=4, d_kv_heads=2, d_dim=12, d_vdim=8, mlp=O.mlp(40)),
            O.attention_layer(heads=3, kv_heads=1, dim=8, vdim=12, conv=4, window=26,
                              diff=0.6, scale=0.3, cap=2.0,
                              rotation=O.rot(4, 20.0, None)),
            O.parallel_layer(heads=6, kv_heads=1, dim=20, window=34, bias_max=20,
                             buckets=6, d_heads=3, d_kv_heads=3, d_dim=8, d_vdim=24,
                             conv=2, a_rank=2, g_rank=11, mlp=O.mlp(16)),
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
    inside, nine positions in ten inside, none far outside (the outputs of
    differential heads and of the delta rule are divided by their own RMS, so
    rounding is amplified where they happen to be small)."""
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
        cfg = both_kinds_config()
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
        assert len(streams) == len(cfg["layers"])
        if backend[1] == "float32":
            for mine, ref in zip(streams, res):
                scale = ref.abs().max().item()
                assert (mine.double().cpu() - ref).abs().max().item() < 1e-3 * scale

    def test_first_tokens(self, backend):
        """Prompts of 1, 2 and 3 tokens: shorter than every convolution and
        window; all history before position 0 is zero."""
        cfg = both_kinds_config()
        sd = checkpoint(cfg, backend, seed=3)
        eng = make_engine(cfg, sd, backend)
        for n in (1, 2, 3):
            toks = random_prompt(n, cfg["vocab"], 10 + n)
            got = run_schedule(eng, [toks], [[(0, n)]])[0]
            assert close(got, O.forward(cfg, sd, toks), backend)

    def test_sizes_equal_to_one_and_missing_parts(self, backend):
        """Single heads, one tap, a window of one, no rotation, one norm
        group, ranks of one, no caps, unit scales."""
        cfg = O.make_config(
            vocab=31, width=24, groups=1, emb_scale=1.0, cap=0.0,
            layers=[
                O.attention_layer(heads=1, kv_heads=1, dim=8, vdim=8, conv=1, window=1,
                                  diff=0.0, scale=1.0, cap=0.0, rotation=None,
                                  mlp=O.mlp(8)),
                O.parallel_layer(heads=1, kv_heads=1, dim=24, scale=1.0, window=1,
                                 bias_max=2, buckets=2, d_heads=1, d_kv_heads=1,
                                 d_dim=8, d_vdim=8, conv=1, a_rank=1, g_rank=1),
                O.parallel_layer(heads=2, kv_heads=2, dim=7, window=300, bias_max=9,
                                 buckets=4, d_heads=2, d_kv_heads=1, d_dim=17, d_vdim=5,
                                 conv=5, mlp=O.mlp(12)),
                O.attention_layer(heads=2, kv_heads=2, dim=5, vdim=3, conv=6, window=300,
                                  rotation=O.rot(2, 10.0, O.yarn(1.0, 12, 2.0, 0.1))),
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
        cfg = O.make_config(
            vocab=40, width=48, groups=8,
            layers=[
                O.attention_layer(heads=12, kv_heads=3, dim=72, vdim=40, window=30,
                                  rotation=O.rot(30, 100.0, O.yarn(2.0, 50))),
                O.parallel_layer(heads=20, kv_heads=10, dim=16, window=30, bias_max=50,
                                 buckets=16, d_heads=2, d_kv_heads=1, d_dim=72, d_vdim=40,
                                 conv=3, mlp=O.mlp(64)),
            ],
        )
        sd = checkpoint(cfg, backend, seed=21)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(50, cfg["vocab"], 22)
        got = run_schedule(eng, [toks], [[(0, 40)]] + [[(0, 1)]] * 10)[0]
        assert close(got, O.forward(cfg, sd, toks), backend)


class TestSchedules:
    def test_prefill_then_decode(self, backend):
        cfg = both_kinds_config()
        sd = checkpoint(cfg, backend, seed=5)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(75, cfg["vocab"], 6)
        sched = [[(0, 30)]] + [[(0, 1)] for _ in range(45)]
        got = run_schedule(eng, [toks], sched)[0]
        assert close(got, O.forward(cfg, sd, toks), backend)

    def test_graphs_equal_eager(self, backend):
        if backend[0] != "cuda":
            pytest.skip("captured graphs are a GPU path")
        cfg = both_kinds_config()
        sd = checkpoint(cfg, backend, seed=15)
        toks = random_prompt(50, cfg["vocab"], 16)
        sched = [[(0, 20)]] + [[(0, 1)] for _ in range(30)]
        outs = []
        for eager in (False, True):
            eng = make_engine(cfg, sd, backend, eager=eager)
            outs.append(run_schedule(eng, [toks], sched)[0])
        assert row_err(outs[0], outs[1].double()).max() < 1e-5

    def test_token_by_token_from_the_start(self, backend):
        cfg = both_kinds_config()
        sd = checkpoint(cfg, backend, seed=6)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(40, cfg["vocab"], 7)
        got = run_schedule(eng, [toks], [[(0, 1)] for _ in toks])[0]
        assert close(got, O.forward(cfg, sd, toks), backend)

    @pytest.mark.parametrize("sizes", [[2] * 20, [3, 17, 2, 16, 1, 5, 2, 2, 31],
                                       [16, 16, 16, 1, 15, 2, 14], [9, 9, 21, 21, 1, 8]])
    def test_portions(self, backend, sizes):
        """Portions down to two tokens, cut inside pages, windows and
        scan chunks and shorter than the convolutions' history."""
        cfg = both_kinds_config()
        sd = checkpoint(cfg, backend, seed=7)
        eng = make_engine(cfg, sd, backend)
        toks = random_prompt(sum(sizes), cfg["vocab"], 8)
        got = run_schedule(eng, [toks], [[(0, n)] for n in sizes])[0]
        assert close(got, O.forward(cfg, sd, toks), backend)

    def test_mixed_batches_and_reuse(self, backend):
        """Unequal requests side by side — portions next to decode tokens,
        requests skipped for a step — in a pool too small for all of them at
        once, so pages and state slots are handed out again."""
        cfg = both_kinds_config()
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
        cfg = both_kinds_config()
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
            vocab=50, width=32,
            layers=[
                O.parallel_layer(heads=2, kv_heads=1, dim=16, window=40, bias_max=60,
                                 d_heads=2, d_kv_heads=1, d_dim=8, d_vdim=16, conv=3),
                O.attention_layer(heads=2, kv_heads=1, dim=8, vdim=16, window=70),
            ],
        )
        sd = checkpoint(cfg, backend, seed=10)
        eng = make_engine(cfg, sd, backend, num_blocks=32)
        toks = random_prompt(300, cfg["vocab"], 11)
        got = run_schedule(eng, [toks], [[(0, 4)]] + [[(0, 1)]] * 296)[0]
        assert close(got, O.forward(cfg, sd, toks), backend)


class TestNeedles:
    """One layer whose weights make a single early token decide the output,
    so that a key lost at a page border, one position off a window's edge or
    dropped from a carried state shows at once.

    Token 1 is the needle. Every other embedding has no component along
    coordinate 0, and all embeddings share a large coordinate 1. One key
    channel reads coordinate 0 (non-zero for the needle only), the query
    channel beside it reads coordinate 1 (the same for every token); the
    needle's value is far from the others'. Rotation is kept off that channel.
    In a parallel layer the branch that is not looked at is silenced by its
    output weight."""

    def _setup(self, kind, backend, window=40):
        if kind == "differential":
            layer = O.attention_layer(heads=2, kv_heads=1, dim=8, vdim=8, scale=1.5,
                                      conv=2, cap=20.0, diff=0.1, window=window,
                                      rotation=O.rot(4, 50.0, O.yarn()))
        else:
            layer = O.parallel_layer(heads=2, kv_heads=1, dim=8, scale=1.0, window=window,
                                     bias_max=30, d_heads=2, d_kv_heads=1, d_dim=8,
                                     d_vdim=8, conv=2)
        cfg = O.make_config(vocab=40, width=16, groups=2, layers=[layer], cap=0.0,
                            emb_scale=1.0)
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
        # small additions would drown in the stream: make the norm's output large
        edit("l0.norm1", lambda w: w.fill_(4.0))

        def channel(col, gain):
            """Every head's (and map's) channel 7 reads one coordinate; no
            other channel reads coordinates 0 and 1."""
            def fn(w):
                w[:, :2] = 0.0
                for r in range(7, w.shape[0], 8):
                    w[r] = 0.0
                    w[r, col] = gain
            return fn

        def take_now(w):
            w.zero_()
            w[:, -1] = 1.0

        if kind == "differential":
            p = "l0.mix."
            edit(p + "q", channel(1, 3.0))
            edit(p + "k", channel(0, 3.0))
            edit(p + "v", lambda w: w[:, 0].fill_(2.0))
            for n in ("q", "k", "v"):
                edit(p + n + ".conv", take_now)
            # the second map looks at every key alike: the difference keeps the
            # needle
            edit(p + "q", lambda w: w.view(-1, 2, 8, w.shape[1])[:, 1].zero_())
        elif kind == "talking":
            p = "l0.mix.left."
            edit(p + "q", channel(1, 6.0))
            edit(p + "k", channel(0, 6.0))
            edit(p + "k.norm", lambda w: w.fill_(1.0))
            edit(p + "q.norm", lambda w: w.fill_(1.0))
            edit(p + "talk", lambda w: w.copy_(torch.tensor([[1.0, 0.2], [0.3, 1.0]])))
            edit("l0.mix.right.out", lambda w: w.zero_())
            edit(p + "g", lambda w: w.zero_())
        else:
            p = "l0.mix.right."
            edit(p + "k", channel(0, 3.0))
            edit(p + "v", lambda w: w[:, 0].fill_(2.0))
            for n in ("q", "k", "v"):
                edit(p + n + ".conv", take_now)
            edit(p + "A_log", lambda w: w.fill_(-7.0))

            # unit-norm queries: leave them nothing but the needle's channel,
            # so that the read-out is the needle's row of the state
            def only_needle(w):
                w.zero_()
                w[7, 1] = 3.0
            edit(p + "q", only_needle)
            edit("l0.mix.left.out", lambda w: w.zero_())
        return cfg, sd

    def _prompt(self, total, needle_at, vocab, seed):
        toks = [2 + t for t in random_prompt(total, vocab - 2, seed)]
        toks[needle_at] = 1
        return toks

    def _without(self, cfg, sd, toks):
        other = list(toks)
        other[toks.index(1)] = 2
        return O.forward(cfg, sd, other)

    @pytest.mark.parametrize("kind", ["differential", "talking"])
    @pytest.mark.parametrize("window", [33, 48, 64])
    @pytest.mark.parametrize("cut", ["whole", "decode", "portions"])
    def test_window_edges(self, backend, kind, window, cut):
        """The needle just inside and just outside the window, for queries
        in a prompt portion and decoded alone; windows smaller than, equal to
        and no multiple of the 16-token page."""
        cfg, sd = self._setup(kind, backend, window=window)
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
        assert e.max() < (8e-2 if backend[1] == "bfloat16" else 2e-4), e.argmax()

    @pytest.mark.parametrize("kind", ["differential", "talking", "delta"])
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
        assert e.max() < (8e-2 if backend[1] == "bfloat16" else 2e-4), e.argmax()


class TestGeneration:
    def test_greedy_through_the_engine(self, backend):
        """LLMEngine.generate with its own scheduler, multi-step decode
        windows, mixed batches and a pool that forces preemption equals
        step-by-step argmax of the oracle for every request."""
        cfg = both_kinds_config(cap=30.0)
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
        cfg = both_kinds_config()
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

        cfg = both_kinds_config()
        sd = O.random_weights(cfg, seed=2, dtype=torch.bfloat16)
        d = tmp_path / "model"
        write_model(d, cfg, sd)
        mc = load_model_config(str(d))
        assert mc.architecture == "Mededra"
        assert native_modules_for(str(d)) == ("kserve_amd_seq_C",)
        assert mc.has_recurrent_state
        assert mc.norm_groups == 2 and mc.embedding_scale == 3.0 and mc.logit_softcap == 9.0
        df = mc.layers[2].differential
        assert (df.window, df.conv, df.diff, df.softcap, df.rot_scaling) == (26, 4, 0.6, 2.0, None)
        assert mc.layers[0].differential.rot_scaling["factor"] == 3.0
        assert mc.layers[2].mlp is None and mc.layers[1].mlp.ff == 40
        assert mc.layers[3].talking.bias_max == 20 and mc.layers[3].talking.window == 34
        assert mc.layers[3].delta.channel_decay and mc.layers[3].delta.conv == 2
        mc.dtype = "bfloat16"
        model = build_model(mc, device="cpu")
        layout = model.cache_layout()
        assert layout[0] == ((2, 24, 20), {"conv": ((2, 2 * 6 * 12 + 2 * 20), torch.bfloat16)})
        assert layout[1][0] == (2, 8, 0)
        assert set(layout[1][1]) == {"k_scale", "ssm", "conv"}
        assert layout[1][1]["ssm"][0] == (4, 8, 12)
        # two key maps + values; un-normed keys and an fp32 factor
        per_token = 2 * (2 * (24 + 20) + 2 * 8 + (16 + 12) + 20) + 2 * 4
        assert mc.kv_bytes_per_block(16, 2) == 16 * per_token
        # sizes that only tensors carry
        model.load_hf_state_dict(sd)
        assert model.layers[3].left.rel.shape == (6, 6)
        assert (model.layers[3].right.a_rank, model.layers[3].right.g_rank) == (2, 11)

    def test_only_convolutions_count_as_state(self):
        one = O.make_config([O.attention_layer(conv=1)])
        two = O.make_config([O.attention_layer(conv=2)])
        assert not HybridModelConfig.from_dict(one).has_recurrent_state
        assert HybridModelConfig.from_dict(two).has_recurrent_state

    def test_server_cli_picks_the_engine(self, tmp_path):
        from kserve_amd.runtimes.huggingfaceserver import detect_backend

        (tmp_path / "config.json").write_text(json.dumps(both_kinds_config()))
        assert detect_backend(str(tmp_path)) == "engine"

    def test_unknown_parts_are_refused(self):
        for change in (
            lambda c: c["layers"][0].update(type="something-else"),
            lambda c: c["layers"][0]["mlp"].update(kind="moe"),
            lambda c: c["layers"][1]["mixer"]["left"].update(vdim=9),
            lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
        ):
            cfg = both_kinds_config()
            change(cfg)
            with pytest.raises(ValueError):
                HybridModelConfig.from_dict(cfg)
        cfg = both_kinds_config(groups=3)
        with pytest.raises(ValueError):
            build_model(HybridModelConfig.from_dict(cfg))

    def test_weights_can_be_loaded_again(self):
        cfg = both_kinds_config()
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

        cfg = both_kinds_config()
        sd = O.random_weights(cfg, seed=2)
        d = tmp_path / "model"
        write_model(d, cfg, sd)
        ec = engine_config_for_trace(str(d), "float32", 128, "cpu", block_size=16)
        eng = LLMEngine(ec)
        toks = random_prompt(30, cfg["vocab"], 3)
        got = run_schedule(eng, [toks], [[(0, 17)], [(0, 13)]])[0]
        assert close(got, O.forward(cfg, sd, toks), ("cpu", "float32"))
