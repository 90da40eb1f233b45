"""Kebesun: a decoder whose layers are listed one by one in the config, a span
of which may run several times over.

A layer is parallel: with h = norm1(x),

    x += ls1 * mixer(h) + ls2 * ff(h)

— one RMS norm (gain 1 + w per channel) read by both sublayers, and a factor
per channel on each result. Mixers: ``GatedLinearMixer``
("gla"), ``LatentAttention`` with directly projected queries and a half-split
YaRN rotation ("latent_attention"), and sliding-window softmax attention that
keeps the first positions visible (``RotaryChunkSinkAttention`` without norms
and sink, "attention"). The feed-forward is ``SiluGLU``, a
``SoftmaxRoutedMoE`` whose weights are the softmax over the chosen logits, or
absent.

``loop``: layers start .. stop-1 run ``times`` times with the same weights,
every pass with a cache of its own; each pass starts from L [x; x0], x0 the
embedding output. With L = [A | B] the part B x0 is the same in every pass:
it is computed once, and "add it to A x, norm for the pass's first layer" is
the same kernel as every other addition to the stream.

The residual stream is fp32 whatever the activation dtype. "Multiply the two
sublayer outputs by their channel factors, sum a token's expert rows, add
everything, norm for the next layer" is one kernel.
"""

from __future__ import annotations

from typing import List, Optional

import torch
import torch.nn as nn

from kserve_amd import ops
from kserve_amd.engine.config import (
    HybridLayerSpec,
    HybridModelConfig,
    SiluGLUSpec,
    SoftmaxMoESpec,
)
from kserve_amd.models.mixers import (
    ExpertRows,
    GatedLinearMixer,
    LatentAttention,
    RotaryChunkSinkAttention,
    SiluGLU,
    SoftmaxRoutedMoE,
)
from kserve_amd.parallel import comm


def _vec(n: int):
    return nn.Parameter(torch.empty(n, dtype=torch.float32), requires_grad=False)


class KebesunLayer(nn.Module):
    def __init__(self, width: int, spec: HybridLayerSpec, eps: float, dtype):
        super().__init__()
        self.spec = spec
        if spec.gated_linear is not None:
            self.mix = GatedLinearMixer(width, spec.gated_linear, eps, dtype)
        elif spec.latent is not None:
            self.mix = LatentAttention(width, spec.latent, eps, dtype)
        elif spec.attention is not None:
            self.mix = RotaryChunkSinkAttention(
                width, spec.attention, eps, dtype, sink=False,
                value_unit_norm=False, rotate_values=False, qk_norm=False,
            )
        else:
            raise ValueError("a Kebesun layer needs a mixer")
        if isinstance(spec.mlp, SoftmaxMoESpec):
            self.mlp = SoftmaxRoutedMoE(width, spec.mlp, dtype)
        elif isinstance(spec.mlp, SiluGLUSpec):
            self.mlp = SiluGLU(width, spec.mlp.ff, dtype)
        elif spec.mlp is None:
            self.mlp = None
        else:
            raise ValueError(f"unsupported feed-forward {type(spec.mlp).__name__}")
        self.norm1 = _vec(width)
        self.ls1 = _vec(width)
        self.ls2 = _vec(width) if self.mlp is not None else None

    def cache_entry(self):
        s = self.spec
        if s.gated_linear is not None:
            return None, self.mix.state_shapes()
        if s.latent is not None:
            # one row per token, values are its leading columns
            return (1, s.latent.cache_dim, 0), {}
        a = s.attention
        return (a.kv_heads, a.dim, a.vdim), {}

    def forward(self, h, positions, cache, meta):
        """Both sublayer outputs, as keyword arguments of the kernel that adds
        them to the stream."""
        out = {"d0": self.mix(h, positions, cache, meta), "c0": self.ls1}
        if self.mlp is None:
            return out
        y = (
            self.mlp.rows(h) if isinstance(self.mlp, SoftmaxRoutedMoE)
            else ExpertRows(self.mlp(h))
        )
        out.update(d1=y.y, c1=self.ls2, d1_index=y.index, d1_weights=y.weights,
                   d1_top=y.top)
        return out


class KebesunForCausalLM(nn.Module):
    # every step attends through the paged cache (no separate un-paged
    # prefill kernel)
    paged_prefill_only = True

    def __init__(
        self,
        config: HybridModelConfig,
        dtype: Optional[torch.dtype] = None,
        device: str = "cpu",
    ):
        super().__init__()
        st = comm.get_state()
        if st.tp_size != 1 or st.pp_size != 1:
            raise NotImplementedError(
                "Kebesun runs on one GPU per replica (no tensor/pipeline split)"
            )
        self.config = config
        dtype = dtype or (
            torch.bfloat16 if config.dtype == "bfloat16" else torch.float32
        )
        self.dtype = dtype
        W = config.hidden_size
        self.embed = nn.Parameter(
            torch.empty(config.vocab_size, W, dtype=dtype), requires_grad=False
        )
        self.layers = nn.ModuleList(
            [KebesunLayer(W, spec, config.rms_norm_eps, dtype) for spec in config.layers]
        )
        self.needs_state_slots = config.has_recurrent_state
        self.runs = config.layer_runs()
        looped = any(t is not None for _, t in self.runs)
        self.loop_start = config.loop.start if looped else -1
        # the halves of the pass-opening matrix that meet x and the embedding
        self.loop_x = self.loop_x0 = None
        if looped:
            self.loop_x = nn.Parameter(torch.empty(W, W, dtype=dtype), requires_grad=False)
            self.loop_x0 = nn.Parameter(torch.empty(W, W, dtype=dtype), requires_grad=False)
        self.num_local_layers = len(self.runs)
        self.final_norm = _vec(W)
        self.head = nn.Parameter(
            torch.empty(config.vocab_size, W, dtype=dtype), requires_grad=False
        )
        self.eps = config.rms_norm_eps
        # largest decode batch worth capturing: above it the routed experts
        # switch to their sorted form, which synchronises with the host
        caps = [
            l.mlp.dense_max_tokens for l in self.layers
            if isinstance(l.mlp, SoftmaxRoutedMoE)
        ]
        self.decode_graph_max_tokens = min(caps) if caps else None
        if any(getattr(l.mix, "expanded", False) for l in self.layers):
            # the expanded form of wide rows reads context lengths on the host
            self.decode_graph_max_tokens = 0
        # when a list, forward() appends the residual stream after each layer run
        self.debug_residuals: Optional[List[torch.Tensor]] = None
        self.to(device)

    # -- cache layout (read by the model runner) ------------------------------
    def cache_layout(self):
        """One entry per layer RUN (a looped layer once per pass):
        (kv_heads, key columns, value columns) or None, and
        {name: (shape_per_slot, dtype)} of recurrent state."""
        return [self.layers[i].cache_entry() for i, _ in self.runs]

    # -- init -----------------------------------------------------------------
    @torch.no_grad()
    def random_init(self, std: float = 0.02, seed: int = 0):
        dev = self.embed.device
        gen = torch.Generator(device=dev)
        gen.manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("loop_x", "loop_x0"):
                p.normal_(0.0, (2 * p.shape[-1]) ** -0.5, generator=gen)
            elif p.dim() >= 2:
                # keep activations O(1) through the stack
                fan_in = p.shape[-2] if leaf == "uk_t" else p.shape[-1]
                p.normal_(0.0, fan_in ** -0.5, generator=gen)
            elif leaf in ("ls1", "ls2"):
                p.fill_(0.5)
            elif leaf in ("kv_norm", "norm_w"):
                p.fill_(1.0)
            else:  # norm gains (their distance from one), biases
                p.normal_(0.0, 0.1, generator=gen)
        return self

    # -- forward --------------------------------------------------------------
    def forward(self, input_ids, positions, caches, meta):
        x = ops.embed_scale_sinpos(self.embed, input_ids, positions, None, 1.0)
        from_embedding = None
        if self.loop_x is not None:
            # bf16: embedding rows are exact in the activation dtype
            from_embedding = ops.linear_f32out(self._as_activation(x), self.loop_x0)
        pending = {}
        dbg = self.debug_residuals
        for (i, t), cache in zip(self.runs, caches):
            layer = self.layers[i]
            if t is not None and i == self.loop_start:
                x = ops.linear_f32out(self._as_activation(x, pending), self.loop_x)
                pending = {"d0": from_embedding}
            h = self._add(x, layer.norm1, pending)
            pending = layer(h, positions, cache, meta)
            if dbg is not None:
                r = x.clone()
                self._add(r, None, pending, want_out=False)
                dbg.append(r)
        return self._add(x, self.final_norm, pending)

    def _add(self, x, weight, pending, want_out: bool = True):
        """The stream takes what is pending; returns its norm (gain
        1 + ``weight``), or the stream itself in the activation dtype."""
        return ops.add_rms_norm_f32res(
            x, weight, self.eps, 1.0, self.dtype, want_out=want_out, **pending
        )

    def _as_activation(self, x, pending=None):
        if self.dtype == torch.float32:
            if pending:
                self._add(x, None, pending, want_out=False)
            return x
        return self._add(x, None, pending or {})

    def compute_logits(self, hidden):
        return ops.linear_f32out(hidden, self.head)

    # -- weights ----------------------------------------------------------------
    @torch.no_grad()
    def load_hf_state_dict(self, tensors) -> None:
        """Tensor names: embed, loop.in, l<i>.norm1|ls1|ls2, l<i>.mix.*
        (attention: q|k|v|o; latent_attention: q|dkv|dkv.norm|uk|uv|o; gla:
        q|k|v|g|o|a1|a2|a2.b|norm), l<i>.mlp.gate|up|down or
        l<i>.mlp.router|router.b|e<j>.gate|up|down, final.norm, head."""

        def get(name):
            t = tensors[name]
            return t() if callable(t) else t

        self.embed.copy_(get("embed").to(self.dtype))
        self.head.copy_(get("head").to(self.dtype))
        self.final_norm.copy_(get("final.norm").float())
        if self.loop_x is not None:
            w = get("loop.in").to(self.dtype)
            self.loop_x.copy_(w[:, : w.shape[0]])
            self.loop_x0.copy_(w[:, w.shape[0] :])
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            layer.norm1.copy_(get(p + "norm1").float())
            layer.ls1.copy_(get(p + "ls1").float())
            layer.mix.load(get, p + "mix.")
            if layer.mlp is not None:
                layer.ls2.copy_(get(p + "ls2").float())
                layer.mlp.load(get, p + "mlp.")

    def num_parameters(self) -> int:
        return sum(p.numel() for p in self.parameters())
