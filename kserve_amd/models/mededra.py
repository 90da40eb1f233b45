"""Mededra: a decoder whose layers are listed one by one in the config, each
reading the un-normed residual stream.

A sublayer reads the stream x itself; its OUTPUT goes through an RMS norm in
equal groups of channels before it is added:

    x += GroupRMS(mixer(x)) * w1
    x += GroupRMS(ff(x)) * w2        (if the layer has a feed-forward)

Mixers: ``DifferentialAttention`` ("attention"), or ``TalkingHeadsAttention``
beside ``ChannelDeltaMixer`` ("parallel"), both reading the same x through ONE
projection GEMM, each output RMS-normed over the width with a weight of its
own and half their sum taken. The feed-forward is ``SiluGLU``. The embedding
is scaled; logits are soft-capped with tanh.

The stream is fp32 whatever the activation dtype. "Norm the sublayer's output
(for a parallel mixer: norm both outputs and halve their sum first), add it,
hand the new stream to the next sublayer in the activation dtype" is one
kernel, and the last one applies the model's final norm instead.
"""

from __future__ import annotations

from typing import List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from kserve_amd import ops
from kserve_amd.engine.config import HybridLayerSpec, HybridModelConfig, SiluGLUSpec
from kserve_amd.models.mixers import (
    ChannelDeltaMixer,
    DifferentialAttention,
    SiluGLU,
    TalkingHeadsAttention,
)
from kserve_amd.parallel import comm


def _vec(n: int):
    return nn.Parameter(torch.empty(n, dtype=torch.float32), requires_grad=False)


class MededraLayer(nn.Module):
    def __init__(self, width: int, spec: HybridLayerSpec, eps: float, dtype):
        super().__init__()
        self.spec = spec
        self.attn = self.left = self.right = None
        if spec.differential is not None:
            self.attn = DifferentialAttention(width, spec.differential, eps, dtype)
        elif spec.talking is not None and spec.delta is not None:
            self.left = TalkingHeadsAttention(width, spec.talking, eps, dtype)
            self.right = ChannelDeltaMixer(width, spec.delta, eps, dtype)
            self.left_out = _vec(width)
            self.right_out = _vec(width)
        else:
            raise ValueError("a Mededra layer is differential or talking + delta")
        # both branches read the same input: one projection for the two
        self.fused_proj = None
        self.norm1 = _vec(width)
        self.mlp = None
        if spec.mlp is not None:
            if not isinstance(spec.mlp, SiluGLUSpec):
                raise ValueError(f"unsupported feed-forward {type(spec.mlp).__name__}")
            self.mlp = SiluGLU(width, spec.mlp.ff, dtype)
            self.norm2 = _vec(width)

    def finish_load(self):
        if self.attn is not None:
            self.attn.finish_load()
            return
        self.left.finish_load()
        self.right.finish_load()
        self.fused_proj = nn.Parameter(
            torch.cat([self.left.qkg.data, self.right.proj.data], dim=0),
            requires_grad=False,
        )
        # the branch modules keep views of the fused storage
        a = self.left.proj_width
        self.left.qkg.data = self.fused_proj.data[:a]
        self.right.proj.data = self.fused_proj.data[a:]

    def cache_entry(self):
        if self.attn is not None:
            return self.attn.kv_shape(), self.attn.state_shapes()
        return (
            self.left.kv_shape(),
            {**self.left.state_shapes(), **self.right.state_shapes()},
        )

    def mixer(self, h, positions, cache, meta):
        """Arguments that describe the mixer's output to the norm-and-add
        kernel: (delta, delta2, pre_w, pre_w2)."""
        if self.attn is not None:
            return self.attn(h, positions, cache, meta), None, None, None
        proj = F.linear(h, self.fused_proj)
        a = self.left.proj_width
        left = self.left.mix(proj[:, :a], positions, cache, meta)
        right = self.right.mix(proj[:, a:], positions, cache, meta)
        return left, right, self.left_out, self.right_out


class MededraForCausalLM(nn.Module):
    # every step attends through the paged cache (no separate un-paged
    # prefill kernel), and steps carry per-sequence state slots
    paged_prefill_only = True
    needs_state_slots = True

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
                "Mededra runs on one GPU per replica (no tensor/pipeline split)"
            )
        self.config = config
        dtype = dtype or (
            torch.bfloat16 if config.dtype == "bfloat16" else torch.float32
        )
        self.dtype = dtype
        W = config.hidden_size
        self.groups = config.norm_groups
        if self.groups < 1 or W % self.groups:
            raise ValueError("norm groups must divide the width")
        self.embed = nn.Parameter(
            torch.empty(config.vocab_size, W, dtype=dtype), requires_grad=False
        )
        self.layers = nn.ModuleList(
            [MededraLayer(W, spec, config.rms_norm_eps, dtype) for spec in config.layers]
        )
        self.num_local_layers = len(self.layers)
        self.final_norm = _vec(W)
        self.head = nn.Parameter(
            torch.empty(config.vocab_size, W, dtype=dtype), requires_grad=False
        )
        self.eps = config.rms_norm_eps
        # when a list, forward() appends the residual stream after each layer
        self.debug_residuals: Optional[List[torch.Tensor]] = None
        self.to(device)

    # -- cache layout (read by the model runner) ------------------------------
    def cache_layout(self):
        """Per layer: (kv_heads, key columns, value columns) and
        {name: (shape_per_slot, dtype)} of recurrent state (``k_scale``: the
        pages carry a factor per key row)."""
        return [layer.cache_entry() for layer in self.layers]

    # -- init -----------------------------------------------------------------
    @torch.no_grad()
    def random_init(self, std: float = 0.02, seed: int = 0):
        dev = self.embed.device
        gen = torch.Generator(device=dev)
        gen.manual_seed(seed)
        for name, p in self.named_parameters():
            if "fused_" in name:
                continue
            leaf = name.rsplit(".", 1)[-1]
            if leaf == "conv_w":
                p.normal_(0.0, 0.5, generator=gen)
            elif leaf == "rel":
                p.normal_(0.0, 1.0, generator=gen)
            elif leaf == "lambda_vecs":
                p.normal_(0.0, 0.1, generator=gen)
            elif p.dim() >= 2:
                # keep activations O(1) through the stack
                p.normal_(0.0, p.shape[-1] ** -0.5, generator=gen)
            elif leaf == "a_log":
                p.uniform_(-1.0, 1.0, generator=gen)
            elif leaf == "dt_bias":
                p.uniform_(-3.0, 0.0, generator=gen)
            else:  # norm weights
                p.fill_(1.0)
        for layer in self.layers:
            layer.finish_load()
        return self

    # -- forward --------------------------------------------------------------
    def forward(self, input_ids, positions, caches, meta):
        x = ops.embed_scale_sinpos(
            self.embed, input_ids, positions, None, self.config.embedding_scale
        )
        # (delta, weight of its norm, delta2, pre_w, pre_w2) not yet added
        pending = (None, None, None, None, None)
        dbg = self.debug_residuals
        for layer, cache in zip(self.layers, caches):
            h = self._add(x, pending)
            d, d2, w, w2 = layer.mixer(h, positions, cache, meta)
            pending = (d, layer.norm1, d2, w, w2)
            if layer.mlp is not None:
                h = self._add(x, pending)
                pending = (layer.mlp(h), layer.norm2, None, None, None)
            if dbg is not None:
                r = x.clone()
                self._add(r, pending)
                dbg.append(r)
        return self._add(x, pending, self.final_norm)

    def _add(self, x, pending, next_weight=None):
        d, w, d2, pw, pw2 = pending
        return ops.post_group_norm_add(
            x, d, w, self.groups, self.eps, self.dtype, delta2=d2, pre_w=pw,
            pre_w2=pw2, next_weight=next_weight,
        )

    def compute_logits(self, hidden):
        return ops.scale_softcap(
            F.linear(hidden, self.head), self.config.logit_scale,
            self.config.logit_softcap,
        )

    # -- weights ----------------------------------------------------------------
    @torch.no_grad()
    def load_hf_state_dict(self, tensors) -> None:
        """Tensor names: embed, l<i>.norm1|norm2, l<i>.mix.* (attention:
        q|k|v|o, .conv and .norm of them, lq1|lk1|lq2|lk2; parallel:
        left.q|k|g|o|rel|talk, left.q.norm|k.norm, right.q|k|v|b|o, right.*.conv,
        right.A_log|dt_bias|norm, right.a1|a2|g1|g2, left.out|right.out),
        l<i>.mlp.gate|up|down, final.norm, head."""

        def get(name):
            t = tensors[name]
            return t() if callable(t) else t

        self.embed.copy_(get("embed").to(self.dtype))
        self.head.copy_(get("head").to(self.dtype))
        self.final_norm.copy_(get("final.norm").float())
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            layer.norm1.copy_(get(p + "norm1").float())
            if layer.attn is not None:
                layer.attn.load(get, p + "mix.")
            else:
                layer.left.load(get, p + "mix.left.")
                layer.right.load(get, p + "mix.right.")
                layer.left_out.copy_(get(p + "mix.left.out").float())
                layer.right_out.copy_(get(p + "mix.right.out").float())
            if layer.mlp is not None:
                layer.norm2.copy_(get(p + "norm2").float())
                layer.mlp.load(get, p + "mlp.")
            layer.finish_load()

    def num_parameters(self) -> int:
        return sum(
            p.numel() for n, p in self.named_parameters() if "fused_" not in n
        )
