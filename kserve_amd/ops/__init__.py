"""Custom op dispatch: CDNA4 HIP kernels on GPU, torch reference on CPU.

Policy: GPU tensors MUST run the native
extension — if ``kserve_amd_C`` is missing on a CUDA/ROCm device the op
raises ``NoNativeExtension`` instead of silently falling back to eager
torch. CPU tensors use the fp32 torch reference (tests, engine logic).
"""

from __future__ import annotations

from typing import Optional, Tuple

import torch

from kserve_amd.errors import NoNativeExtension
from kserve_amd.ops import torch_ref

_C = None
_IMPORT_ERROR: Optional[str] = None
try:
    import kserve_amd_C as _C  # built in-tree by setup.py (travels to GPU box)
except ImportError as e:  # pragma: no cover - exercised on GPU box
    _IMPORT_ERROR = str(e)


# kernels of the 32-bit-residual / recurrent-state mechanisms (own module so
# a model built from them compiles nothing else); carries the samplers too
_SEQ = None
_SEQ_IMPORT_ERROR: Optional[str] = None
try:
    import kserve_amd_seq_C as _SEQ
except ImportError as e:  # pragma: no cover - exercised on GPU box
    _SEQ_IMPORT_ERROR = str(e)


def has_native() -> bool:
    return _C is not None


def has_native_seq() -> bool:
    return _SEQ is not None


def _native_seq(op: str):
    if _SEQ is None:
        raise NoNativeExtension(op, f"(import error: {_SEQ_IMPORT_ERROR})")
    return _SEQ


def _native_sampling(op: str):
    """The samplers are linked into every extension module."""
    return _C if _C is not None else _native_seq(op)


def _native(op: str):
    if _C is None:
        raise NoNativeExtension(op, f"(import error: {_IMPORT_ERROR})")
    return _C


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    if x.is_cuda:
        out = torch.empty_like(x)
        _native("rms_norm").rms_norm(out, x, weight, eps)
        return out
    return torch_ref.rms_norm(x, weight, eps)


def fused_add_rms_norm(
    x: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor, eps: float
) -> Tuple[torch.Tensor, torch.Tensor]:
    """In-place on GPU: x <- rmsnorm(x+residual), residual <- x+residual."""
    if x.is_cuda:
        _native("fused_add_rms_norm").fused_add_rms_norm(x, residual, weight, eps)
        return x, residual
    return torch_ref.fused_add_rms_norm(x, residual, weight, eps)


def silu_and_mul(x: torch.Tensor) -> torch.Tensor:
    if x.is_cuda:
        d = x.shape[-1] // 2
        out = torch.empty(
            (*x.shape[:-1], d), dtype=x.dtype, device=x.device
        )
        _native("silu_and_mul").silu_and_mul(out, x)
        return out
    return torch_ref.silu_and_mul(x)


def rotary_embedding(
    positions: torch.Tensor,
    q: torch.Tensor,
    k: torch.Tensor,
    cos_sin_cache: torch.Tensor,
) -> Tuple[torch.Tensor, torch.Tensor]:
    """Neox-style RoPE. GPU path mutates q/k in place and returns them."""
    if q.is_cuda:
        _native("rotary_embedding").rotary_embedding(positions, q, k, cos_sin_cache)
        return q, k
    return torch_ref.rotary_embedding(positions, q, k, cos_sin_cache)


def reshape_and_cache(
    k: torch.Tensor,
    v: torch.Tensor,
    k_cache: torch.Tensor,
    v_cache: torch.Tensor,
    slot_mapping: torch.Tensor,
) -> None:
    if k.is_cuda:
        _native("reshape_and_cache").reshape_and_cache(
            k, v, k_cache, v_cache, slot_mapping
        )
        return
    torch_ref.reshape_and_cache(k, v, k_cache, v_cache, slot_mapping)


def paged_attention_decode(
    q: torch.Tensor,
    k_cache: torch.Tensor,
    v_cache: torch.Tensor,
    block_tables: torch.Tensor,
    context_lens: torch.Tensor,
    scale: float,
    out: Optional[torch.Tensor] = None,
    window: int = 0,
) -> torch.Tensor:
    if q.is_cuda:
        if out is None:
            out = torch.empty_like(q)
        _native("paged_attention_decode").paged_attention_decode(
            out, q, k_cache, v_cache, block_tables, context_lens, scale,
            window,
        )
        return out
    return torch_ref.paged_attention_decode(
        q, k_cache, v_cache, block_tables, context_lens, scale,
        window=window,
    )


def flash_prefill_varlen(
    q: torch.Tensor,
    k: torch.Tensor,
    v: torch.Tensor,
    cu_seqlens: torch.Tensor,
    max_seqlen: int,
    scale: float,
    window: int = 0,
) -> torch.Tensor:
    if q.is_cuda:
        out = torch.empty_like(q)
        _native("flash_prefill").flash_prefill_varlen(
            out, q, k, v, cu_seqlens, int(max_seqlen), scale,
            causal=True, window=window,
        )
        return out
    return torch_ref.flash_prefill_varlen(
        q, k, v, cu_seqlens, scale, causal=True, window=window
    )


def context_attention_varlen(
    q: torch.Tensor,
    k_cache: torch.Tensor,
    v_cache: torch.Tensor,
    block_tables: torch.Tensor,
    cu_seqlens_q: torch.Tensor,
    context_lens: torch.Tensor,
    max_q_len: int,
    scale: float,
    window: int = 0,
) -> torch.Tensor:
    """Prefill attention against the paged cache (chunked prefill): the
    chunk's KV must already be written to the cache; queries attend causally
    to the whole per-seq context (bounded below by the sliding window when
    window > 0)."""
    if q.is_cuda:
        out = torch.empty_like(q)
        _native("context_prefill").context_prefill_varlen(
            out, q, k_cache, v_cache, block_tables, context_lens,
            cu_seqlens_q, int(max_q_len), scale, window
        )
        return out
    return torch_ref.context_attention_varlen(
        q, k_cache, v_cache, block_tables, cu_seqlens_q, context_lens, scale,
        window=window,
    )


def greedy_sample(logits: torch.Tensor) -> torch.Tensor:
    if logits.is_cuda:
        # bf16 or fp32: an fp32 argmax sees every bit of the logits
        out = torch.empty(
            logits.shape[0], dtype=torch.int64, device=logits.device
        )
        _native_sampling("greedy_sample").greedy_sample(out, logits)
        return out
    return torch_ref.greedy_sample(logits)


def random_sample(
    logits: torch.Tensor,
    temperatures: torch.Tensor,
    top_p: torch.Tensor,
    top_k: torch.Tensor,
    seeds: Optional[torch.Tensor] = None,
    generator: Optional[torch.Generator] = None,
    min_p: Optional[torch.Tensor] = None,
) -> torch.Tensor:
    """Temperature/top-k/top-p/min-p sampling.

    GPU: one fused HIP kernel. Plain temperature sampling is Gumbel-max;
    top-k/top-p use a bf16 radix-histogram select (exact k-th value / mass
    threshold, no sort) followed by Gumbel-max over the surviving set.
    min_p (rare) routes to the fp32 sort path.
    """
    has_min_p = min_p is not None and bool((min_p > 0).any())
    if logits.is_cuda and seeds is not None and not has_min_p:
        if logits.dtype != torch.bfloat16:
            logits = logits.to(torch.bfloat16)  # the fused samplers' format
        out = torch.empty(
            logits.shape[0], dtype=torch.int64, device=logits.device
        )
        needs_trunc = bool((top_p < 1.0).any()) or bool((top_k > 0).any())
        if needs_trunc:
            _native_sampling("random_sample").topk_topp_sample(
                out, logits, temperatures, top_p, top_k.to(torch.int32), seeds
            )
        else:
            _native_sampling("random_sample").gumbel_sample(
                out, logits, temperatures, top_k.to(torch.int32), seeds
            )
        return out
    # min-p (or CPU): fp32 sort path
    return torch_ref.random_sample(
        logits, temperatures, top_p, top_k, generator=generator, min_p=min_p
    )


def linear(x: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """GEMM dispatch: custom MFMA skinny-GEMM for decode-sized batches
    (weight-streaming regime where hipBLASLt underperforms ~4x on gfx950 —
    see tools/gemm_bench.py), hipBLASLt via F.linear otherwise."""
    import torch.nn.functional as F

    # measured crossover (tools/gemm_bench.py on MI355X): the custom kernel
    # beats hipBLASLt only for small token batches on qkv/o-sized shapes;
    # hipBLASLt keeps the wide-M / large-K / large-N shapes.
    if (
        _C is not None
        and x.is_cuda
        and bias is None
        and x.dim() == 2
        and 0 < x.shape[0] <= 64
        and weight.shape[0] % 64 == 0
        and weight.shape[0] <= 8192
        and weight.shape[1] % 64 == 0
        and weight.shape[1] <= 8192
        and x.stride(1) == 1
    ):
        out = torch.empty(
            (x.shape[0], weight.shape[0]), dtype=x.dtype, device=x.device
        )
        _C.skinny_gemm(out, x, weight)
        return out
    return F.linear(x, weight, bias)


def layer_norm(x, weight, bias, eps: float):
    if x.is_cuda:
        out = torch.empty_like(x)
        _native("layer_norm").layer_norm(out, x, weight, bias, eps)
        return out
    return torch_ref.layer_norm(x, weight, bias, eps)


def fused_add_layer_norm(x, residual, weight, bias, eps: float):
    if x.is_cuda:
        out = torch.empty_like(x)
        _native("fused_add_layer_norm").fused_add_layer_norm(
            out, x, residual, weight, bias, eps
        )
        return out
    return torch_ref.fused_add_layer_norm(x, residual, weight, bias, eps)


def gelu(x):
    if x.is_cuda:
        out = torch.empty_like(x)
        _native("gelu").gelu(out, x)
        return out
    return torch_ref.gelu(x)


def flash_attn_varlen(q, k, v, cu_seqlens, max_seqlen, scale, causal=True):
    """Bidirectional-capable variant (encoder models)."""
    if q.is_cuda:
        out = torch.empty_like(q)
        _native("flash_prefill").flash_prefill_varlen(
            out, q, k, v, cu_seqlens, int(max_seqlen), scale, causal
        )
        return out
    return torch_ref.flash_prefill_varlen(q, k, v, cu_seqlens, scale, causal=causal)


def topk_topp_sample_into(
    out: torch.Tensor,
    logits: torch.Tensor,
    temperatures: torch.Tensor,
    top_p: torch.Tensor,
    top_k: torch.Tensor,
    seeds: torch.Tensor,
) -> torch.Tensor:
    """Destination-passing form of the fused sampler for hipGraph capture
    (static out buffer, per-row device seeds; see model_runner
    _ensure_sampled_graph). GPU-only."""
    if logits.dtype != torch.bfloat16:
        logits = logits.to(torch.bfloat16)  # the fused samplers' format
    _native_sampling("random_sample").topk_topp_sample(
        out, logits, temperatures, top_p,
        top_k if top_k.dtype == torch.int32 else top_k.to(torch.int32),
        seeds,
    )
    return out


# -- 32-bit residual stream, recurrent state, fp32 attention -----------------

def _f32_like(rows: int, cols: int, ref: torch.Tensor) -> torch.Tensor:
    return torch.empty((rows, cols), dtype=torch.float32, device=ref.device)


def embed_scale_sinpos(table, tokens, positions, inv_freq, scale: float):
    """fp32 [T, width]: table[token] * scale + interleaved sin/cos of
    position * inv_freq (the start of an fp32 residual stream)."""
    if table.is_cuda:
        out = _f32_like(tokens.shape[0], table.shape[1], table)
        # inv_freq None: no positional term
        _native_seq("embed_scale_sinpos").embed_scale_sinpos(
            out, table, tokens, positions, inv_freq, float(scale)
        )
        return out
    return torch_ref.embed_scale_sinpos(table, tokens, positions, inv_freq, scale)


def add_rms_norm_f32res(
    residual, weight, eps: float, w_offset: float, out_dtype,
    d0=None, s0: float = 1.0, d1=None, s1: float = 1.0, c0=None, c1=None,
    d1_index=None, d1_weights=None, d1_top: int = 1, want_out: bool = True,
):
    """residual (fp32, in place) += s0*c0*d0 + s1*c1*d1 (``c0``, ``c1``: fp32
    factors per channel, None for 1), then RMS norm with weight (w_offset + w);
    returns the normed rows in ``out_dtype`` (``weight`` None: the new residual
    itself; ``want_out`` off: nothing). With ``d1_index`` [T*d1_top] int32 the
    second delta of token t is the sum over k of d1_weights[t*d1_top + k] *
    d1[d1_index[t*d1_top + k]] (fp32 weights or None for 1)."""
    if residual.is_cuda:
        out = (
            torch.empty(residual.shape, dtype=out_dtype, device=residual.device)
            if want_out else None
        )
        _native_seq("add_rms_norm_f32res").add_rms_norm_f32res(
            residual, d0, float(s0), d1, float(s1), weight, float(w_offset),
            float(eps), out, c0, c1, d1_index, d1_weights, int(d1_top),
        )
        return out
    return torch_ref.add_rms_norm_f32res(
        residual, weight, eps, w_offset, out_dtype, d0, s0, d1, s1, c0, c1,
        d1_index, d1_weights, d1_top, want_out,
    )


def gated_group_rms_norm(
    y, z, weight, eps: float, groups: int, out_dtype, gate_after: bool = False,
    gate_sigmoid: bool = False,
):
    """RMS norm of fp32 ``y`` in ``groups`` equal parts with a silu(z) gate
    (``gate_sigmoid``: sigmoid(z)): on the input of the norm, or
    (``gate_after``) on its output. ``weight``
    may be shorter than a row (it repeats: one vector shared by the groups)
    or None."""
    if y.is_cuda:
        out = torch.empty(y.shape, dtype=out_dtype, device=y.device)
        _native_seq("gated_group_rms_norm").gated_group_rms_norm(
            out, y, z, weight, float(eps), int(groups), bool(gate_after),
            bool(gate_sigmoid),
        )
        return out
    return torch_ref.gated_group_rms_norm(
        y, z, weight, eps, groups, out_dtype, gate_after, gate_sigmoid
    )


def causal_conv_silu(
    x_in, w, bias, conv_state, positions, seq_of_token, cu_seqlens, slots,
    silu: bool = True,
):
    """Depthwise causal conv (+ silu) over a flat varlen batch; reads and then
    advances each sequence's conv history in ``conv_state[slot]``."""
    if x_in.is_cuda:
        out = _f32_like(x_in.shape[0], x_in.shape[1], x_in)
        _native_seq("causal_conv_silu").causal_conv_silu(
            out, x_in, w, bias, conv_state, positions, seq_of_token,
            cu_seqlens, slots, bool(silu),
        )
        return out
    return torch_ref.causal_conv_silu(
        x_in, w, bias, conv_state, positions, cu_seqlens, slots, silu
    )


def ssd_scan(
    xbc, dt_raw, dt_bias, a_log, d_skip, state, positions, cu_seqlens, slots,
    groups: int,
):
    """State-space scan; carries ``state[slot]`` ([heads, P, N] fp32)."""
    if xbc.is_cuda:
        heads, P = state.shape[1], state.shape[2]
        y = _f32_like(xbc.shape[0], heads * P, xbc)
        _native_seq("ssd_scan").ssd_scan(
            y, xbc, dt_raw, dt_bias, a_log, d_skip, state, positions,
            cu_seqlens, slots, int(groups),
        )
        return y
    return torch_ref.ssd_scan(
        xbc, dt_raw, dt_bias, a_log, d_skip, state, positions, cu_seqlens,
        slots, groups,
    )


def qk_norm_temp_cache(
    q, k, v, qw, kw, positions, slot_mapping, k_cache, v_cache, eps: float,
    temp_coef: float, temp_every: int, heads: int,
):
    if q.is_cuda:
        q_out = _f32_like(q.shape[0], q.shape[1], q)
        _native_seq("qk_norm_temp_cache").qk_norm_temp_cache(
            q_out, q, k, v, qw, kw, positions, slot_mapping, k_cache, v_cache,
            float(eps), float(temp_coef), int(temp_every), int(heads),
        )
        return q_out
    return torch_ref.qk_norm_temp_cache(
        q, k, v, qw, kw, positions, slot_mapping, k_cache, v_cache, eps,
        temp_coef, temp_every, heads,
    )


def ctx_attention_f32(
    q, k_cache, v_cache, block_tables, cu_q, ctx_lens, scale: float,
    max_q_len: int, heads: int, gate=None, out_dtype=torch.float32,
    sink=None, chunk: int = 0, out_inv_freq=None, window: int = 0,
    maps: int = 1, softcap: float = 0.0, keep_first: int = 0,
):
    """Paged causal attention with fp32 scores and weights. Optional parts:
    ``gate`` [T, heads] (output times sigmoid), ``sink`` [heads] fp32 (one
    more term exp(sink) in the softmax denominator), ``chunk`` (a query sees
    only keys of its own block of that many positions), ``window`` (a query
    sees itself and the window-1 positions before it, and with ``keep_first``
    the sequence's first positions), ``out_inv_freq``
    [vdim/2] fp32 (each head output turned back by its query position).
    ``v_cache`` may be a view of the leading columns of ``k_cache`` (values
    that are a prefix of the keys are stored once). ``maps``: every cached key
    row holds that many keys side by side, and query head h reads number
    h % maps of its group's (all of them share the group's values); ``softcap``:
    scores become softcap * tanh(score / softcap). With bf16 pages the output
    may be bf16 or fp32."""
    if q.is_cuda:
        out = torch.empty(
            (q.shape[0], heads * v_cache.shape[3]), dtype=out_dtype,
            device=q.device,
        )
        _native_seq("ctx_attention_f32").ctx_attention_f32(
            out, q, k_cache, v_cache, block_tables, cu_q, ctx_lens, gate,
            float(scale), int(max_q_len), int(heads), sink, int(chunk),
            out_inv_freq, int(window), int(maps), float(softcap),
            int(keep_first),
        )
        return out
    return torch_ref.ctx_attention_f32(
        q, k_cache, v_cache, block_tables, cu_q, ctx_lens, scale, heads,
        gate, out_dtype, sink, chunk, out_inv_freq, window, maps, softcap,
        keep_first,
    )


def qk_headnorm_rope_cache(
    q, k, v, qw, kw, positions, slot_mapping, k_cache, v_cache, eps: float,
    heads: int, qk_inv_freq=None, v_unit_norm: bool = False, v_inv_freq=None,
    pairs: bool = False, rot_mult: float = 1.0, maps: int = 1,
    qk_norm: bool = True,
):
    """Per-head q/k RMS norm (weights [dim]; off with ``qk_norm``) + rotary positions (``pairs``:
    coordinate 2i turns with 2i+1 instead of i with i + half; turned
    coordinates times ``rot_mult``), optional unit-norm and rotation of the
    values, KV page scatter (``maps`` k heads share a cached row and a value
    head); returns q fp32. q, k, v may be fp32 beside bf16 pages."""
    if q.is_cuda:
        q_out = _f32_like(q.shape[0], q.shape[1], q)
        _native_seq("qk_headnorm_rope_cache").qk_headnorm_rope_cache(
            q_out, q, k, v, qw, kw, positions, slot_mapping, k_cache, v_cache,
            float(eps), int(heads), qk_inv_freq, bool(v_unit_norm), v_inv_freq,
            bool(pairs), float(rot_mult), int(maps), bool(qk_norm),
        )
        return q_out
    return torch_ref.qk_headnorm_rope_cache(
        q, k, v, qw, kw, positions, slot_mapping, k_cache, v_cache, eps,
        heads, qk_inv_freq, v_unit_norm, v_inv_freq, pairs, rot_mult, maps,
        qk_norm,
    )


def post_norm_add_rms_norm(
    residual, delta, post_gain: float, layer_scale, eps: float,
    next_gain: float, out_dtype, add_rows=None, add_vec=None,
    want_out: bool = True,
):
    """Close one sandwich-normed sublayer and open the next in one pass over
    the fp32 residual (in place): += layer_scale * scalar-gain RMS norm of the
    sublayer output, += optional per-token rows and one shared row, then the
    scalar-gain RMS norm of the result in ``out_dtype``."""
    if residual.is_cuda:
        out = (
            torch.empty(residual.shape, dtype=out_dtype, device=residual.device)
            if want_out else None
        )
        _native_seq("post_norm_add_rms_norm").post_norm_add_rms_norm(
            residual, delta, float(post_gain), layer_scale, float(eps),
            float(next_gain), out, add_rows, add_vec,
        )
        return out
    return torch_ref.post_norm_add_rms_norm(
        residual, delta, post_gain, layer_scale, eps, next_gain, out_dtype,
        add_rows, add_vec, want_out,
    )


def router_topk(
    logits, top: int, softmax: bool = False, renorm: bool = False,
    dense: bool = False, correction=None, renorm_eps: float = 0.0,
    weight_scale: float = 1.0, over_chosen: bool = False,
):
    """fp32 router logits [T, E] -> (expert ids int32 [T, top], weights fp32
    [T, top], dense [T, E] weights or None) by sigmoid (or softmax) score;
    with ``correction`` [E] fp32 the choice goes by score + correction.
    ``over_chosen``: the largest logits, weighted by the softmax over those
    logits only."""
    if logits.is_cuda:
        T, E = logits.shape
        idx = torch.empty((T, top), dtype=torch.int32, device=logits.device)
        w = torch.empty((T, top), dtype=torch.float32, device=logits.device)
        dw = (
            torch.empty((T, E), dtype=torch.float32, device=logits.device)
            if dense else None
        )
        _native_seq("router_topk").router_topk(
            idx, w, dw, logits, bool(softmax), bool(renorm), correction,
            float(renorm_eps), float(weight_scale), bool(over_chosen),
        )
        return idx, w, dw
    return torch_ref.router_topk(
        logits, top, softmax, renorm, dense, correction, renorm_eps,
        weight_scale, over_chosen,
    )


def route_tokens(
    h, router, top: int, softmax: bool = False, renorm: bool = False,
    dense: bool = False, want_logits: bool = False, correction=None,
    renorm_eps: float = 0.0, weight_scale: float = 1.0,
    over_chosen: bool = False, bias=None,
):
    """The router in one kernel: fp32 logits of h [T, W] (activation dtype)
    against fp32 router rows [E, W] (+ fp32 ``bias`` [E]), scores, the ``top``
    experts (as in ``router_topk``). Returns
    (expert ids int32 [T, top], weights fp32 [T, top], dense [T, E] weights or
    None, logits fp32 [T, E] or None)."""
    if h.is_cuda:
        T, E = h.shape[0], router.shape[0]
        dev = h.device
        idx = torch.empty((T, top), dtype=torch.int32, device=dev)
        w = torch.empty((T, top), dtype=torch.float32, device=dev)
        dw = torch.empty((T, E), dtype=torch.float32, device=dev) if dense else None
        lg = torch.empty((T, E), dtype=torch.float32, device=dev) if want_logits else None
        _native_seq("route_tokens").route_tokens(
            idx, w, dw, lg, h, router, bool(softmax), bool(renorm), correction,
            float(renorm_eps), float(weight_scale), bool(over_chosen), bias,
        )
        return idx, w, dw, lg
    return torch_ref.route_tokens(
        h, router, top, softmax, renorm, dense, want_logits, correction,
        renorm_eps, weight_scale, over_chosen, bias,
    )


def gather_scale_rows(x, rows, scales=None):
    """out[r] = x[rows[r]] * scales[r] in x's dtype (rows int32, scales fp32
    or None for a plain gather)."""
    if x.is_cuda:
        out = torch.empty((rows.numel(), x.shape[1]), dtype=x.dtype, device=x.device)
        _native_seq("gather_scale_rows").gather_scale_rows(out, x, rows, scales)
        return out
    return torch_ref.gather_scale_rows(x, rows, scales)


def combine_rows(
    y, index, top: int, extra=None, weights=None, scaled=None, scaled_w=None
):
    """fp32 out[t] = sum_k weights[t*top + k] * y[index[t*top + k]]
    (+ extra[t]) (+ scaled_w[t] * scaled[t]); weights (fp32) default to 1."""
    if y.is_cuda:
        out = _f32_like(index.numel() // top, y.shape[1], y)
        _native_seq("combine_rows").combine_rows(
            out, y, index, int(top), extra, weights, scaled, scaled_w
        )
        return out
    return torch_ref.combine_rows(y, index, top, extra, weights, scaled, scaled_w)


def clamped_swiglu(x, alpha: float, limit: float):
    if x.is_cuda:
        out = torch.empty(
            (*x.shape[:-1], x.shape[-1] // 2), dtype=x.dtype, device=x.device
        )
        _native_seq("clamped_swiglu").clamped_swiglu(
            out, x, float(alpha), float(limit)
        )
        return out
    return torch_ref.clamped_swiglu(x, alpha, limit)


# -- latent attention, post-layer-norm residual, plain feed-forwards ----------

def post_layer_norm_add(
    residual, delta, weight, mult: float, eps: float, out_dtype,
    next_weight=None, want_out: bool = True,
):
    """fp32 residual (in place) += mult * LayerNorm(delta) * weight (no bias)
    when ``delta`` is given; returns the new residual in ``out_dtype`` or,
    with ``next_weight``, its layer norm times that weight."""
    if residual.is_cuda:
        out = (
            torch.empty(residual.shape, dtype=out_dtype, device=residual.device)
            if want_out else None
        )
        _native_seq("post_layer_norm_add").post_layer_norm_add(
            residual, delta, weight, float(mult), float(eps), out, next_weight
        )
        return out
    return torch_ref.post_layer_norm_add(
        residual, delta, weight, mult, eps, out_dtype, next_weight, want_out
    )


def latent_norm_rope_cache(
    proj, q_rank: int, kv_rank: int, rot_dim: int, qw, kw, positions,
    slot_mapping, cache, eps: float, inv_freq, pairs: bool = True,
    rot_mult: float = 1.0,
):
    """Rows [query latent | kv latent | key part | ...] -> the RMS-normed
    query latent (returned, activation dtype; None when ``q_rank`` is 0) and,
    when ``cache`` is given, [normed kv latent | key part rotated in pairs
    (2i, 2i+1)] scattered into the paged cache [blocks, 1, block,
    kv_rank + rot_dim]. ``pairs`` off: coordinate i turns with i + half;
    turned coordinates times ``rot_mult``."""
    if proj.is_cuda:
        cq = (
            torch.empty((proj.shape[0], q_rank), dtype=proj.dtype, device=proj.device)
            if q_rank else None
        )
        _native_seq("latent_norm_rope_cache").latent_norm_rope_cache(
            cq, proj, int(q_rank), int(kv_rank), int(rot_dim), qw, kw,
            positions, slot_mapping, cache, float(eps), inv_freq, bool(pairs),
            float(rot_mult),
        )
        return cq
    return torch_ref.latent_norm_rope_cache(
        proj, q_rank, kv_rank, rot_dim, qw, kw, positions, slot_mapping,
        cache, eps, inv_freq, pairs, rot_mult,
    )


def head_matmul_rope(
    x, w, heads: int, tail: int = 0, positions=None, inv_freq=None,
    out_dtype=None, pairs: bool = True, rot_mult: float = 1.0,
):
    """Per-head matrix product with an optional rotated tail:
    x [T, heads*(k + tail)], w [heads, n, k] -> [T, heads*(n + tail)], the
    tail coordinates turned in pairs (``pairs`` off: i with i + half) by the
    token's position and multiplied by ``rot_mult``."""
    out_dtype = out_dtype or x.dtype
    if x.is_cuda:
        n = w.shape[1]
        out = torch.empty(
            (x.shape[0], heads * (n + tail)), dtype=out_dtype, device=x.device
        )
        _native_seq("head_matmul_rope").head_matmul_rope(
            out, x, w, int(heads), int(tail), positions, inv_freq, bool(pairs),
            float(rot_mult),
        )
        return out
    return torch_ref.head_matmul_rope(
        x, w, heads, tail, positions, inv_freq, out_dtype, pairs, rot_mult
    )


def glu_silu_scale(x, scales=None):
    """[rows, 2 d] = [gate | up] -> silu(gate) * up (* scales[row])."""
    if x.is_cuda:
        out = torch.empty(
            (x.shape[0], x.shape[1] // 2), dtype=x.dtype, device=x.device
        )
        _native_seq("glu_silu_scale").glu_silu_scale(out, x, scales)
        return out
    return torch_ref.glu_silu_scale(x, scales)


def bias_gelu_tanh(x, bias):
    """gelu (tanh form) of x + bias, in x's dtype."""
    if x.is_cuda:
        out = torch.empty_like(x)
        _native_seq("bias_gelu_tanh").bias_gelu_tanh(out, x, bias)
        return out
    return torch_ref.bias_gelu_tanh(x, bias)


# -- linear-attention recurrences, squared-relu experts, capped logits --------

def rope_scale_heads(
    x, positions, inv_freq, heads_a: int, scale_a: float, heads_b: int,
    scale_b: float, dim: int,
):
    """fp32 copy of rows x [T, width]: the first ``heads_a`` heads of ``dim``
    columns get rotary positions on their first 2*len(inv_freq) coordinates
    (i pairs with i + half) and are multiplied by scale_a, the next
    ``heads_b`` likewise with scale_b; further columns are only widened."""
    if x.is_cuda:
        out = _f32_like(x.shape[0], x.shape[1], x)
        _native_seq("rope_scale_heads").rope_scale_heads(
            out, x, positions, inv_freq, int(heads_a), float(scale_a),
            int(heads_b), float(scale_b), int(dim),
        )
        return out
    return torch_ref.rope_scale_heads(
        x, positions, inv_freq, heads_a, scale_a, heads_b, scale_b, dim
    )


def unit_norm_heads(
    x, heads_a: int, scale_a: float, heads_b: int, scale_b: float, dim: int,
    eps: float,
):
    """In place on fp32 rows: the first ``heads_a`` heads of ``dim`` columns
    become x / sqrt(sum(x^2) + eps) * scale_a, the next ``heads_b`` likewise
    with scale_b; further columns are left alone."""
    if x.is_cuda:
        _native_seq("unit_norm_heads").unit_norm_heads(
            x, int(heads_a), float(scale_a), int(heads_b), float(scale_b),
            int(dim), float(eps),
        )
        return x
    return torch_ref.unit_norm_heads(x, heads_a, scale_a, heads_b, scale_b, dim, eps)


def linear_scan(
    q, k, v, state, positions, cu_seqlens, slots, qk_heads: int,
    decay=None, a_raw=None, b_raw=None, a_log=None, dt_bias=None,
    channel_decay=None, q_scale: float = 1.0,
):
    """Linear-attention recurrence over a flat varlen batch; carries
    ``state[slot]`` ([heads, V, K] fp32). q, k [T, qk_heads*K] and
    v [T, heads*V] are fp32 (rows may be strided). With ``decay`` [heads]:
    S <- d S + k v^T. Without: the gated delta rule with
    g = exp(-exp(a_log) softplus(a_raw + dt_bias)), b = sigmoid(b_raw):
    S <- g S; S <- S + k (b (v - S^T k))^T; ``channel_decay`` [T, heads*K] fp32
    gives g per head and key channel (then a_raw, a_log, dt_bias are not
    used); ``channel_decay`` without ``b_raw``: S <- diag(g) S + k v^T, and
    q, k, v may be bf16. Output o = S^T q * q_scale, fp32."""
    if q.is_cuda:
        heads, V = state.shape[1], state.shape[2]
        o = _f32_like(q.shape[0], heads * V, q)
        _native_seq("linear_scan").linear_scan(
            o, q, k, v, decay, a_raw, b_raw, a_log, dt_bias, channel_decay,
            state, positions, cu_seqlens, slots, int(qk_heads), float(q_scale),
        )
        return o
    return torch_ref.linear_scan(
        q, k, v, state, positions, cu_seqlens, slots, qk_heads, decay, a_raw,
        b_raw, a_log, dt_bias, channel_decay, q_scale,
    )


def lowrank_channel_decay(low, w2, bias, tau: float):
    """Decays of a gated linear recurrence: sigmoid(z)^(1/tau) with
    z = low @ w2^T + bias in fp32; low [T, r] in the activation dtype (rows may
    be strided), w2 [n, r] and bias [n] fp32 -> fp32 [T, n]."""
    if low.is_cuda:
        out = _f32_like(low.shape[0], w2.shape[0], low)
        _native_seq("lowrank_channel_decay").lowrank_channel_decay(
            out, low, w2, bias, float(tau)
        )
        return out
    return torch_ref.lowrank_channel_decay(low, w2, bias, tau)


def linear_f32out(x, w):
    """x @ w^T with an fp32 result that is never rounded to the activation
    dtype (a product that replaces an fp32 stream, or logits)."""
    if x.dtype == torch.float32:
        return torch.nn.functional.linear(x, w)
    if x.is_cuda:
        return torch.mm(x, w.t(), out_dtype=torch.float32)
    return torch_ref.linear_f32out(x, w)


def relu2_scale(x, scales=None):
    """max(x, 0)^2 (* scales[row]) in x's dtype."""
    if x.is_cuda:
        out = torch.empty_like(x)
        _native_seq("relu2_scale").relu2_scale(out, x, scales)
        return out
    return torch_ref.relu2_scale(x, scales)


def scale_softcap(x, scale: float, cap: float):
    """fp32 cap * tanh(x * scale / cap); cap 0 leaves x * scale."""
    if x.is_cuda:
        out = torch.empty(x.shape, dtype=torch.float32, device=x.device)
        _native_seq("scale_softcap").scale_softcap(out, x, float(scale), float(cap))
        return out
    return torch_ref.scale_softcap(x, scale, cap)


# -- two score maps, mixed score heads, per-channel decays, grouped norms -----

def post_group_norm_add(
    residual, delta, weight, groups: int, eps: float, out_dtype, delta2=None,
    pre_w=None, pre_w2=None, next_weight=None, want_out: bool = True,
):
    """fp32 residual (in place) += GroupRMS(d) * weight, where d is ``delta``
    or, with ``delta2``, half of rms(delta) * pre_w + rms(delta2) * pre_w2;
    returns the new residual in ``out_dtype`` or, with ``next_weight``, its
    group RMS norm times that weight."""
    if residual.is_cuda:
        out = (
            torch.empty(residual.shape, dtype=out_dtype, device=residual.device)
            if want_out else None
        )
        _native_seq("post_group_norm_add").post_group_norm_add(
            residual, delta, weight, delta2, pre_w, pre_w2, int(groups),
            float(eps), out, next_weight,
        )
        return out
    return torch_ref.post_group_norm_add(
        residual, delta, weight, groups, eps, out_dtype, delta2, pre_w,
        pre_w2, next_weight, want_out,
    )


def diff_combine(o, lam, heads: int, eps: float, mult: float, out_dtype):
    """fp32 rows with two outputs per head side by side -> their difference
    first - lam * second (lam: fp32 tensor of one element), divided by its RMS
    over the head, times ``mult``."""
    if o.is_cuda:
        out = torch.empty(
            (o.shape[0], o.shape[1] // 2), dtype=out_dtype, device=o.device
        )
        _native_seq("diff_combine").diff_combine(
            out, o, lam, int(heads), float(eps), float(mult)
        )
        return out
    return torch_ref.diff_combine(o, lam, heads, eps, mult, out_dtype)


def talk_prep_cache(
    q, k, w, slot_mapping, k_cache, k_scale, eps: float,
):
    """Whole-row RMS norm of q times ``w`` (fp32, returned); the un-normed
    keys to the pages, 1 / rms of every key row to ``k_scale`` [blocks, block]
    (a weight of the key norm belongs into ``w``: it commutes into the
    query)."""
    if q.is_cuda:
        q_out = _f32_like(q.shape[0], q.shape[1], q)
        _native_seq("talk_prep_cache").talk_prep_cache(
            q_out, q, k, w, slot_mapping, k_cache, k_scale, float(eps)
        )
        return q_out
    return torch_ref.talk_prep_cache(
        q, k, w, slot_mapping, k_cache, k_scale, eps
    )


def talk_attention(
    q, k_cache, k_scale, block_tables, cu_q, ctx_lens, scale: float,
    max_q_len: int, heads: int, talk, bias, window: int = 0, gate=None,
    out_dtype=torch.float32,
):
    """Paged causal attention whose scores are mixed over the heads before
    the softmax: s_h = sum_g talk[h, g] (q_g . k) k_scale scale +
    bias[h, distance] (``bias`` [heads, n] fp32, constant past distance
    n - 1), one added to the softmax denominator, the cached keys as values,
    ``gate`` [T, heads*dim]: output times its sigmoid per element."""
    if q.is_cuda:
        out = torch.empty(
            (q.shape[0], heads * k_cache.shape[3]), dtype=out_dtype,
            device=q.device,
        )
        _native_seq("talk_attention").talk_attention(
            out, q, k_cache, k_scale, block_tables, cu_q, ctx_lens, talk, bias,
            gate, float(scale), int(max_q_len), int(heads), int(window),
        )
        return out
    return torch_ref.talk_attention(
        q, k_cache, k_scale, block_tables, cu_q, ctx_lens, scale, heads, talk,
        bias, window, gate, out_dtype,
    )


def delta_unit_decay(
    qkv, qk_heads: int, dim: int, q_scale: float, eps: float, a_raw, a_log,
    dt_bias,
):
    """What the channel-decay delta rule reads, in one pass per token: fp32
    rows [q | k | v] get unit-norm q and k heads in place (q times
    ``q_scale``); returns exp(-exp(a_log) softplus(a_raw + dt_bias)) per head
    and key channel, fp32 [T, heads*dim]."""
    if qkv.is_cuda:
        g = _f32_like(qkv.shape[0], a_raw.shape[1], qkv)
        _native_seq("delta_unit_decay").delta_unit_decay(
            qkv, g, a_raw, a_log, dt_bias, int(qk_heads), int(dim),
            float(q_scale), float(eps),
        )
        return g
    return torch_ref.delta_unit_decay(
        qkv, qk_heads, dim, q_scale, eps, a_raw, a_log, dt_bias
    )
