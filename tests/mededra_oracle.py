"""Plain float64 implementation of the Mededra design, written from its
equations: one function per mechanism, whole sequences, no caches, no
batching. Shares no code with ``kserve_amd``.

Notation: T tokens, positions 0..T-1; linear weights are [out, in].

  rms(x)       = x / sqrt(mean(x^2) + eps)
  grms(x)      = rms of each of `groups` equal parts of x
  conv(u, w)_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start
  yarn         : f_i = base^(-2i/n), slowed by 1/factor where the ramp between
                 the `fast` and `slow` turning numbers says so; cos and sin
                 times 1 + ln(factor)/10; pairs (2i, 2i+1) turn by p f_i
  differential : q, k, v -> conv; q, k rms-normed per head and map (weights of
                 size dim), turned; two softmax maps over the same values,
                 scores scaled then soft-capped, window; o = a1 - lam a2,
                 rms per head, times (1 - diff)
  talking      : q, k rms-normed over the whole projection; scores times
                 scale plus a bias by distance bucket, mixed over the heads by
                 T, window, softmax with 1 added to the denominator, values
                 are the un-normed keys, gate sigmoid(W_g h) per element
  delta        : q, k, v -> conv -> silu; q, k unit vectors (q times
                 dim^-1/2); per head and key channel
                 g = exp(-exp(A_h) softplus(W_a2 W_a1 h + dt)); S <- g S;
                 u = sigmoid(W_b h) (v - S^T k); S <- S + k u^T; o = S^T q;
                 o -> rms per head times a weight times sigmoid(W_g2 W_g1 h)
  parallel     : (rms(talking) w_l + rms(delta) w_r) / 2
  layer        : x <- x + grms(mixer(x)) w_1;  x <- x + grms(ff(x)) w_2
  model        : x = embed[tok] * scale; layers; head (grms(x) w_f);
                 cap tanh(. / cap)
"""

import math

import numpy as np
import torch


def _np(t):
    return t.detach().to(torch.float64).cpu().numpy()


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def group_rms(x, groups, eps):
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms(parts, eps).reshape(x.shape)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def softcap(z, cap):
    return cap * np.tanh(z / cap) if cap else z


def conv(u, w):
    """u [T, C]; w [C, taps], the last column weighs the current token."""
    T, C = u.shape
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, C)), u], axis=0)
    y = np.zeros((T, C))
    for j in range(taps):
        y += padded[j : j + T] * w[:, j][None, :]
    return y


def rotary_frequencies(rot):
    """-> (angles per position of the pairs, factor on cos and sin)."""
    n, base = rot["dims"], rot["base"]
    i = np.arange(n // 2, dtype=np.float64)
    f = float(base) ** (-2.0 * i / n)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def where(turns):
        return n * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(where(sc["fast"])), 0)
    hi = min(math.ceil(where(sc["slow"])), n - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return (f / sc["factor"]) * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, rot):
    """x [T, ..., dim]: coordinates 2i and 2i+1 of the first rot dims turn."""
    if not rot or not rot.get("dims"):
        return x
    n = rot["dims"]
    f, m = rotary_frequencies(rot)
    pos = np.arange(x.shape[0], dtype=np.float64)
    ang = (pos[:, None] * f[None, :]).reshape(
        (x.shape[0],) + (1,) * (x.ndim - 2) + (n // 2,)
    )
    c, s = m * np.cos(ang), m * np.sin(ang)
    out = x.copy()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


def visible(T, window):
    i = np.arange(T)[:, None]
    j = np.arange(T)[None, :]
    ok = j <= i
    if window:
        ok &= i - j < window
    return ok


def softmax(s):
    w = np.exp(s - s.max(axis=-1, keepdims=True))
    return w / w.sum(axis=-1, keepdims=True)


def softmax_plus_one(s):
    m = np.maximum(s.max(axis=-1, keepdims=True), 0.0)
    w = np.exp(s - m)
    return w / (w.sum(axis=-1, keepdims=True) + np.exp(-m))


def lam(W, p, diff):
    return (
        math.exp(float((W[p + "lq1"] * W[p + "lk1"]).sum()))
        - math.exp(float((W[p + "lq2"] * W[p + "lk2"]).sum()))
        + diff
    )


def differential(h, W, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    u = {}
    for n in ("q", "k", "v"):
        u[n] = h @ W[p + n].T
        if m.get("conv"):
            u[n] = conv(u[n], W[p + n + ".conv"])
    q = rms(u["q"].reshape(T, H, 2, D), eps) * W[p + "q.norm"]
    k = rms(u["k"].reshape(T, G, 2, D), eps) * W[p + "k.norm"]
    q, k = rotate_pairs(q, m.get("rot")), rotate_pairs(k, m.get("rot"))
    v = u["v"].reshape(T, G, V)
    ok = visible(T, (m.get("mask") or {}).get("size", 0))
    l = lam(W, p, m["diff"])
    o = np.zeros((T, H, V))
    for a in range(H):
        g = a // (H // G)
        maps = []
        for b in range(2):
            s = softcap((q[:, a, b] @ k[:, g, b].T) * m["scale"], m.get("softcap", 0.0))
            maps.append(softmax(np.where(ok, s, -np.inf)) @ v[:, g])
        o[:, a] = maps[0] - l * maps[1]
    o = rms(o, eps) * (1.0 - m["diff"])
    return o.reshape(T, H * V) @ W[p + "o"].T


def bucket(n, B, D):
    half = B // 2
    if n < half:
        return n
    return min(B - 1, half + math.floor(math.log(n / half) / math.log(D / half) * (B - half)))


def talking(h, W, p, m, eps):
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q = (rms(h @ W[p + "q"].T, eps) * W[p + "q.norm"]).reshape(T, H, D)
    kp = h @ W[p + "k"].T
    k = (rms(kp, eps) * W[p + "k.norm"]).reshape(T, G, D)
    v = kp.reshape(T, G, D)
    rel = W[p + "rel"]
    row = np.array([bucket(n, rel.shape[0], m["bias_max"]) for n in range(T)])
    dist = np.maximum(np.arange(T)[:, None] - np.arange(T)[None, :], 0)
    s = np.zeros((H, T, T))
    for a in range(H):
        s[a] = (q[:, a] @ k[:, a // (H // G)].T) * m["scale"] + rel[row[dist], a]
    mixed = np.einsum("hg,gij->hij", W[p + "talk"], s)
    ok = visible(T, (m.get("mask") or {}).get("size", 0))
    w = softmax_plus_one(np.where(ok[None], mixed, -np.inf))
    o = np.zeros((T, H, D))
    for a in range(H):
        o[:, a] = w[a] @ v[:, a // (H // G)]
    return (o.reshape(T, H * D) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k [T, G, D] unit vectors, v [T, H, V], g [T, H, D], beta [T, H]."""
    T, H, V = v.shape
    G, D = q.shape[1:]
    o = np.zeros((T, H, V))
    for a in range(H):
        c = a // (H // G)
        S = np.zeros((D, V))
        for t in range(T):
            S = g[t, a][:, None] * S
            u = beta[t, a] * (v[t, a] - S.T @ k[t, c])
            S = S + np.outer(k[t, c], u)
            o[t, a] = S.T @ q[t, c]
    return o


def delta(h, W, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def branch(n):
        return silu(conv(h @ W[p + n].T, W[p + n + ".conv"]))

    q = unit(branch("q").reshape(T, G, D)) * D ** -0.5
    k = unit(branch("k").reshape(T, G, D))
    v = branch("v").reshape(T, H, V)
    beta = sigmoid(h @ W[p + "b"].T)
    a = ((h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]).reshape(T, H, D)
    g = np.exp(-np.exp(W[p + "A_log"])[None, :, None] * softplus(a))
    o = rms(delta_rule(q, k, v, g, beta), eps) * W[p + "norm"]
    gate = sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T)
    return (o.reshape(T, H * V) * gate) @ W[p + "o"].T


def parallel(h, W, p, m, eps):
    l = rms(talking(h, W, p + "left.", m["left"], eps), eps) * W[p + "left.out"]
    r = rms(delta(h, W, p + "right.", m["right"], eps), eps) * W[p + "right.out"]
    return 0.5 * (l + r)


def feed_forward(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


MIXERS = {"attention": differential, "parallel": parallel}


def forward(cfg, sd, tokens, streams=None):
    """Logits [T, vocab] (float64 torch); ``streams`` collects the residual
    stream after every layer."""
    W = {k: _np(v) for k, v in sd.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = W["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[layer["type"]](x, W, p + "mix.", layer["mixer"], eps)
        x = x + group_rms(y, groups, eps) * W[p + "norm1"]
        if layer.get("mlp"):
            y = feed_forward(x, W, p + "mlp.")
            x = x + group_rms(y, groups, eps) * W[p + "norm2"]
        if streams is not None:
            streams.append(torch.from_numpy(x.copy()))
    lg = (group_rms(x, groups, eps) * W["final.norm"]) @ W["head"].T
    return torch.from_numpy(softcap(lg, cfg.get("logit_softcap", 0.0)))


# -- builders -----------------------------------------------------------------

def mlp(ff=24):
    return {"kind": "dense", "ff": ff}


def rot(dims=8, base=500.0, scaling=None):
    r = {"dims": dims, "base": base}
    if scaling:
        r["scaling"] = scaling
    return r


def yarn(factor=3.0, original=24, fast=4.0, slow=0.5):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def attention_layer(heads=4, kv_heads=2, dim=12, vdim=20, conv=3, diff=0.2,
                    scale=0.4, cap=5.0, window=9, rotation="default", mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "conv": conv, "diff": diff, "scale": scale, "softcap": cap,
         "mask": {"size": window}}
    m["rot"] = rot(scaling=yarn()) if rotation == "default" else rotation
    return {"type": "attention", "mixer": m, "mlp": mlp}


def parallel_layer(heads=4, kv_heads=2, dim=8, scale=0.5, window=21, bias_max=30,
                   buckets=8, d_heads=4, d_kv_heads=2, d_dim=12, d_vdim=8, conv=4,
                   a_rank=5, g_rank=7, mlp=None):
    """``buckets``, ``a_rank`` and ``g_rank`` show only in tensor shapes."""
    return {"type": "parallel", "mlp": mlp,
            "_shapes": {"buckets": buckets, "a_rank": a_rank, "g_rank": g_rank},
            "mixer": {
                "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
                         "scale": scale, "bias_max": bias_max, "mask": {"size": window}},
                "right": {"heads": d_heads, "kv_heads": d_kv_heads, "dim": d_dim,
                          "vdim": d_vdim, "conv": conv}}}


def make_config(layers, vocab=61, width=32, groups=2, eps=1e-5, emb_scale=3.0, cap=9.0):
    return {"architecture": "Mededra", "vocab": vocab, "width": width,
            "embedding": {"scale": emb_scale}, "norm": {"eps": eps, "groups": groups},
            "logit_softcap": cap, "layers": layers}


def random_weights(cfg, seed=0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def mat(o, i, gain=1.0):
        return (torch.randn(o, i, generator=g) * gain * i ** -0.5).to(dtype)

    def vec(n, std, mean=0.0):
        return (mean + std * torch.randn(n, generator=g)).to(dtype)

    sd = {"embed": torch.randn(cfg["vocab"], W, generator=g).to(dtype),
          "final.norm": vec(W, 0.1, 1.0), "head": mat(cfg["vocab"], W)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        sd[p + "norm1"] = vec(W, 0.2, 1.0)
        x = p + "mix."
        if layer["type"] == "attention":
            H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for n, rows in (("q", H * 2 * D), ("k", G * 2 * D), ("v", G * V)):
                sd[x + n] = mat(rows, W)
                sd[x + n + ".conv"] = vec((rows * m["conv"]), 0.5).view(rows, m["conv"])
            sd[x + "q.norm"], sd[x + "k.norm"] = vec(D, 0.2, 1.2), vec(D, 0.2, 1.2)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                sd[x + n] = vec(D, 0.3)
            sd[x + "o"] = mat(W, H * V)
        else:
            l, r, sh = m["left"], m["right"], layer["_shapes"]
            H, G, D = l["heads"], l["kv_heads"], l["dim"]
            y = x + "left."
            sd[y + "q"], sd[y + "k"] = mat(H * D, W), mat(G * D, W)
            sd[y + "q.norm"], sd[y + "k.norm"] = vec(H * D, 0.2, 1.0), vec(G * D, 0.2, 1.0)
            sd[y + "rel"] = vec(sh["buckets"] * H, 1.0).view(-1, H)
            sd[y + "talk"] = (torch.eye(H) + 0.3 * torch.randn(H, H, generator=g)).to(dtype)
            sd[y + "g"], sd[y + "o"] = mat(H * D, W), mat(W, H * D)
            H, G, D, V = r["heads"], r["kv_heads"], r["dim"], r["vdim"]
            y = x + "right."
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
                sd[y + n] = mat(rows, W)
                sd[y + n + ".conv"] = vec(rows * r["conv"], 0.5).view(rows, r["conv"])
            sd[y + "b"] = mat(H, W)
            sd[y + "A_log"] = (torch.rand(H, generator=g) * 2 - 2).to(dtype)
            sd[y + "dt_bias"] = (torch.rand(H * D, generator=g) * 2 - 2).to(dtype)
            sd[y + "norm"] = vec(V, 0.2, 1.0)
            sd[y + "a1"], sd[y + "a2"] = mat(sh["a_rank"], W), mat(H * D, sh["a_rank"])
            sd[y + "g1"], sd[y + "g2"] = mat(sh["g_rank"], W), mat(H * V, sh["g_rank"])
            sd[y + "o"] = mat(W, H * V)
            sd[x + "left.out"], sd[x + "right.out"] = vec(W, 0.2, 1.0), vec(W, 0.2, 1.0)
        if layer.get("mlp"):
            f, y = layer["mlp"]["ff"], p + "mlp."
            sd[p + "norm2"] = vec(W, 0.2, 1.0)
            sd[y + "gate"], sd[y + "up"], sd[y + "down"] = mat(f, W), mat(f, W), mat(W, f)
    return sd
