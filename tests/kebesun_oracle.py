"""Plain float64 implementation of the Kebesun design, written from its
equations: one function per mechanism, whole sequences, no caches, no
batching. Shares no code with ``kserve_amd``.

Notation: T tokens, positions 0..T-1; linear weights are [out, in].

  rms(x)     = x / sqrt(mean(x^2) + eps)
  turn       : coordinates i and i + n/2 of the first n of a head turn by
               p f_i, f_i = base^(-2i/n); "linear": f_i / factor; "yarn": f_i
               slowed by 1/factor along a ramp between the `fast` and `slow`
               turning numbers, cos and sin times 1 + ln(factor)/10
  attention  : q, k turned; key j is seen from i if j <= i and (i - j < size
               or j < keep_first); softmax(q.k scale) v
  latent     : q per head = [q_u | q_r]; D h = [c' | r']; c = rms(c') w,
               r = turn(r'); k_h = [U_k,h c | r], v_h = U_v,h c; causal softmax
               of ([q_u | turn(q_r)] . k_h) scale
  gla        : a = sigmoid(A_2 A_1 h + b)^(1/tau) per head and key channel;
               S <- diag(a) S + k v^T; o = S^T q dim^(-1/2);
               o -> rms per head times a weight times silu(G h)
  dense      : D (silu(G h) * U h)
  experts    : z = R h + b; the `top` largest; weights softmax of those z;
               sum of weight times expert
  layer      : h = rms(x) (1 + n); x <- x + s_1 mixer(h) + s_2 ff(h)
  loop       : layers start..stop-1 run `times` times; before each pass
               x <- L [x; embedding]
  model      : x = embed[tok]; layer runs; head rms(x) (1 + n)
"""

import math

import numpy as np
import torch


def _np(t):
    return t.detach().to(torch.float64).cpu().numpy()


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softmax(s):
    w = np.exp(s - s.max(axis=-1, keepdims=True))
    return w / w.sum(axis=-1, keepdims=True)


def frequencies(rot):
    """-> (turning speed of every pair, factor on cos and sin)."""
    n, base = rot["dims"], float(rot["base"])
    i = np.arange(n // 2, dtype=np.float64)
    f = base ** (-2.0 * i / n)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    if "original" not in sc:
        return f / sc["factor"], 1.0

    def where(turns):
        return n * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(where(sc["fast"])), 0)
    hi = min(math.ceil(where(sc["slow"])), n - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return (f / sc["factor"]) * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def turn(x, rot):
    """x [T, ..., dim]: coordinates i and i + n/2 of the first n turn."""
    if not rot or not rot.get("dims"):
        return x
    n = rot["dims"]
    f, m = frequencies(rot)
    pos = np.arange(x.shape[0], dtype=np.float64)
    ang = (pos[:, None] * f[None, :]).reshape(
        (x.shape[0],) + (1,) * (x.ndim - 2) + (n // 2,)
    )
    c, s = m * np.cos(ang), m * np.sin(ang)
    u, v = x[..., : n // 2], x[..., n // 2 : n]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., n:]], axis=-1)


def visible(T, mask):
    i = np.arange(T)[:, None]
    j = np.arange(T)[None, :]
    ok = j <= i
    if mask:
        ok &= (i - j < mask["size"]) | (j < mask.get("keep_first", 0))
    return ok


def attention(h, W, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = turn((h @ W[p + "q"].T).reshape(T, H, D), m.get("rot"))
    k = turn((h @ W[p + "k"].T).reshape(T, G, D), m.get("rot"))
    v = (h @ W[p + "v"].T).reshape(T, G, V)
    ok = visible(T, m.get("mask"))
    o = np.zeros((T, H, V))
    for a in range(H):
        g = a // (H // G)
        s = np.where(ok, (q[:, a] @ k[:, g].T) * m["scale"], -np.inf)
        o[:, a] = softmax(s) @ v[:, g]
    return o.reshape(T, H * V) @ W[p + "o"].T


def latent_attention(h, W, p, m, eps):
    T = h.shape[0]
    H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ W[p + "q"].T).reshape(T, H, D + R)
    qu, qr = q[..., :D], turn(q[..., D:], m["rot"])
    row = h @ W[p + "dkv"].T
    c = rms(row[:, :C], eps) * W[p + "dkv.norm"]
    kr = turn(row[:, C:], m["rot"])
    ku = (c @ W[p + "uk"].T).reshape(T, H, D)
    v = (c @ W[p + "uv"].T).reshape(T, H, V)
    ok = visible(T, None)
    o = np.zeros((T, H, V))
    for a in range(H):
        s = (qu[:, a] @ ku[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        o[:, a] = softmax(np.where(ok, s, -np.inf)) @ v[:, a]
    return o.reshape(T, H * V) @ W[p + "o"].T


def channel_decays(h, W, p, m):
    """[T, heads, dim]."""
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    return (sigmoid(z) ** (1.0 / m["tau"])).reshape(h.shape[0], m["heads"], m["dim"])


def gla_recurrence(q, k, v, a):
    """q, k, a [T, H, D], v [T, H, V] -> [T, H, V]."""
    T, H, D = q.shape
    o = np.zeros((T, H, v.shape[-1]))
    for b in range(H):
        S = np.zeros((D, v.shape[-1]))
        for t in range(T):
            S = a[t, b][:, None] * S + np.outer(k[t, b], v[t, b])
            o[t, b] = S.T @ q[t, b]
    return o


def gla(h, W, p, m, eps):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ W[p + "k"].T).reshape(T, H, D)
    v = (h @ W[p + "v"].T).reshape(T, H, V)
    o = gla_recurrence(q, k, v, channel_decays(h, W, p, m))
    o = (rms(o, eps) * W[p + "norm"]).reshape(T, H * V)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def gated(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def routing(z, top):
    """z [T, E] -> [T, E] weights, zero where an expert is not chosen."""
    w = np.zeros_like(z)
    for t in range(z.shape[0]):
        best = np.argsort(-z[t], kind="stable")[:top]
        w[t, best] = softmax(z[t, best])
    return w


def experts(h, W, p, m):
    w = routing(h @ W[p + "router"].T + W[p + "router.b"], m["router"]["top"])
    y = np.zeros_like(h)
    for e in range(m["router"]["experts"]):
        y += w[:, e : e + 1] * gated(h, W, p + f"e{e}.")
    return y


MIXERS = {"attention": attention, "latent_attention": latent_attention, "gla": gla}


def layer_delta(h, W, i, layer, eps):
    p = f"l{i}."
    d = MIXERS[layer["type"]](h, W, p + "mix.", layer["mixer"], eps) * W[p + "ls1"]
    m = layer.get("mlp")
    if m:
        y = experts(h, W, p + "mlp.", m) if m["kind"] == "moe" else gated(h, W, p + "mlp.")
        d = d + y * W[p + "ls2"]
    return d


def run_order(cfg):
    """[(layer index, first layer of a pass?)]."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    span = [(i, i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return (
        [(i, False) for i in range(lp["start"])] + span * lp["times"]
        + [(i, False) for i in range(lp["stop"], n)]
    )


def forward(cfg, sd, tokens, streams=None):
    """Logits [T, vocab] (float64 torch); ``streams`` collects the residual
    stream after every layer run."""
    W = {k: _np(v) for k, v in sd.items()}
    eps = cfg["norm"]["eps"]
    x0 = W["embed"][np.asarray(tokens)]
    x = x0
    for i, opens in run_order(cfg):
        if opens:
            x = np.concatenate([x, x0], axis=-1) @ W["loop.in"].T
        x = x + layer_delta(norm(x, W[f"l{i}.norm1"], eps), W, i, cfg["layers"][i], eps)
        if streams is not None:
            streams.append(torch.from_numpy(x.copy()))
    return torch.from_numpy(norm(x, W["final.norm"], eps) @ W["head"].T)


# -- builders -----------------------------------------------------------------

def dense(ff=24):
    return {"kind": "dense", "ff": ff}


def moe(n=5, top=2, ff=16):
    return {"kind": "moe", "router": {"experts": n, "top": top}, "expert": {"ff": ff}}


def linear_rot(dims=8, base=300.0, factor=2.0):
    return {"dims": dims, "base": base, "scaling": {"factor": factor}}


def yarn_rot(dims=8, base=500.0, factor=3.0, original=40, fast=4.0, slow=0.5):
    return {"dims": dims, "base": base,
            "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow}}


def attention_layer(heads=4, kv_heads=2, dim=12, vdim=20, scale=0.3, window=9, keep=3,
                    rot="default", mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
         "rot": linear_rot() if rot == "default" else rot}
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def latent_layer(heads=3, dim=12, rot_dim=8, vdim=20, kv_rank=28, scale=0.3, rot="default",
                 mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
                      "kv_rank": kv_rank, "scale": scale,
                      "rot": yarn_rot(rot_dim) if rot == "default" else rot}}


def gla_layer(heads=2, dim=12, vdim=20, tau=8.0, rank=5, mlp=None):
    """``rank`` shows only in tensor shapes."""
    return {"type": "gla", "mlp": mlp, "_rank": rank,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def make_config(layers, vocab=61, width=32, eps=1e-5, loop=None):
    cfg = {"architecture": "Kebesun", "vocab": vocab, "width": width,
           "norm": {"eps": eps}, "layers": layers}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def random_weights(cfg, seed=0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def mat(o, i, gain=1.0):
        return (torch.randn(o, i, generator=g) * gain * i ** -0.5).to(dtype)

    def vec(n, std, mean=0.0):
        return (mean + std * torch.randn(n, generator=g)).to(dtype)

    sd = {"embed": torch.randn(cfg["vocab"], W, generator=g).to(dtype),
          "final.norm": vec(W, 0.1), "head": mat(cfg["vocab"], W)}
    if cfg.get("loop"):
        sd["loop.in"] = mat(W, 2 * W)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        sd[p + "norm1"] = vec(W, 0.2)
        sd[p + "ls1"] = vec(W, 0.2, 0.7)
        x = p + "mix."
        if layer["type"] == "attention":
            H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            sd[x + "q"], sd[x + "k"] = mat(H * D, W, 1.5), mat(G * D, W, 1.5)
            sd[x + "v"], sd[x + "o"] = mat(G * V, W), mat(W, H * V)
        elif layer["type"] == "latent_attention":
            H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            sd[x + "q"], sd[x + "dkv"] = mat(H * (D + R), W, 1.5), mat(C + R, W)
            sd[x + "dkv.norm"] = vec(C, 0.2, 1.2)
            sd[x + "uk"], sd[x + "uv"] = mat(H * D, C), mat(H * V, C)
            sd[x + "o"] = mat(W, H * V)
        else:
            H, D, V, r = m["heads"], m["dim"], m["vdim"], layer["_rank"]
            sd[x + "q"], sd[x + "k"] = mat(H * D, W), mat(H * D, W)
            sd[x + "v"], sd[x + "g"] = mat(H * V, W), mat(H * V, W)
            sd[x + "a1"], sd[x + "a2"] = mat(r, W), mat(H * D, r)
            sd[x + "a2.b"] = vec(H * D, 1.0, 1.0)
            sd[x + "norm"], sd[x + "o"] = vec(V, 0.2, 1.0), mat(W, H * V)
        f = layer.get("mlp")
        if not f:
            continue
        sd[p + "ls2"] = vec(W, 0.2, 0.7)
        y = p + "mlp."
        if f["kind"] == "moe":
            E, n = f["router"]["experts"], f["expert"]["ff"]
            sd[y + "router"], sd[y + "router.b"] = mat(E, W), vec(E, 0.5)
            names = [f"e{e}." for e in range(E)]
        else:
            n, names = f["ff"], [""]
        for e in names:
            sd[y + e + "gate"], sd[y + e + "up"] = mat(n, W), mat(n, W)
            sd[y + e + "down"] = mat(W, n)
    return sd
