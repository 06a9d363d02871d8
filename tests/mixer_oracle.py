"""Plain, slow restatement of the mixer-stack models (architectures "Bipotar" and
"Taredra"): one function per mechanism, numpy, one sequence at a time, every
position from the definition (no cache, no chunks, no absorbed products).  Shares
no code with the product path; the tests compare the engine with it.

``prec`` is the working dtype of every sum (float32 or float64).
"""
from __future__ import annotations

import numpy as np


def bf16_to_f32(bits: np.ndarray) -> np.ndarray:
    return (bits.astype(np.uint32) << 16).view(np.float32)


def f32_to_bf16(x: np.ndarray) -> np.ndarray:
    """Round to nearest even; finite inputs."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    return ((u + np.uint32(0x7FFF) + ((u >> np.uint32(16)) & np.uint32(1))) >> np.uint32(16)).astype(np.uint16)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + x.dtype.type(eps)) * w


def rotate_half_pairs(x, positions, base, dims):
    """x [T, ..., >= dims]: dimension i turns with dimension i + dims/2."""
    half = dims // 2
    freq = float(base) ** (-2.0 * np.arange(half) / dims)
    ang = np.asarray(positions, dtype=np.float64)[:, None] * freq[None]
    shape = (len(positions),) + (1,) * (x.ndim - 2) + (half,)
    c, s = np.cos(ang).reshape(shape).astype(x.dtype), np.sin(ang).reshape(shape).astype(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


def lightning(h, w, cfg, eps, state=None):
    """Decayed linear attention; returns (out [T, width], final state [heads, dim, vdim])."""
    H, D, V = cfg["heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    q = silu(h @ w["q"].T).reshape(T, H, D)
    k = silu(h @ w["k"].T).reshape(T, H, D)
    v = silu(h @ w["v"].T).reshape(T, H, V)
    decay = np.asarray(cfg["decay"], dtype=h.dtype)[:, None, None]
    S = np.zeros((H, D, V), dtype=h.dtype) if state is None else state.copy()
    o = np.empty((T, H, V), dtype=h.dtype)
    for t in range(T):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    o = rms_norm(o.reshape(T, H * V), w["norm"], eps) * sigmoid(h @ w["g"].T)
    return o @ w["o"].T, S


def latent_attention(h, w, cfg, eps, positions=None):
    """Attention through a low-rank latent with a shared rotated key part and a sliding window."""
    H, D, V = cfg["heads"], cfg["dim"], cfg["vdim"]
    rank, rd, rot = cfg["kv_rank"], cfg["rot_dim"], cfg["rot"]
    T = h.shape[0]
    pos = np.arange(T) if positions is None else np.asarray(positions)
    cq = rms_norm(h @ w["dq"].T, w["dq.norm"], eps)
    q = (cq @ w["uq"].T).reshape(T, H, D + rd)
    qu, qr = q[..., :D], rotate_half_pairs(q[..., D:], pos, rot["base"], rot["dims"])
    dkv = h @ w["dkv"].T
    c = rms_norm(dkv[:, :rank], w["dkv.norm"], eps)
    kr = rotate_half_pairs(dkv[:, rank:], pos, rot["base"], rot["dims"])
    k = (c @ w["uk"].T).reshape(T, H, D)
    v = (c @ w["uv"].T).reshape(T, H, V)
    gap = pos[:, None] - pos[None, :]
    seen = (gap >= 0) & (gap < cfg["mask"]["size"])
    out = np.empty((T, H, V), dtype=h.dtype)
    for hh in range(H):
        s = (qu[:, hh] @ k[:, hh].T + qr[:, hh] @ kr.T) * h.dtype.type(cfg["scale"])
        s = np.where(seen, s, -np.inf)
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, hh] = (e / e.sum(axis=1, keepdims=True)) @ v[:, hh]
    return out.reshape(T, H * V) @ w["o"].T


def dense_mlp(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def router_margin(h, w, cfg):
    """How far the last chosen logit lies above the first one left out, per token, in units of the logits' spread."""
    z = np.sort(h @ w["router"].T, axis=-1)
    top = cfg["router"]["top"]
    if top == z.shape[-1]:
        return np.full(len(z), np.inf)
    return (z[:, -top] - z[:, -top - 1]) / z.std()


def moe_mlp(h, w, cfg):
    top, n_exp = cfg["router"]["top"], cfg["router"]["experts"]
    z = h @ w["router"].T
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        chosen = np.argsort(-z[t], kind="stable")[:top]
        e = np.exp(z[t][chosen] - z[t][chosen].max())
        g = e / e.sum()
        for gi, ei in zip(g, chosen):
            assert ei < n_exp
            a = np.maximum(w[f"e{ei}.up"] @ h[t], 0)
            out[t] += gi * (w[f"e{ei}.down"] @ (a * a))
    return out


def _sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + x.dtype.type(eps))


def token_shift(h, mu, before=None):
    """Every row moved towards the row before it (zeros, or `before`, ahead of the first)."""
    prev = np.concatenate([np.zeros_like(h[:1]) if before is None else before[None], h[:-1]])
    return h + (prev - h) * mu


def wkv(h, w, cfg, eps):
    """Matrix-state recurrence with a decay per head and key channel made from the input, and a bonus for the
    current token; returns (out [T, width], final state [heads, dim, dim])."""
    H, D = cfg["heads"], cfg["dim"]
    T = h.shape[0]
    mix = {s: token_shift(h, w["mu." + s]) for s in "rkvgw"}
    r, k, v = ((mix[s] @ w[s].T).reshape(T, H, D) for s in "rkv")
    decay = np.exp(-np.exp(np.tanh(mix["w"] @ w["w1"].T) @ w["w2"].T + w["w0"])).reshape(T, H, D)
    S = np.zeros((H, D, D), dtype=h.dtype)
    o = np.empty((T, H, D), dtype=h.dtype)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S + w["u"][:, :, None] * kv, r[t])
        S = decay[t][:, :, None] * S + kv
    o = unit_rms(o, eps).reshape(T, H * D) * w["norm"] * silu(mix["g"] @ w["g"].T)
    return o @ w["o"].T, S


def delta_rule(h, w, cfg, eps):
    """Matrix-state recurrence that decays per key channel, removes along the unit key and adds k v^T; returns
    (out [T, width], final state [heads, dim, dim])."""
    H, D = cfg["heads"], cfg["dim"]
    T = h.shape[0]
    r, k, v = ((h @ w[s].T).reshape(T, H, D) for s in "rkv")
    decay = np.exp(-np.exp(-0.5) * sigmoid(np.tanh(h @ w["w1"].T) @ w["w2"].T + w["w0"])).reshape(T, H, D)
    rate = sigmoid(h @ w["a"].T + w["a.b"]).reshape(T, H, D)
    u = k / np.sqrt((k * k).sum(-1, keepdims=True) + h.dtype.type(1e-6))
    S = np.zeros((H, D, D), dtype=h.dtype)
    o = np.empty((T, H, D), dtype=h.dtype)
    for t in range(T):
        seen = np.einsum("hd,hdv->hv", u[t], S)
        S = (decay[t][:, :, None] * S - (rate[t] * u[t])[:, :, None] * seen[:, None, :]
             + k[t][:, :, None] * v[t][:, None, :])
        o[t] = np.einsum("hdv,hd->hv", S, r[t])
    o = unit_rms(o, eps).reshape(T, H * D) * w["norm"] * sigmoid(h @ w["g"].T)
    return o @ w["o"].T, S


def window_attention(h, w, cfg, eps, positions=None):
    """Grouped-query attention in a sliding window: rotated queries and keys, normed values, a sink in the softmax."""
    H, G, D, V, rot = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"], cfg["rot"]
    T = h.shape[0]
    pos = np.arange(T) if positions is None else np.asarray(positions)
    q = rotate_half_pairs((h @ w["q"].T).reshape(T, H, D), pos, rot["base"], rot["dims"])
    k = rotate_half_pairs((h @ w["k"].T).reshape(T, G, D), pos, rot["base"], rot["dims"])
    v = unit_rms((h @ w["v"].T).reshape(T, G, V), eps)
    gap = pos[:, None] - pos[None, :]
    seen = (gap >= 0) & (gap < cfg["mask"]["size"])
    out = np.empty((T, H, V), dtype=h.dtype)
    for hh in range(H):
        g = hh // (H // G)
        s = np.where(seen, (q[:, hh] @ k[:, g].T) * h.dtype.type(cfg["scale"]), -np.inf)
        top = np.maximum(s.max(axis=1, keepdims=True), w["sink"][hh])
        e = np.exp(s - top)
        out[:, hh] = (e / (e.sum(axis=1, keepdims=True) + np.exp(w["sink"][hh] - top))) @ v[:, g]
    return out.reshape(T, H * V) @ w["o"].T


def parallel(h, w, cfg, eps):
    left = window_attention(h, _sub(w, "left."), cfg["left"], eps)
    right, _ = delta_rule(h, _sub(w, "right."), cfg["right"], eps)
    return h.dtype.type(cfg["left_scale"]) * left + h.dtype.type(cfg["right_scale"]) * right


def gelu_mlp(h, w):
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


MIXERS = {"lightning": lambda *a: lightning(*a)[0], "latent_attention": latent_attention,
          "wkv": lambda *a: wkv(*a)[0], "parallel": parallel}


def prenorm_layer(x, w, cfg, eps):
    """A layer with a norm ahead of each sublayer only; stored w means the factor 1 + w."""
    x = x + MIXERS[cfg["type"]](rms_norm(x, 1 + w["norm1"], eps), _sub(w, "mix."), cfg["mixer"], eps)
    if cfg.get("mlp"):
        x = x + gelu_mlp(rms_norm(x, 1 + w["norm2"], eps), _sub(w, "mlp."))
    return x


def layer(x, w, cfg, eps, margins=None):
    """One layer on the residual rows x [T, width]; w holds the layer's tensors without 'l<i>.'.
    `margins`: a list that receives router_margin of an expert layer."""
    h = rms_norm(x, w["norm1"], eps)
    x = x + rms_norm(MIXERS[cfg["type"]](h, _sub(w, "mix."), cfg["mixer"], eps), w["norm1b"], eps)
    mlp = cfg.get("mlp")
    if mlp:
        h = rms_norm(x, w["norm2"], eps)
        if margins is not None and mlp["kind"] == "moe":
            margins.append(router_margin(h, _sub(w, "mlp."), mlp))
        y = dense_mlp(h, _sub(w, "mlp.")) if mlp["kind"] == "dense" else moe_mlp(h, _sub(w, "mlp."), mlp)
        x = x + rms_norm(y, w["norm2b"], eps)
    return x


def layer_order(cfg):
    """[(layer, add the embedding output first?)] in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    return ([(i, False) for i in range(a)] + [(i, p > 0 and i == a) for p in range(times) for i in range(a, b)] +
            [(i, False) for i in range(b, n)])


def forward(cfg, tensors, tokens, prec=np.float32, capture=None, margins=None):
    """Logits [T, vocab] of one sequence.  `capture`: a list that receives the rows after every layer run."""
    w = {k: (v if v.dtype == np.int32 else v.astype(prec)) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    if cfg["architecture"] == "Taredra":
        x = w["embed"][np.asarray(tokens)] * prec(cfg["embedding"]["scale"])
        for i, c in enumerate(cfg["layers"]):
            x = prenorm_layer(x, _sub(w, f"l{i}."), c, eps)
            if capture is not None:
                capture.append(x.copy())
        return rms_norm(x, 1 + w["final.norm"], eps) @ w["embed"].T
    x = rms_norm(w["embed"][np.asarray(tokens)], w["embed.norm"], eps)
    x0 = x
    for i, again in layer_order(cfg):
        if again:
            x = x + x0
        x = layer(x, _sub(w, f"l{i}."), cfg["layers"][i], eps, margins)
        if capture is not None:
            capture.append(x.copy())
    return (rms_norm(x, w["final.norm"], eps) @ w["head"].T) * prec(cfg["logit_scale"])
