"""Plain, slow restatement of the mixer-stack models (architectures "Bipotar",
"Taredra", "Fedirax" and "Marosun"): one function per mechanism, numpy, one sequence at a time, every
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


def rotate_neighbours(x, positions, base, dims):
    """x [T, ..., >= dims]: dimension 2i turns with dimension 2i + 1."""
    freq = float(base) ** (-2.0 * np.arange(dims // 2) / dims)
    ang = np.asarray(positions, dtype=np.float64)[:, None] * freq[None]
    out = x.copy()
    for i in range(dims // 2):
        shape = (len(positions),) + (1,) * (x.ndim - 2)
        c, s = np.cos(ang[:, i]).reshape(shape).astype(x.dtype), np.sin(ang[:, i]).reshape(shape).astype(x.dtype)
        out[..., 2 * i] = x[..., 2 * i] * c - x[..., 2 * i + 1] * s
        out[..., 2 * i + 1] = x[..., 2 * i + 1] * c + x[..., 2 * i] * s
    return out


def in_window(pos, size):
    """[T, T]: row i sees its own position and the size - 1 before it."""
    gap = pos[:, None] - pos[None, :]
    return (gap >= 0) & (gap < size)


def soft_cap(score, cap):
    return score if not cap else cap * np.tanh(score / cap)


def keys_as_values_attention(h, w, cfg, eps, positions=None):
    """Grouped-query attention whose values are the projected keys ahead of their rotation: biases, capped scores, a sink
    per head, and each head's output times a logistic gate of its own."""
    H, G, D = cfg["heads"], cfg["kv_heads"], cfg["dim"]
    assert cfg["vdim"] == D
    T = h.shape[0]
    pos = np.arange(T) if positions is None else np.asarray(positions)
    rot = cfg["rot"]
    q = rotate_neighbours((h @ w["q"].T + w["q.b"]).reshape(T, H, D), pos, rot["base"], rot["dims"])
    v = (h @ w["k"].T + w["k.b"]).reshape(T, G, D)
    k = rotate_neighbours(v, pos, rot["base"], rot["dims"])
    seen = in_window(pos, cfg["mask"]["size"])
    out = np.empty((T, H, D), dtype=h.dtype)
    for hh in range(H):
        g = hh // (H // G)
        s = np.where(seen, soft_cap((q[:, hh] @ k[:, g].T) * h.dtype.type(cfg["scale"]), cfg.get("softcap")), -np.inf)
        top = np.maximum(s.max(axis=1, keepdims=True), w["sink"][hh])
        e = np.exp(s - top)
        out[:, hh] = (e / (e.sum(axis=1, keepdims=True) + np.exp(w["sink"][hh] - top))) @ v[:, g]
    out = out * sigmoid(h @ w["g"].T)[:, :, None]
    return out.reshape(T, H * D) @ w["o"].T


def differential_weight(w, diff):
    """How much of the second map's output is taken off the first's."""
    return np.exp((w["lq1"] * w["lk1"]).sum()) - np.exp((w["lq2"] * w["lk2"]).sum()) + w["lq1"].dtype.type(diff)


def differential_keys(h, w, cfg, eps, pos):
    """Keys [T, G, 2, dim] as a cache holds them, and values [T, G, vdim]."""
    G, D, V, T = cfg["kv_heads"], cfg["dim"], cfg["vdim"], h.shape[0]
    k = rms_norm((h @ w["k"].T).reshape(T, G, 2, D), w["k.norm"], eps)
    return rotate_neighbours(k, pos, cfg["rot"]["base"], cfg["rot"]["dims"]), (h @ w["v"].T).reshape(T, G, V)


def differential_attention(h, w, cfg, eps, kv=None, positions=None):
    """Two softmax maps per head over the same values, the second taken off the first, the difference over its root
    mean square.  `kv`: another layer's keys and values; returns (out [T, width], the keys and values used)."""
    H, G, D, V = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    pos = np.arange(T) if positions is None else np.asarray(positions)
    q = rms_norm((h @ w["q"].T).reshape(T, H, 2, D), w["q.norm"], eps)
    q = rotate_neighbours(q, pos, cfg["rot"]["base"], cfg["rot"]["dims"])
    k, v = differential_keys(h, w, cfg, eps, pos) if kv is None else kv
    seen = in_window(pos, cfg["mask"]["size"])
    lam, keep = differential_weight(w, cfg["diff"]), h.dtype.type(1.0 - cfg["diff"])
    out = np.empty((T, H, V), dtype=h.dtype)
    for hh in range(H):
        g = hh // (H // G)
        maps = []
        for m in range(2):
            s = np.where(seen, (q[:, hh, m] @ k[:, g, m].T) * h.dtype.type(cfg["scale"]), -np.inf)
            e = np.exp(s - s.max(axis=1, keepdims=True))
            maps.append((e / e.sum(axis=1, keepdims=True)) @ v[:, g])
        out[:, hh] = unit_rms(maps[0] - lam * maps[1], eps) * keep
    return out.reshape(T, H * V) @ w["o"].T, (k, v)


def clamped_expert(h, w, limit):
    """One feed-forward part of clamped gated units; h is one row or several."""
    g = np.minimum(h @ w["gate"].T, h.dtype.type(limit))
    u = np.clip(h @ w["up"].T, -h.dtype.type(limit), h.dtype.type(limit))
    return (g * sigmoid(h.dtype.type(1.702) * g) * (u + 1)) @ w["down"].T


def grouped_choice(z, correction, top, groups):
    """One token's logits: the chosen outputs (by corrected score, best groups only) and the uncorrected scores of all."""
    e = np.exp(z - z.max())
    s = e / e.sum()
    c = s + correction
    if groups:
        by_group = c.reshape(groups["count"], -1)
        best = np.argsort(-by_group.max(axis=1), kind="stable")[:groups["keep"]]
        allowed = np.isin(np.arange(len(z)) // by_group.shape[1], best)
        c = np.where(allowed, c, -np.inf)
    return np.argsort(-c, kind="stable")[:top], s


def grouped_moe(h, w, cfg):
    """Experts and outputs that pass the input on, chosen inside the best groups; a gated shared expert beside them."""
    r, n = cfg["router"], cfg["router"]["experts"]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, s = grouped_choice(w["router"] @ h[t], w["correction"], r["top"], r.get("groups"))
        weight = s[chosen] / (s[chosen].sum() + 1e-20) * h.dtype.type(r["scale"])
        for g, e in zip(weight, chosen):
            out[t] += g * (clamped_expert(h[t], _sub(w, f"e{e}."), cfg["expert"]["limit"]) if e < n else h[t])
    if cfg.get("shared"):
        out = out + sigmoid(h @ w["shared.sg"].T) * clamped_expert(h, _sub(w, "shared."), cfg["shared"]["limit"])
    return out


def grouped_margin(h, w, cfg):
    """How little would change a token's choice: the gap between the last group kept and the first left out, and
    between the last output chosen and the first not, over the scores' spread."""
    r, out = cfg["router"], np.full(h.shape[0], np.inf)
    for t in range(h.shape[0]):
        z = w["router"] @ h[t]
        chosen, s = grouped_choice(z, w["correction"], r["top"], r.get("groups"))
        c, g = s + w["correction"], r.get("groups")
        if g:
            best = c.reshape(g["count"], -1).max(axis=1)
            if g["keep"] < g["count"]:
                order = np.sort(best)[::-1]
                out[t] = min(out[t], (order[g["keep"] - 1] - order[g["keep"]]) / s.std())
            kept = np.argsort(-best, kind="stable")[:g["keep"]]
            c = c[np.isin(np.arange(len(z)) // (len(z) // g["count"]), kept)]
        c = np.sort(c)[::-1]
        if r["top"] < len(c):
            out[t] = min(out[t], (c[r["top"] - 1] - c[r["top"]]) / s.std())
    return out


def shared_kv_layer(x, w, cfg, eps, kvs, margins=None):
    """A pre-norm layer of differential or keys-as-values attention with an expert feed-forward.  `kvs`: the keys and
    values of the layers so far, which receives this layer's."""
    m, h = cfg["mixer"], rms_norm(x, 1 + w["norm1"], eps)
    if cfg["type"] == "attention_2":
        j = m.get("kv_from")
        y, kv = differential_attention(h, _sub(w, "mix."), m, eps, None if j is None else kvs[j])
    else:
        y, kv = keys_as_values_attention(h, _sub(w, "mix."), m, eps), None
    kvs.append(kv)
    x = x + y
    if cfg.get("mlp"):
        h = rms_norm(x, 1 + w["norm2"], eps)
        if margins is not None:
            margins.append(grouped_margin(h, _sub(w, "mlp."), cfg["mlp"]))
        x = x + grouped_moe(h, _sub(w, "mlp."), cfg["mlp"])
    return x


def rotation(rot):
    """(frequencies, factor of cosine and sine) of a rotation, the far pairs slowed down where it is scaled: a pair that
    turns more than `fast` times over the original length keeps its frequency, one that turns less than `slow` times has
    it divided by the factor, with a ramp over the pairs between."""
    dims, base, sc = rot["dims"], float(rot["base"]), rot.get("scaling")
    f = base ** (-2.0 * np.arange(dims // 2) / dims)
    if not sc:
        return f, 1.0
    pair = lambda turns: dims * np.log(sc["original"] / (2 * np.pi * turns)) / (2 * np.log(base))
    lo, hi = max(np.floor(pair(sc["fast"])), 0), min(np.ceil(pair(sc["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0, 1)
    return f / sc["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(sc["factor"]) + 1


def turn_neighbours(x, positions, freq, gain=1.0):
    """x [T, heads, >= 2 len(freq)]: dimension 2i turns with dimension 2i + 1 by position * freq[i]."""
    out, n = x.copy(), len(freq)
    ang = np.asarray(positions, dtype=np.float64)[:, None, None] * freq
    c, s = (np.cos(ang) * gain).astype(x.dtype), (np.sin(ang) * gain).astype(x.dtype)
    u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
    out[..., 0:2 * n:2], out[..., 1:2 * n:2] = u * c - v * s, v * c + u * s
    return out


def in_chunk(pos, size):
    """[T, T]: row i sees what came before it in its own chunk of positions, itself included."""
    return (pos[:, None] >= pos[None, :]) & (pos[:, None] // size == pos[None, :] // size)


def sunk_weights(score, sink):
    """Softmax of the rows of `score` (-inf: unseen) with exp(sink) added to the denominator."""
    top = np.maximum(score.max(axis=1, keepdims=True), sink)
    e = np.exp(score - top)
    return e / (e.sum(axis=1, keepdims=True) + np.exp(sink - top))


def sink_heads(q, k, v, scale, seen, sink):
    """Every head's weighted values [T, H, vdim]; heads share the key/value heads in equal runs."""
    H, G = q.shape[1], k.shape[1]
    out = np.empty((q.shape[0], H, v.shape[-1]), dtype=q.dtype)
    for hh in range(H):
        g = hh // (H // G)
        score = np.where(seen, (q[:, hh] @ k[:, g].T) * q.dtype.type(scale), -np.inf)
        out[:, hh] = sunk_weights(score, sink[hh]) @ v[:, g]
    return out


def biased(h, w, name):
    return h @ w[name].T + w[name + ".b"]


def normed_turned(h, w, cfg, eps, pos):
    """Queries and keys with biases, normed head by head and rotated; values with biases."""
    H, G, D, V, T = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"], h.shape[0]
    turn = rotation(cfg["rot"])
    q = turn_neighbours(rms_norm(biased(h, w, "q").reshape(T, H, D), w["q.norm"], eps), pos, *turn)
    k = turn_neighbours(rms_norm(biased(h, w, "k").reshape(T, G, D), w["k.norm"], eps), pos, *turn)
    return q, k, biased(h, w, "v").reshape(T, G, V)


def turned_values_attention(h, w, cfg, eps, positions=None):
    """Causal attention whose values are rotated by their position and whose outputs are turned back by the row's."""
    pos = np.arange(h.shape[0]) if positions is None else np.asarray(positions)
    q, k, v = normed_turned(h, w, cfg, eps, pos)
    freq, _ = rotation({"base": cfg["rot"]["base"], "dims": cfg["vdim"]})
    o = sink_heads(q, k, turn_neighbours(v, pos, freq), cfg["scale"], pos[:, None] >= pos[None, :], w["sink"])
    return biased(turn_neighbours(o, -pos, freq).reshape(len(h), -1), w, "o")


def one_more_attention(h, w, cfg, eps, positions=None):
    """Causal attention with one added to the softmax's denominator."""
    pos = np.arange(h.shape[0]) if positions is None else np.asarray(positions)
    q, k, v = normed_turned(h, w, cfg, eps, pos)
    o = sink_heads(q, k, v, cfg["scale"], pos[:, None] >= pos[None, :], np.zeros(cfg["heads"], dtype=h.dtype))
    return biased(o.reshape(len(h), -1), w, "o")


def chunked_attention(h, w, cfg, eps, positions=None):
    """Attention inside chunks of positions, without rotation, every output element with a logistic gate."""
    pos, T = np.arange(h.shape[0]) if positions is None else np.asarray(positions), len(h)
    q, k, v = ((h @ w[n].T).reshape(T, c, d) for n, c, d in (("q", cfg["heads"], cfg["dim"]), ("k", cfg["kv_heads"], cfg["dim"]),
                                                            ("v", cfg["kv_heads"], cfg["vdim"])))
    o = sink_heads(q, k, v, cfg["scale"], in_chunk(pos, cfg["mask"]["size"]), w["sink"])
    return (o.reshape(T, -1) * sigmoid(h @ w["g"].T)) @ w["o"].T


def forget_gate_recurrence(h, w, cfg, eps):
    """Linear attention whose keys are what the forget gate lets go; returns (out [T, width], final state [heads, dim, vdim])."""
    H, D, V, T = cfg["heads"], cfg["dim"], cfg["vdim"], h.shape[0]
    q, v = silu(h @ w["q"].T).reshape(T, H, D), (h @ w["v"].T).reshape(T, H, V)
    low = w["lower"]
    f = (low + (1 - low) * sigmoid(h @ w["f"].T + w["f.b"])).reshape(T, H, D)
    S = np.zeros((H, D, V), dtype=h.dtype)
    o = np.empty((T, H, V), dtype=h.dtype)
    for t in range(T):
        S = f[t][:, :, None] * S + (1 - f[t])[:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return rms_norm(o, w["norm"], eps).reshape(T, H * V) @ w["o"].T, S


def min_gru(h, w, cfg, eps):
    """A gated recurrence element by element; returns (out [T, width], final state [size])."""
    z, u = sigmoid(biased(h, w, "z")), biased(h, w, "x")
    candidate = np.where(u >= 0, u + h.dtype.type(0.5), sigmoid(u))
    S = np.zeros(cfg["width"], dtype=h.dtype)
    states = np.empty_like(z)
    for t in range(len(h)):
        S = (1 - z[t]) * S + z[t] * candidate[t]
        states[t] = S
    return (states * silu(h @ w["g"].T)) @ w["o"].T, S


def chunked_beside_forget_gate(h, w, cfg, eps):
    left = chunked_attention(h, _sub(w, "left."), cfg["left"], eps)
    right, _ = forget_gate_recurrence(h, _sub(w, "right."), cfg["right"], eps)
    return h.dtype.type(cfg["left_scale"]) * left + h.dtype.type(cfg["right_scale"]) * right


def one_more_beside_gru(h, w, cfg, eps):
    left = one_more_attention(h, _sub(w, "left."), cfg["left"], eps)
    right, _ = min_gru(h, _sub(w, "right."), cfg["right"], eps)
    return (rms_norm(left, w["left.out"], eps) + rms_norm(right, w["right.out"], eps)) / 2


def logistic_choice(z, top):
    """One token's logits: the chosen experts and their scores."""
    s = sigmoid(z)
    chosen = np.argsort(-s, kind="stable")[:top]
    return chosen, s[chosen]


def weighted_input_moe(h, w, cfg):
    """Gated experts whose input, not output, is multiplied by the weight."""
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(*logistic_choice(w["router"] @ h[t], cfg["router"]["top"])):
            out[t] += dense_mlp(s * h[t], _sub(w, f"e{e}."))
    return out


SIDE_MIXERS = {"attention": turned_values_attention, "parallel": chunked_beside_forget_gate, "parallel_2": one_more_beside_gru}


def side_by_side_layer(x, w, cfg, eps, margins=None):
    """A layer whose mixer and feed-forward read the same norm and join the residual together."""
    h, f = rms_norm(x, 1 + w["norm1"], eps), cfg.get("mlp")
    y = SIDE_MIXERS[cfg["type"]](h, _sub(w, "mix."), cfg["mixer"], eps)
    if f and f["kind"] == "dense":
        y = y + clamped_expert(h, _sub(w, "mlp."), f["limit"])
    elif f:
        y = y + weighted_input_moe(h, _sub(w, "mlp."), f)
        if margins is not None:
            margins.append(router_margin(h, _sub(w, "mlp."), f))
    return x + y


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
    if cfg["architecture"] == "Marosun":
        x = w["embed"][np.asarray(tokens)]
        for i, c in enumerate(cfg["layers"]):
            x = side_by_side_layer(x, _sub(w, f"l{i}."), c, eps, margins)
            if capture is not None:
                capture.append(x.copy())
        return rms_norm(x, 1 + w["final.norm"], eps) @ w["head"].T
    if cfg["architecture"] == "Fedirax":
        x, kvs = w["embed"][np.asarray(tokens)] * prec(cfg["embedding"]["scale"]), []
        for i, c in enumerate(cfg["layers"]):
            x = shared_kv_layer(x, _sub(w, f"l{i}."), c, eps, kvs, margins)
            if capture is not None:
                capture.append(x.copy())
        return rms_norm(x, 1 + w["final.norm"], eps) @ w["head"].T
    x = rms_norm(w["embed"][np.asarray(tokens)], w["embed.norm"], eps)
    x0 = x
    for i, again in layer_order(cfg):
        if again:
            x = x + x0
        x = layer(x, _sub(w, f"l{i}."), cfg["layers"][i], eps, margins)
        if capture is not None:
            capture.append(x.copy())
    return (rms_norm(x, w["final.norm"], eps) @ w["head"].T) * prec(cfg["logit_scale"])
