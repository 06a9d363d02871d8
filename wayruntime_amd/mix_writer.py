"""Writes mixer-stack models (architectures "Bipotar", "Taredra", "Fedirax" and "Marosun") as a
folder with config.json and model.safetensors: random-init models for the tests and the benchmark,
and any set of bfloat16 tensors a caller has."""
from __future__ import annotations

import json
import os
import struct

import numpy as np


def lightning(heads: int, dim: int, vdim: int, decay=None) -> dict:
    if decay is None:
        decay = np.exp(-np.exp2(-np.linspace(1.0, 8.0, heads))).tolist()
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": [float(d) for d in decay]}}


def latent_attention(heads: int, dim: int, vdim: int, q_rank: int, kv_rank: int, rot_dim: int, window: int,
                     base: float = 10000.0, scale: float | None = None) -> dict:
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "rot_dim": rot_dim,
                      "rot": {"base": base, "dims": rot_dim}, "mask": {"size": window},
                      "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}}


def wkv(heads: int, dim: int) -> dict:
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}}


def window_and_delta(heads: int, kv_heads: int, dim: int, vdim: int, window: int, right_heads: int, right_dim: int,
                     rot_dims: int | None = None, base: float = 10000.0, scale: float | None = None,
                     left_scale: float = 1.0, right_scale: float = 1.0) -> dict:
    """Windowed grouped-query attention and a delta-rule recurrence side by side."""
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
            "rot": {"base": base, "dims": dim if rot_dims is None else rot_dims}, "scale": dim ** -0.5 if scale is None else scale}
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": right_heads, "dim": right_dim},
                                          "left_scale": left_scale, "right_scale": right_scale}}


def keys_as_values(heads: int, kv_heads: int, dim: int, window: int, rot_dims: int | None = None, base: float = 10000.0,
                   scale: float | None = None, softcap: float | None = 30.0) -> dict:
    """Grouped-query attention whose values are the keys ahead of their rotation."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": window},
         "rot": {"base": base, "dims": dim if rot_dims is None else rot_dims}, "scale": dim ** -0.5 if scale is None else scale}
    return {"type": "attention", "mixer": m if softcap is None else dict(m, softcap=softcap)}


def difference(heads: int, kv_heads: int, dim: int, vdim: int, window: int, rot_dims: int | None = None, base: float = 10000.0,
               scale: float | None = None, diff: float = 0.5, kv_from: int | None = None) -> dict:
    """Attention of two maps per head, the second taken off the first."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "diff": diff,
         "rot": {"base": base, "dims": dim if rot_dims is None else rot_dims}, "scale": dim ** -0.5 if scale is None else scale}
    return {"type": "attention_2", "mixer": m if kv_from is None else dict(m, kv_from=kv_from)}


def _heads(heads: int, kv_heads: int, dim: int, vdim: int, scale: float | None) -> dict:
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale}


def turned_values(heads: int, kv_heads: int, dim: int, vdim: int, rot_dims: int | None = None, base: float = 10000.0,
                  scale: float | None = None, scaling=(4.0, 4096, 32.0, 1.0)) -> dict:
    """Causal attention with normed queries and keys whose values turn with their positions; scaling: (factor, original
    length, fast, slow) of the rotation's far pairs, or None."""
    rot = {"base": base, "dims": dim if rot_dims is None else rot_dims}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "attention", "mixer": dict(_heads(heads, kv_heads, dim, vdim, scale), rot=rot)}


def chunks_and_forget(heads: int, kv_heads: int, dim: int, vdim: int, chunk: int, right_heads: int, right_dim: int,
                      right_vdim: int, scale: float | None = None, left_scale: float = 1.0, right_scale: float = 1.0) -> dict:
    """Attention inside chunks of positions and a recurrence whose forget gate makes the keys, side by side."""
    return {"type": "parallel", "mixer": {"left": dict(_heads(heads, kv_heads, dim, vdim, scale), mask={"size": chunk}),
                                          "right": {"heads": right_heads, "dim": right_dim, "vdim": right_vdim},
                                          "left_scale": left_scale, "right_scale": right_scale}}


def one_more_and_gru(heads: int, kv_heads: int, dim: int, vdim: int, size: int, rot_dims: int | None = None,
                     base: float = 10000.0, scale: float | None = None) -> dict:
    """Causal attention with one added to the softmax's denominator and a gated recurrence of `size` elements, averaged."""
    rot = {"base": base, "dims": dim if rot_dims is None else rot_dims}
    return {"type": "parallel_2", "mixer": {"left": dict(_heads(heads, kv_heads, dim, vdim, scale), rot=rot),
                                            "right": {"width": size}}}


def clamped_dense(ff: int, limit: float = 7.0) -> dict:
    return {"kind": "dense", "ff": ff, "limit": limit}


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def moe(experts: int, top: int, ff: int) -> dict:
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def grouped_moe(experts: int, top: int, ff: int, identity: int = 0, groups=None, scale: float = 1.0, limit: float = 7.0,
                shared=None) -> dict:
    """groups: (count, keep) or None; shared: (ff, limit) of a shared expert, or None."""
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "identity": identity, "top": top, "scale": scale,
                       "groups": None if groups is None else dict(zip(("count", "keep"), groups))},
            "shared": None if shared is None else dict(zip(("ff", "limit"), shared))}


def config(width: int, vocab: int, layers, loop=None, eps: float = 1e-6, logit_scale: float = 1.0) -> dict:
    """layers: [(mixer, feed-forward or None)]; loop: (start, stop, times) or None."""
    return {"architecture": "Bipotar", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop)),
            "layers": [dict(m, mlp=f) for m, f in layers]}


def prenorm_config(width: int, vocab: int, layers, eps: float = 1e-6, embed_scale: float | None = None) -> dict:
    """layers: [(mixer, feed-forward or None)] of wkv and window_and_delta mixers."""
    return {"architecture": "Taredra", "width": width, "vocab": vocab, "norm": {"eps": eps},
            "embedding": {"scale": width ** 0.5 if embed_scale is None else embed_scale},
            "layers": [dict(m, mlp=f) for m, f in layers]}


def shared_kv_config(width: int, vocab: int, layers, eps: float = 1e-6, embed_scale: float = 1.0) -> dict:
    """layers: [(mixer, feed-forward or None)] of keys_as_values and difference mixers."""
    return dict(prenorm_config(width, vocab, layers, eps, embed_scale), architecture="Fedirax")


def joint_config(width: int, vocab: int, layers, eps: float = 1e-6) -> dict:
    """layers: [(mixer, feed-forward or None)] of turned_values, chunks_and_forget and one_more_and_gru mixers with
    clamped_dense or moe feed-forwards; both read one norm."""
    return {"architecture": "Marosun", "width": width, "vocab": vocab, "norm": {"eps": eps},
            "layers": [dict(m, mlp=f) for m, f in layers]}


def _joint_shapes(cfg: dict) -> dict:
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}

    def heads(p, m, biases):
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n, rows, cols in (("q", H * D, W), ("k", G * D, W), ("v", G * V, W), ("o", W, H * V)):
            out[p + n] = (rows, cols)
            if biases:
                out[p + n + ".b"] = (rows,)
        if biases:
            out.update({p + "q.norm": (D,), p + "k.norm": (D,)})
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        out[p + "norm1"] = (W,)
        q = p + "mix."
        if layer["type"] == "attention":
            heads(q, m, True)
            out[q + "sink"] = (m["heads"],)
        elif layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            heads(q + "left.", a, False)
            out.update({q + "left.sink": (a["heads"],), q + "left.g": (a["heads"] * a["vdim"], W)})
            hd, hv = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            out.update({q + "right.q": (hd, W), q + "right.v": (hv, W), q + "right.f": (hd, W), q + "right.f.b": (hd,),
                        q + "right.lower": (hd,), q + "right.norm": (r["vdim"],), q + "right.o": (W, hv)})
        else:
            heads(q + "left.", m["left"], True)
            n = m["right"]["width"]
            out.update({q + "right.z": (n, W), q + "right.z.b": (n,), q + "right.x": (n, W), q + "right.x.b": (n,),
                        q + "right.g": (n, W), q + "right.o": (W, n), q + "left.out": (W,), q + "right.out": (W,)})
        if f and f["kind"] == "dense":
            out.update({p + "mlp.gate": (f["ff"], W), p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"])})
        elif f:
            out[p + "mlp.router"] = (f["router"]["experts"], W)
            for e in range(f["router"]["experts"]):
                e, ff = p + f"mlp.e{e}.", f["expert"]["ff"]
                out.update({e + "gate": (ff, W), e + "up": (ff, W), e + "down": (W, ff)})
    out["final.norm"] = (W,)
    out["head"] = (cfg["vocab"], W)
    return out


def _shared_kv_shapes(cfg: dict) -> dict:
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n in ("norm1",) + (("norm2",) if f else ()):
            out[p + n] = (W,)
        q = p + "mix."
        if layer["type"] == "attention":
            out.update({q + "q": (H * D, W), q + "q.b": (H * D,), q + "k": (G * D, W), q + "k.b": (G * D,), q + "sink": (H,),
                        q + "g": (H, W), q + "o": (W, H * D)})
        else:
            out.update({q + "q": (H * 2 * D, W), q + "q.norm": (D,)})
            if m.get("kv_from") is None:
                out.update({q + "k": (G * 2 * D, W), q + "v": (G * V, W), q + "k.norm": (D,)})
            out.update({q + n: (D,) for n in ("lq1", "lk1", "lq2", "lk2")})
            out[q + "o"] = (W, H * V)
        if f:
            r, q = f["router"], p + "mlp."
            parts = [(f"e{e}.", f["expert"]["ff"]) for e in range(r["experts"])]
            if f["shared"]:
                parts.append(("shared.", f["shared"]["ff"]))
                out[q + "shared.sg"] = (1, W)
            out.update({q + "router": (r["experts"] + r["identity"], W), q + "correction": (r["experts"] + r["identity"],)})
            for n, ff in parts:
                out.update({q + n + "gate": (ff, W), q + n + "up": (ff, W), q + n + "down": (W, ff)})
    out["final.norm"] = (W,)
    out["head"] = (cfg["vocab"], W)
    return out


def _recur_shapes(p: str, hd: int, W: int, rank: int) -> dict:
    out = {p + n: (hd, W) for n in "rkvg"}
    out.update({p + "w1": (rank, W), p + "w2": (hd, rank), p + "w0": (hd,), p + "norm": (hd,), p + "o": (W, hd)})
    return out


def _prenorm_shapes(cfg: dict, rank: int) -> dict:
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        for n in ("norm1",) + (("norm2",) if f else ()):
            out[p + n] = (W,)
        if layer["type"] == "wkv":
            hd = m["heads"] * m["dim"]
            out.update(_recur_shapes(p + "mix.", hd, W, rank))
            out.update({p + "mix.mu." + n: (W,) for n in "rkvgw"})
            out[p + "mix.u"] = (m["heads"], m["dim"])
        else:
            a, hd = m["left"], m["right"]["heads"] * m["right"]["dim"]
            q = p + "mix.left."
            out.update({q + "q": (a["heads"] * a["dim"], W), q + "k": (a["kv_heads"] * a["dim"], W),
                        q + "v": (a["kv_heads"] * a["vdim"], W), q + "sink": (a["heads"],), q + "o": (W, a["heads"] * a["vdim"])})
            q = p + "mix.right."
            out.update(_recur_shapes(q, hd, W, rank))
            out.update({q + "a": (hd, W), q + "a.b": (hd,)})
        if f:
            out.update({p + "mlp.gate": (f["ff"], W), p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"])})
    out["final.norm"] = (W,)
    return out


def tensor_shapes(cfg: dict, rank: int = 24) -> dict:
    """`rank`: of the decays' low-rank products, which no configuration names."""
    if cfg["architecture"] == "Taredra":
        return _prenorm_shapes(cfg, rank)
    if cfg["architecture"] == "Fedirax":
        return _shared_kv_shapes(cfg)
    if cfg["architecture"] == "Marosun":
        return _joint_shapes(cfg)
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "embed.norm": (cfg["width"],)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            out[p + n] = (W,)
        H, D, V = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "lightning":
            out.update({p + "mix.q": (H * D, W), p + "mix.k": (H * D, W), p + "mix.v": (H * V, W), p + "mix.g": (H * V, W),
                        p + "mix.o": (W, H * V), p + "mix.norm": (H * V,)})
        else:
            r, qr, kr = m["rot_dim"], m["q_rank"], m["kv_rank"]
            out.update({p + "mix.dq": (qr, W), p + "mix.dq.norm": (qr,), p + "mix.uq": (H * (D + r), qr),
                        p + "mix.dkv": (kr + r, W), p + "mix.dkv.norm": (kr,), p + "mix.uk": (H * D, kr),
                        p + "mix.uv": (H * V, kr), p + "mix.o": (W, H * V)})
        if f and f["kind"] == "dense":
            out.update({p + "mlp.gate": (f["ff"], W), p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"])})
        elif f:
            out[p + "mlp.router"] = (f["router"]["experts"], W)
            for e in range(f["router"]["experts"]):
                out[p + f"mlp.e{e}.up"] = (f["expert"]["ff"], W)
                out[p + f"mlp.e{e}.down"] = (W, f["expert"]["ff"])
    out["final.norm"] = (W,)
    out["head"] = (cfg["vocab"], W)
    return out


def to_bf16(x: np.ndarray) -> np.ndarray:
    """Bit patterns, round to nearest even."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    return ((u + np.uint32(0x7FFF) + ((u >> np.uint32(16)) & np.uint32(1))) >> np.uint32(16)).astype(np.uint16)


# what the vectors of a pre-norm model are drawn around, and how widely
_VECTORS = {"norm1": (0, 0.1), "norm2": (0, 0.1), "final.norm": (0, 0.1), "sink": (0, 1), "w0": (-3, 2), "a.b": (0, 1),
            "q.b": (0, 0.5), "k.b": (0, 0.5), "correction": (0, 0.05), "lq1": (0, 0.1), "lk1": (0, 0.1), "lq2": (0, 0.1),
            "lk2": (0, 0.1), "v.b": (0, 0.5), "o.b": (0, 0.2), "f.b": (1, 1), "z.b": (-1, 1), "x.b": (0, 0.5)}


def random_tensors(cfg: dict, seed: int = 0, gain: float = 1.0, rank: int = 24):
    """Yields (name, bfloat16 bits): norms 1 + 0.1 N(0, 1), matrices gain * N(0, 1 / inputs), the embedding N(0, 1);
    of a pre-norm model the vectors as _VECTORS says, mixing factors and lower bounds in [0, 1], bonuses N(0, 1/4), the embedding N(0, 1 / width).
    Large matrices repeat a pool of samples at different offsets."""
    prenorm = cfg["architecture"] != "Bipotar"
    rng = np.random.default_rng(seed)
    pool = rng.standard_normal(1 << 22, dtype=np.float32)
    for i, (name, shape) in enumerate(tensor_shapes(cfg, rank).items()):
        n = int(np.prod(shape))
        at = int(rng.integers(0, pool.size))
        x = pool[(at + np.arange(n)) % pool.size] if n <= pool.size else np.resize(np.roll(pool, at), n)
        end = name.split(".", 2)[-1] if name.startswith("l") else name
        end = end.removeprefix("left.").removeprefix("right.")
        if prenorm and (".mu." in name or end == "lower"):
            x = 1.0 / (1.0 + np.exp(-x))
        elif prenorm and end == "u":
            x = 0.5 * x
        elif prenorm and name == "embed" and cfg["architecture"] == "Taredra":
            x = x * np.float32(shape[1] ** -0.5)
        elif prenorm and end in _VECTORS:
            at, spread = _VECTORS[end]
            x = at + spread * x
        elif len(shape) == 1:
            x = 1.0 + 0.1 * x
        elif name != "embed":
            x = x * np.float32(gain / np.sqrt(shape[1]))
        yield name, to_bf16(x).reshape(shape)


def write_model(folder: str, cfg: dict, tensors=None, seed: int = 0, rank: int = 24) -> str:
    """tensors: {name: bfloat16 bits} or an iterable of such pairs; None draws random ones."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    shapes = tensor_shapes(cfg, rank)
    header, at = {}, 0
    for name, shape in shapes.items():
        n = 2 * int(np.prod(shape))
        header[name] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [at, at + n]}
        at += n
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    if tensors is None:
        tensors = random_tensors(cfg, seed, rank=rank)
    pairs = tensors.items() if isinstance(tensors, dict) else tensors
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        base = f.tell()
        f.truncate(base + at)
        for name, bits in pairs:
            assert bits.dtype == np.uint16 and bits.shape == tuple(shapes[name]), name
            f.seek(base + header[name]["data_offsets"][0])
            f.write(bits.tobytes())
    return folder
