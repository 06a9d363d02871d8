"""Prefill and decode throughput of mixer-stack models (random weights, layers of
real sizes) beside a grouped-query model of the same width, through the host
engine.

    python -m wayruntime_amd.mix_timing [--size w2048 w4096] [--only mixer taredra fedirax marosun gqa] [--json]

Each size has four layers.  mixer: linear attention with a dense feed-forward and
with experts, latent attention with experts and with a dense feed-forward.
taredra: windowed grouped-query attention beside a delta-rule recurrence, and a
wkv recurrence, each twice, all with dense feed-forwards.  fedirax: differential
attention, keys-as-values attention, differential attention and such over the first
layer's keys and values, all with experts and a shared one.  marosun: attention over
turned values, attention beside an element-wise gated recurrence (both with dense
feed-forwards), chunked attention beside a forget-gate recurrence, attention over turned
values (both with experts).  gqa: the engine's
Llama-style model with four layers of the same width, head dimension and
feed-forward width (F16 weights)."""
from __future__ import annotations

import argparse
import ctypes as C
import json
import os
import sys
import tempfile
import time

import numpy as np

from wayruntime_amd import engine as E, gguf_writer as gw, mix_writer as mw

VOCAB = 32768


def mixer_config(width: int, heads: int, q_rank: int, ff: int, experts: int, top: int, expert_ff: int) -> dict:
    light = mw.lightning(heads, 128, 128)
    latent = mw.latent_attention(heads, 128, 128, q_rank, 512, 64, window=4096)
    d, m = mw.dense(ff), mw.moe(experts, top, expert_ff)
    return mw.config(width, VOCAB, [(light, d), (light, m), (latent, m), (latent, d)])


def taredra_config(width: int, heads: int, ff: int) -> dict:
    """Heads of 128 over eight key/value heads; recurrences with heads of 64 over the whole width."""
    par = mw.window_and_delta(heads, 8, 128, 128, window=4096, right_heads=width // 64, right_dim=64)
    return mw.prenorm_config(width, VOCAB, [(m, mw.dense(ff)) for m in (par, mw.wkv(width // 64, 64)) * 2])


def fedirax_config(width: int, heads: int, experts: int, top: int, expert_ff: int, shared_ff: int) -> dict:
    """Two maps of 64 per head over values of 128, eight key/value heads; eight of the router's outputs pass the input on."""
    diff = dict(heads=heads, kv_heads=8, dim=64, vdim=128, window=4096)
    keys = mw.keys_as_values(heads, 8, 128, window=4096)
    moe = mw.grouped_moe(experts, top, expert_ff, identity=8, groups=(8, 4), scale=2.0, shared=(shared_ff, 7.0))
    return mw.shared_kv_config(width, VOCAB, [(m, moe) for m in (mw.difference(**diff), keys, mw.difference(**diff),
                                                                 mw.difference(**diff, kv_from=0))])


def marosun_config(width: int, heads: int, ff: int, experts: int, top: int, expert_ff: int) -> dict:
    """Heads of 128 over eight key/value heads; recurrences with heads of 128 x 128, and of the model's width."""
    a = dict(heads=heads, kv_heads=8, dim=128, vdim=128)
    turned, d, m = mw.turned_values(**a, rot_dims=64), mw.clamped_dense(ff), mw.moe(experts, top, expert_ff)
    return mw.joint_config(width, VOCAB, [
        (turned, d), (mw.one_more_and_gru(**a, size=width), d),
        (mw.chunks_and_forget(**a, chunk=4096, right_heads=width // 128, right_dim=128, right_vdim=128), m), (turned, m)])


KINDS = ("mixer", "taredra", "fedirax", "marosun", "gqa")
RANK = 64                                   # of the decays' low-rank products
SIZES = {
    "w2048": (mixer_config(2048, 16, 768, 8192, 64, 6, 1024), taredra_config(2048, 16, 8192),
              fedirax_config(2048, 16, 64, 6, 1024, 2048), marosun_config(2048, 16, 8192, 64, 6, 1024),
              gw.ModelShape(arch="llama", n_layers=4, hidden=2048, ffn=8192, n_q=16, n_kv=8, vocab=VOCAB, context=8192)),
    "w4096": (mixer_config(4096, 32, 1536, 12288, 32, 4, 2048), taredra_config(4096, 32, 12288),
              fedirax_config(4096, 32, 32, 4, 2048, 4096), marosun_config(4096, 32, 12288, 32, 4, 2048),
              gw.ModelShape(arch="llama", n_layers=4, hidden=4096, ffn=12288, n_q=32, n_kv=8, vocab=VOCAB, context=8192)),
}


def tokens(n: int) -> np.ndarray:
    return ((np.arange(n, dtype=np.uint64) * 2654435761 + 12345) % VOCAB).astype(np.uint32)


def best_prefill(m, n: int, reps: int) -> float:
    best = None
    for _ in range(reps):
        s = m.session()
        t = time.perf_counter()
        assert s.prefill(tokens(n)) == n
        dt = time.perf_counter() - t
        best = dt if best is None else min(best, dt)
        s.close()
    return best


def decode(m, n_sessions: int, ctx: int, steps: int) -> float:
    """Median seconds per step, the engine call alone."""
    ss = [m.session() for _ in range(n_sessions)]
    for i, s in enumerate(ss):
        assert s.prefill(tokens(ctx + i)) == ctx + i
    hs = (C.c_void_p * n_sessions)(*[s.h for s in ss])
    outs = (C.POINTER(C.c_float) * n_sessions)()
    per = []
    for k in range(steps + 3):
        t_c = (C.c_uint32 * n_sessions)(*[(7 * k + i) % VOCAB for i in range(n_sessions)])
        t = time.perf_counter()
        rc = ss[0].lib.wr_batch_step(hs, t_c, n_sessions, outs)
        per.append(time.perf_counter() - t)
        assert rc == n_sessions
    for s in ss:
        s.close()
    return float(np.median(per[3:]))


def measure(eng, path: str, reps: int, steps: int) -> dict:
    m = eng.load(path, max_context=4352)
    out = {}
    for n in (512, 2048, 4096):
        best_prefill(m, n, 1)
        dt = best_prefill(m, n, reps)
        out[f"prefill_{n}_ms"] = round(dt * 1e3, 3)
        out[f"prefill_{n}_tok_s"] = round(n / dt)
    for b in (1, 16):
        dt = decode(m, b, 2048, steps)
        out[f"decode_b{b}_ms"] = round(dt * 1e3, 4)
        out[f"decode_b{b}_tok_s"] = round(b / dt)
    m.close()
    return out


def run(sizes, reps: int = 3, steps: int = 40, only=KINDS, log=print) -> dict:
    figures = {}
    with tempfile.TemporaryDirectory() as tmp:
        eng = E.Engine(E.HOST_SO)
        for name in sizes:
            models = dict(zip(KINDS, SIZES[name]))
            fig = figures[name] = {}
            for kind in only:
                t = time.perf_counter()
                path = os.path.join(tmp, name + "_" + kind)
                if kind == "gqa":
                    path += ".gguf"
                    gw.write_model(path, models[kind])
                else:
                    mw.write_model(path, models[kind], rank=RANK)
                log(f"{name}: {kind} model written in {time.perf_counter() - t:.1f} s")
                fig[kind] = measure(eng, path, reps, steps)
                log(f"{name}: {kind} {fig[kind]}")
        eng.close()
    return figures


def main() -> int:
    ap = argparse.ArgumentParser(description=__doc__.split("\n\n")[0])
    ap.add_argument("--size", nargs="*", default=list(SIZES), choices=list(SIZES))
    ap.add_argument("--only", nargs="*", default=list(KINDS), choices=list(KINDS))
    ap.add_argument("--reps", type=int, default=3)
    ap.add_argument("--steps", type=int, default=40)
    ap.add_argument("--json", action="store_true", help="one JSON line with the figures at the end")
    args = ap.parse_args()
    figures = run(args.size, args.reps, args.steps, args.only, log=lambda *a: print(*a, flush=True))
    if args.json:
        print(json.dumps(figures), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
