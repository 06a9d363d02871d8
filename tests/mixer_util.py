"""What the device tests of mixer-stack models share: a model with random weights on
the device beside its plain implementation, and a request cut into portions."""
import numpy as np

from tests import mixer_oracle as O
from wayruntime_amd import engine as E, mix_writer as mw

# error of a row of logits: RMS of the difference over RMS of the row.  32-bit: rounding of
# long sums; bfloat16: operands carry eight bits through a dozen products.
TOL = {"f32": 2e-5, "bf16": 4e-2}


class Case:
    """A model on the device and its oracle."""

    def __init__(self, eng, tmp_path, cfg, prec, seed=1, edit=None, pool=1024, slots=4):
        self.cfg, self.prec = cfg, prec
        bits = dict(mw.random_tensors(cfg, seed))
        if edit:
            edit(bits)
        self.w = {k: O.bf16_to_f32(v) for k, v in bits.items()}
        self.m = eng.load(mw.write_model(str(tmp_path / "model"), cfg, bits), max_context=pool,
                          quant=E.WR_QUANT_F32 if prec == "f32" else E.WR_QUANT_AUTO)
        self.m.set_cache_pool(pool, slots)

    def tokens(self, n, seed=3):
        return np.random.default_rng(seed).integers(0, self.cfg["vocab"], n)

    def oracle(self, tokens):
        return O.forward(self.cfg, self.w, tokens, np.float64)

    def check(self, got, want, what, deep=False):
        """deep: several layers, where in bfloat16 a row now and then is ill-conditioned (a small sum ahead of a
        norm): at most one row in fifty above the tolerance then, and none above five times it."""
        bad = np.flatnonzero(~np.isfinite(got).all(axis=-1))
        assert bad.size == 0, (what, "rows not finite", bad[:20].tolist(), bad.size)
        d = got.astype(np.float64) - want
        err = np.sqrt((d ** 2).mean(axis=-1)) / np.sqrt((want ** 2).mean(axis=-1))
        print(f"{what} {self.prec}: worst row {err.max():.2e} of {len(err)}", flush=True)
        if deep and self.prec == "bf16":
            assert (err > TOL["bf16"]).sum() <= max(1, 0.02 * len(err)) and err.max() < 5 * TOL["bf16"], (what, err.max())
        else:
            assert err.max() < TOL[self.prec], (what, int(err.argmax()), float(err.max()))

    def close(self):
        self.m.close()


def f32_edit(change):
    """An edit of a model's tensors as floats."""
    def edit(bits):
        f = {k: O.bf16_to_f32(v).copy() for k, v in bits.items()}
        change(f)
        for k, v in f.items():
            bits[k] = O.f32_to_bf16(v)
    return edit


def run_cut(case, tokens, cuts):
    """All logits of one request whose tokens come in portions of the given sizes (the last repeats)."""
    s, out, at, i = case.m.session(), [], 0, 0
    while at < len(tokens):
        n = min(cuts[min(i, len(cuts) - 1)], len(tokens) - at)
        rc, lg = E.mixed_step([(s, tokens[at:at + n], range(n))])
        assert rc == n
        out.append(lg[0])
        at, i = at + n, i + 1
    s.close()
    return np.concatenate(out)
