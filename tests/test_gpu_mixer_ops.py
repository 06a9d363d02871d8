"""The matrix products of mixer-stack models by themselves, through the C ABI: every
kernel the row and output counts can select, every place an output can go, against
numpy on the same (bfloat16-exact) operands."""
import ctypes as C

import numpy as np
import pytest

from tests import mixer_oracle as O
from wayruntime_amd import hipattn

pytestmark = pytest.mark.gpu

ROWS_F32, ROWS, FRAG, SPLIT, GATED, SPLIT_GATED = range(6)
u32, vp = C.c_uint32, C.c_void_p


class Gemm(C.Structure):
    _fields_ = [("w", vp), ("x", vp), ("x_kt", u32), ("x_kt_z", u32), ("rows", u32), ("group_expert", vp),
                ("tile_groups", u32), ("out", u32), ("y_f32", vp), ("y_act", vp), ("ldy", u32), ("h", vp), ("h_kt", u32),
                ("col_z", u32), ("n_split", u32), ("silu_end", u32), ("sigmoid_end", u32), ("relu2", u32), ("scale", C.c_float),
                ("tanh_end", u32), ("gelu", u32), ("x_kt0", u32), ("bias", vp), ("limit", C.c_float), ("slope", C.c_float),
                ("up_bias", C.c_float), ("x_perm", vp), ("h_kt0", u32), ("x_scale", vp)]


@pytest.fixture(scope="module")
def lib():
    hipattn.init(0)
    lib = hipattn.lib()
    lib.wr_hip_mix_mat_create.argtypes = [u32, u32, u32, vp, C.POINTER(vp)]
    lib.wr_hip_mix_mat_destroy.argtypes = [vp]
    lib.wr_hip_mix_mat_destroy.restype = None
    lib.wr_hip_mix_gemm_run.argtypes = [C.c_int, C.POINTER(Gemm)]
    return lib


def frag(x):
    """[rows][K] -> operand order [rows/16][K/32][64][8], rows padded with NaN (nobody may use them)."""
    r = -(-x.shape[0] // 16) * 16
    p = np.full((r, x.shape[1]), np.nan, dtype=np.float32)
    p[:len(x)] = x
    return np.ascontiguousarray(p.reshape(r // 16, 16, -1, 4, 8).transpose(0, 2, 3, 1, 4))


def unfrag(f, rows, K):
    return f.reshape(-1, K // 32, 4, 16, 8).transpose(0, 3, 1, 2, 4).reshape(-1, K)[:rows]


class Run:
    def __init__(self, lib, f32, batch, N, K, rows, seed=0):
        rng = np.random.default_rng(seed)
        self.lib, self.f32, self.N, self.K, self.rows = lib, f32, N, K, rows
        self.bits = O.f32_to_bf16(rng.standard_normal((batch, N, K), dtype=np.float32) / np.float32(np.sqrt(K)))
        self.w = O.bf16_to_f32(self.bits)
        self.h = vp()
        assert lib.wr_hip_mix_mat_create(batch, N, K, self.bits.ctypes.data, C.byref(self.h)) == 0
        self.rng = rng

    def act(self, rows, K):
        x = self.rng.standard_normal((rows, K), dtype=np.float32)
        return x if self.f32 else O.bf16_to_f32(O.f32_to_bf16(x))

    def up(self, x):
        f = frag(x)
        return hipattn.DeviceBuffer.from_host(f if self.f32 else O.f32_to_bf16(np.nan_to_num(f, nan=0.0)) +
                                              np.where(np.isnan(f), np.uint16(0x7FC0), np.uint16(0)).astype(np.uint16))

    def go(self, x, **kw):
        g = Gemm(w=self.h, x=x.p, x_kt=kw.pop("x_kt", self.K // 32), rows=kw.pop("rows", self.rows), **kw)
        assert self.lib.wr_hip_mix_gemm_run(int(self.f32), C.byref(g)) == 0
        hipattn.sync()

    def frag_down(self, buf, rows, K):
        n = -(-rows // 16) * 16 * K
        if self.f32:
            return unfrag(buf.to_host((n,)), rows, K)
        b = buf.to_host((n // 2,)).view(np.uint16)
        return unfrag(O.bf16_to_f32(b), rows, K)

    def close(self, got, want, eight_bits=False):
        tol = 2.0 ** -7 if eight_bits and not self.f32 else 2e-5
        assert np.isfinite(got).all()
        err = np.abs(got - want).max() / max(1.0, np.abs(want).max())
        assert err < tol, err

    def end(self):
        self.lib.wr_hip_mix_mat_destroy(self.h)


# (outputs, inputs, rows): what each picks among the streaming kernels and the three LDS-staged tiles
SHAPES = [(16, 32, 1), (48, 96, 7), (32, 416, 16), (4096, 64, 3), (80, 4096, 16), (64, 64, 17), (96, 160, 33), (160, 96, 70),
          (1024, 512, 200), (8192, 96, 256), (16384, 64, 250), (16384, 64, 600), (2064, 352, 1100)]


@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("N,K,rows", SHAPES)
def test_rows_out(lib, f32, N, K, rows):
    r = Run(lib, f32, 1, N, K, rows)
    x = r.act(rows, K)
    y = hipattn.DeviceBuffer(rows * N * 4)
    xd = r.up(x)
    want = x.astype(np.float64) @ r.w[0].T.astype(np.float64)
    r.go(xd, out=ROWS_F32, y_f32=y.p, ldy=N, scale=0.5)
    r.close(y.to_host((rows, N)), 0.5 * want)
    silu, sig = N // 2 + 3, N - 5                          # ends inside a tile
    r.go(xd, out=ROWS_F32, y_f32=y.p, ldy=N, silu_end=silu, sigmoid_end=sig)
    act = want.copy()
    act[:, :silu] = O.silu(want[:, :silu])
    act[:, silu:sig] = O.sigmoid(want[:, silu:sig])
    r.close(y.to_host((rows, N)), act)
    r.go(xd, out=ROWS_F32, y_f32=y.p, ldy=N, silu_end=N // 4, tanh_end=N - 7)
    act = want.copy()
    act[:, :N // 4] = O.silu(want[:, :N // 4])
    act[:, N // 4:N - 7] = np.tanh(want[:, N // 4:N - 7])
    r.close(y.to_host((rows, N)), act)
    bias = r.rng.standard_normal(N).astype(np.float32)
    bd = hipattn.DeviceBuffer.from_host(bias)
    r.go(xd, out=ROWS_F32, y_f32=y.p, ldy=N, bias=bd.p)
    r.close(y.to_host((rows, N)), want + bias)
    r.end()
    for b in (y, xd, bd):
        b.free()


@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("N,K,rows", [(64, 96, 1), (128, 64, 20), (512, 64, 90), (16384, 32, 300)])
def test_frag_split_and_gated_out(lib, f32, N, K, rows):
    r = Run(lib, f32, 1, N, K, rows)
    x = r.act(rows, K)
    xd = r.up(x)
    want = x.astype(np.float64) @ r.w[0].T.astype(np.float64)
    esize = 4 if f32 else 2
    h = hipattn.DeviceBuffer(-(-rows // 16) * 16 * N * esize)
    r.go(xd, out=FRAG, h=h.p, h_kt=N // 32, relu2=1)
    r.close(r.frag_down(h, rows, N), np.maximum(want, 0) ** 2, eight_bits=True)
    split = N // 2 // 32 * 32
    y = hipattn.DeviceBuffer(rows * (N - split) * 4)
    r.go(xd, out=SPLIT, h=h.p, h_kt=split // 32, n_split=split, y_f32=y.p, ldy=N - split)
    r.close(r.frag_down(h, rows, split), want[:, :split], eight_bits=True)
    r.close(y.to_host((rows, N - split)), want[:, split:])
    r.go(xd, out=GATED, h=h.p, h_kt=N // 64)
    t = want.reshape(rows, N // 32, 2, 16)
    r.close(r.frag_down(h, rows, N // 2), (O.silu(t[:, :, 0]) * t[:, :, 1]).reshape(rows, -1), eight_bits=True)
    r.go(xd, out=GATED, h=h.p, h_kt=N // 64, gelu=1)
    r.close(r.frag_down(h, rows, N // 2), (O.gelu_tanh(t[:, :, 0]) * t[:, :, 1]).reshape(rows, -1), eight_bits=True)

    def clamped(g, u, limit, slope, more):
        g = np.minimum(g, limit)
        return g * O.sigmoid(slope * g) * (np.clip(u, -limit, limit) + more)
    for limit in (0.3, 5.0):
        r.go(xd, out=GATED, h=h.p, h_kt=N // 64, limit=limit, slope=1.5, up_bias=0.75)
        r.close(r.frag_down(h, rows, N // 2), clamped(t[:, :, 0], t[:, :, 1], limit, 1.5, 0.75).reshape(rows, -1), eight_bits=True)
    # rows ahead of the gated outputs
    for split in (32, N // 2 // 32 * 32):
        r.go(xd, out=SPLIT_GATED, h=h.p, h_kt=(N - split) // 64 + 1, n_split=split, y_f32=y.p, ldy=split, limit=0.6, slope=2.0, up_bias=1.0)
        r.close(y.to_host((rows, split)), want[:, :split])
        u = want[:, split:].reshape(rows, -1, 2, 16)
        got = r.frag_down(h, rows, ((N - split) // 64 + 1) * 32)[:, :(N - split) // 2]
        r.close(got, clamped(u[:, :, 0], u[:, :, 1], 0.6, 2.0, 1.0).reshape(rows, -1), eight_bits=True)
    # those rows with a bias and an activation, the gated outputs behind three input tiles of a wider operand
    split, silu, tiles = N // 2 // 32 * 32, 27, (N - N // 2 // 32 * 32) // 64 + 4
    bias = np.pad(r.rng.standard_normal(split).astype(np.float32), (0, N - split), constant_values=np.nan)
    bd, wide = hipattn.DeviceBuffer.from_host(bias), hipattn.DeviceBuffer.from_host(np.full((-(-rows // 16) * 16, tiles * 32), 3.0, np.float32))
    r.go(xd, out=SPLIT_GATED, h=wide.p, h_kt=tiles, h_kt0=3, n_split=split, y_f32=y.p, ldy=split, bias=bd.p, silu_end=silu)
    v = want[:, :split] + bias[:split]
    r.close(y.to_host((rows, split)), np.concatenate([O.silu(v[:, :silu]), v[:, silu:]], axis=1))
    got, u = r.frag_down(wide, rows, tiles * 32), want[:, split:].reshape(rows, -1, 2, 16)
    r.close(got[:, 96:96 + (N - split) // 2], (O.silu(u[:, :, 0]) * u[:, :, 1]).reshape(rows, -1), eight_bits=True)
    blank = 3.0 if f32 else O.bf16_to_f32(np.full(2, 3.0, np.float32).view(np.uint16)[1::2])[0]
    assert set(np.unique(got[:, :96])) <= {blank, np.float32(0)}
    r.end()
    for b in (y, xd, h, bd, wide):
        b.free()


@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("batch,N,K,rows", [(3, 64, 32, 1), (5, 32, 96, 40), (40, 512, 64, 300), (2, 128, 64, 130)])
def test_batch_of_matrices(lib, f32, batch, N, K, rows):
    # matrix z takes its own input columns and writes its own output columns
    r = Run(lib, f32, batch, N, K, rows)
    x = r.act(rows, batch * K)
    xd = r.up(x)
    h = hipattn.DeviceBuffer(-(-rows // 16) * 16 * N * batch * (4 if f32 else 2))
    r.go(xd, x_kt=batch * K // 32, x_kt_z=K // 32, out=FRAG, h=h.p, h_kt=batch * N // 32, col_z=N)
    want = np.einsum("rzk,znk->rzn", x.reshape(rows, batch, K).astype(np.float64), r.w.astype(np.float64)).reshape(rows, -1)
    r.close(r.frag_down(h, rows, batch * N), want, eight_bits=True)
    # and to columns of shared 32-bit rows, from inputs that start further in
    x = r.act(rows, (batch + 1) * K)
    xd2, y = r.up(x), hipattn.DeviceBuffer(rows * batch * N * 4)
    r.go(xd2, x_kt=(batch + 1) * K // 32, x_kt_z=K // 32, x_kt0=K // 32, out=ROWS_F32, y_f32=y.p, ldy=batch * N, col_z=N)
    x = x.reshape(rows, batch + 1, K)[:, 1:]
    r.close(y.to_host((rows, batch * N)), np.einsum("rzk,znk->rzn", x.astype(np.float64), r.w.astype(np.float64)).reshape(rows, -1))
    r.end()
    for b in (xd, xd2, h, y):
        b.free()


@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("N,K,tile", [(64, 96, 1), (48, 64, 8), (4096, 64, 8), (1024, 32, 1)])
def test_matrix_per_row_group(lib, f32, N, K, tile):
    experts = 4
    r = Run(lib, f32, experts, N, K, 0)
    which = np.repeat(np.array([2, 0, -1, 3, 2], dtype=np.int32), tile)
    rows = 16 * len(which)
    x = r.act(rows, K)
    xd, gd = r.up(x), hipattn.DeviceBuffer.from_host(which.view(np.float32))
    y = hipattn.DeviceBuffer.from_host(np.full((rows, N), 7.0, dtype=np.float32))
    r.go(xd, rows=rows, group_expert=gd.p, tile_groups=tile, out=ROWS_F32, y_f32=y.p, ldy=N)
    want = np.full((rows, N), 7.0)                          # groups nobody uses stay as they are
    for g, e in enumerate(which):
        if e >= 0:
            want[16 * g:16 * g + 16] = x[16 * g:16 * g + 16].astype(np.float64) @ r.w[e].T.astype(np.float64)
    r.close(y.to_host((rows, N)), want)
    # a factor per row, ahead of the gated units
    factor = r.rng.uniform(0, 2, rows).astype(np.float32)
    fd, h = hipattn.DeviceBuffer.from_host(factor), hipattn.DeviceBuffer(rows * (N // 32 * 16 + 32) * 4)
    if N % 64 == 0:
        r.go(xd, rows=rows, group_expert=gd.p, tile_groups=tile, out=GATED, h=h.p, h_kt=N // 64, x_scale=fd.p)
        t = (np.where(np.repeat(which, 16)[:, None] >= 0, want, 0) * factor[:, None]).reshape(rows, N // 32, 2, 16)
        live = np.repeat(which, 16) >= 0
        r.close(r.frag_down(h, rows, N // 2)[live], (O.silu(t[:, :, 0]) * t[:, :, 1]).reshape(rows, -1)[live], eight_bits=True)
    for b in (fd, h):
        b.free()
    if tile == 1:                                          # rows picked one by one out of fewer
        pick = r.rng.integers(0, 21, rows).astype(np.uint32)
        used = r.rng.random(rows) < 0.8
        few = r.act(21, K)
        fd = r.up(few)
        pd = hipattn.DeviceBuffer.from_host(np.where(used, pick, np.uint32(0xFFFFFFFF)).astype(np.uint32).view(np.float32))
        r.go(fd, rows=rows, group_expert=gd.p, tile_groups=1, out=ROWS_F32, y_f32=y.p, ldy=N, x_perm=pd.p)
        got = y.to_host((rows, N))
        for g, e in enumerate(which):
            for i in range(16 * g, 16 * g + 16):
                if e >= 0 and used[i]:
                    r.close(got[i], few[pick[i]].astype(np.float64) @ r.w[e].T.astype(np.float64))
        for b in (fd, pd):
            b.free()
    r.end()
    for b in (xd, gd, y):
        b.free()


def test_refusals(lib):
    r = Run(lib, False, 1, 32, 32, 16)
    y = hipattn.DeviceBuffer(16 * 32 * 4)
    ok = dict(w=r.h, x=y.p, x_kt=1, rows=16, out=ROWS_F32, y_f32=y.p, ldy=32)
    for change in (dict(x_kt=0), dict(ldy=28), dict(ldy=33), dict(y_f32=None), dict(out=9), dict(rows=0), dict(w=None),
                   dict(out=FRAG, h=y.p, h_kt=0), dict(out=SPLIT, h=y.p, h_kt=1, n_split=8), dict(out=GATED), dict(x_kt0=1),
                   dict(out=GATED, h=y.p, h_kt=1, bias=y.p), dict(x_perm=y.p), dict(x_scale=y.p),
                   dict(out=GATED, h=y.p, h_kt=1, h_kt0=1), dict(out=SPLIT_GATED, h=y.p, h_kt=1, n_split=16)):
        assert lib.wr_hip_mix_gemm_run(0, C.byref(Gemm(**dict(ok, **change)))) == hipattn.ERR_INVAL, change
    h = vp()
    for shape in ((1, 8, 32), (1, 16, 16), (0, 16, 32)):
        assert lib.wr_hip_mix_mat_create(*shape, r.bits.ctypes.data, C.byref(h)) == hipattn.ERR_INVAL
    r.end()
    y.free()
