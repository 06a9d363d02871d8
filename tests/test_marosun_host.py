"""Mixer-stack models whose layers' mixers and feed-forward read one norm (architecture
"Marosun") through the host engine on the CPU test double (plain loops in place of the
device steps, 32-bit): reading and rearranging weights, the mixed step and rollback,
against the plain implementation of tests/mixer_oracle.py."""
import json
import os

import numpy as np
import pytest

import oracle
from tests import mixer_oracle as O
from wayruntime_amd import engine as E, mix_writer as mw

CFG = mw.joint_config(40, 61, [
    (mw.turned_values(4, 2, 10, 14, rot_dims=6, base=777.0, scaling=(3.0, 40, 3.0, 0.5)), mw.clamped_dense(18, 0.8)),
    (mw.chunks_and_forget(3, 3, 8, 6, 23, 2, 5, 9, left_scale=0.7, right_scale=1.2), mw.moe(5, 2, 18)),
    (mw.one_more_and_gru(6, 2, 10, 12, 27, rot_dims=4, base=777.0), mw.clamped_dense(8, 2.0)),
    (mw.turned_values(2, 1, 8, 6, scaling=None), mw.moe(4, 1, 10)),
    (mw.one_more_and_gru(1, 1, 8, 8, 33), mw.moe(3, 2, 6)),
    (mw.chunks_and_forget(2, 1, 6, 8, 70, 3, 8, 4), None)], eps=1e-5)


@pytest.fixture(scope="module")
def eng():
    oracle.build(ref=False)
    e = E.Engine(oracle.HOSTCPU_SO, threads=4)
    e.lib.wrh_debug_poison_scratch(1)
    yield e
    e.lib.wrh_debug_poison_scratch(0)
    e.close()


@pytest.fixture(scope="module")
def made(tmp_path_factory):
    bits = dict(mw.random_tensors(CFG, 4))
    return (mw.write_model(str(tmp_path_factory.mktemp("mix") / "m"), CFG, bits),
            {k: O.bf16_to_f32(v) for k, v in bits.items()})


@pytest.fixture()
def model(eng, made):
    m = eng.load(made[0], max_context=256, quant=E.WR_QUANT_F32)
    yield m
    m.close()


def toks(n, seed=0):
    return np.random.default_rng(seed).integers(0, CFG["vocab"], n)


def near(got, want):
    assert np.sqrt(((got - want) ** 2).mean(-1)).max() < 2e-5 * np.sqrt((want ** 2).mean(-1)).max()


def test_info(model):
    i = model.info
    assert (i.arch, i.quant, i.vocab_size, i.hidden_dim, i.max_context) == (b"Marosun", b"BF16", 61, 40, 256)
    assert (i.n_layers, i.n_q_heads, i.n_kv_heads, i.sliding_window, i.tied_lm_head) == (6, 6, 3, 70, 0)


def test_prompt_portions_and_single_tokens(model, made):
    t = toks(150)
    want = O.forward(CFG, made[1], t, np.float64)
    for cuts in ([150], [1], [2, 63, 1, 64, 17, 3]):
        s, at, i = model.session(), 0, 0
        while at < len(t):
            n = min(cuts[i % len(cuts)], len(t) - at)
            rc, lg = E.mixed_step([(s, t[at:at + n], range(n))])
            assert rc == n
            near(lg[0], want[at:at + n])
            at, i = at + n, i + 1
        s.close()


def test_residual_after_every_layer(model, made):
    t, cap = toks(30), []
    O.forward(CFG, made[1], t, np.float64, cap)
    got = np.zeros((len(cap), 30, 40), dtype=np.float32)
    s = model.session()
    model.capture_residual(got)
    E.mixed_step([(s, t, [])])
    model.capture_residual(None)
    for a, b in zip(got, cap):
        near(a, b)
    s.close()


def test_batch_equals_alone_and_pages_come_back(eng, made):
    m = eng.load(made[0], max_context=256, quant=E.WR_QUANT_F32)
    m.set_cache_pool(320, 2)                                # five pages, two slots
    want = {n: O.forward(CFG, made[1], toks(n, n), np.float64) for n in (130, 70, 200, 3)}
    for pair in ((130, 70), (200, 3), (70, 130), (3, 200)):
        ss = [m.session() for _ in pair]
        half = [n // 2 + 1 for n in pair]
        rc, _ = E.mixed_step([(s, toks(n, n)[:h], []) for s, n, h in zip(ss, pair, half)])
        assert rc == 0
        rc, lg = E.mixed_step([(s, toks(n, n)[h:], range(n - h)) for s, n, h in zip(ss, pair, half)])
        for n, h, x in zip(pair, half, lg):
            near(x, want[n][h:])
        for s in ss:
            s.close()
    m.close()


def test_failure_anywhere_changes_nothing(model, made):
    t = toks(90)
    want = O.forward(CFG, made[1], t, np.float64)
    s, other = model.session(), model.session()
    assert s.prefill(t[:33]) == 33 and other.prefill(t[:3]) == 3
    for k in (1, 2, 9, 14):
        s.lib.wr_hip_mix_debug_fail_product_in(k)
        rc, _ = E.mixed_step([(s, t[33:70], [0]), (other, t[3:5], [])])
        assert rc == E.WR_ERR_INTERNAL and (s.pos, other.pos) == (33, 3)
    s.lib.wr_hip_mix_debug_fail_product_in(0)
    for run in range(6):
        s.lib.wrh_debug_fail_attention_at(run)
        assert s.step(int(t[33])) is None and s.pos == 33
    rc, lg = E.mixed_step([(s, t[33:], range(57)), (other, t[3:5], [0, 1])])
    near(lg[0], want[33:])
    near(lg[1], want[3:5])
    s.close()
    other.close()


def test_greedy_through_step_and_batch(model, made):
    p = toks(9)
    t = list(p)
    for _ in range(6):
        t.append(int(O.forward(CFG, made[1], t, np.float64)[-1].argmax()))
    s, u = model.session(), model.session()
    s.prefill(p[:-1])
    u.prefill(p[:-1])
    tok, got = int(p[-1]), []
    for _ in range(6):
        rc, lg = E.batch_step([s, u], [tok, tok])
        assert rc == 2 and np.allclose(lg[0], lg[1], atol=1e-5)
        tok = int(lg[0].argmax())
        got.append(tok)
    assert got == t[9:]
    s.close()
    u.close()


def _rc(eng, tmp_path, change=None, tensor=None):
    cfg = json.loads(json.dumps(CFG))
    d = mw.write_model(str(tmp_path / "b"), cfg)
    if change:
        path, value = change
        o = cfg
        for k in path[:-1]:
            o = o[k]
        o.pop(path[-1], None)
        if value is not None:
            o[path[-1]] = value
        with open(os.path.join(d, "config.json"), "w") as f:
            json.dump(cfg, f)
    if tensor:
        st = os.path.join(d, "model.safetensors")
        whole = open(st, "rb").read()
        assert whole.count(tensor[0]) == 1 and len(tensor[0]) == len(tensor[1])
        with open(st, "wb") as f:
            f.write(whole.replace(*tensor))
    try:
        eng.load(d, max_context=64, quant=E.WR_QUANT_F32).close()
    except E.EngineError as e:
        return e.rc
    return E.WR_OK


MIX = tuple(("layers", i, "mixer") for i in range(6))


@pytest.mark.parametrize("path,value,rc", [
    (("layers", 0, "type"), "wkv", E.WR_ERR_UNSUPPORTED),               # another design's mixer
    (("layers", 0, "mlp", "kind"), "sparse", E.WR_ERR_UNSUPPORTED),
    (("norm", "eps"), None, E.WR_ERR_FORMAT),
    (MIX[0] + ("kv_heads",), 3, E.WR_ERR_FORMAT),                       # four heads over three
    (MIX[0] + ("rot",), None, E.WR_ERR_FORMAT),
    (MIX[0] + ("rot", "dims"), 5, E.WR_ERR_FORMAT),
    (MIX[0] + ("rot", "dims"), 12, E.WR_ERR_LIMIT),
    (MIX[0] + ("rot", "scaling"), None, E.WR_OK),
    (MIX[0] + ("rot", "scaling", "fast"), None, E.WR_ERR_FORMAT),
    (MIX[0] + ("rot", "scaling", "factor"), 0.0, E.WR_ERR_FORMAT),
    (MIX[0] + ("vdim",), 13, E.WR_ERR_FORMAT),                          # values that turn in pairs
    (MIX[0] + ("scale",), None, E.WR_ERR_FORMAT),
    (MIX[1] + ("left", "mask", "size"), 0, E.WR_ERR_LIMIT),
    (MIX[1] + ("left", "mask"), None, E.WR_ERR_FORMAT),
    (MIX[1] + ("left_scale",), None, E.WR_ERR_FORMAT),
    (MIX[1] + ("right_scale",), None, E.WR_ERR_FORMAT),
    (MIX[1] + ("right", "vdim"), None, E.WR_ERR_FORMAT),
    (MIX[1] + ("right", "dim"), 6, E.WR_ERR_FORMAT),                    # no tensor has that shape
    (MIX[1] + ("right", "dim"), 300, E.WR_ERR_LIMIT),
    (MIX[2] + ("right", "width"), None, E.WR_ERR_FORMAT),
    (MIX[2] + ("right",), None, E.WR_ERR_FORMAT),
    (MIX[2] + ("left", "heads"), 4, E.WR_ERR_FORMAT),
    (("layers", 0, "mlp", "limit"), None, E.WR_ERR_FORMAT),
    (("layers", 0, "mlp", "limit"), 0.0, E.WR_ERR_FORMAT),
    (("layers", 1, "mlp", "router", "top"), 6, E.WR_ERR_FORMAT),
    (("layers", 1, "mlp", "expert", "ff"), None, E.WR_ERR_FORMAT),
    (("layers", 1, "mlp"), None, E.WR_OK),
    (("layers", 2, "mlp"), None, E.WR_OK),
])
def test_configurations(eng, tmp_path, path, value, rc):
    assert _rc(eng, tmp_path, (path, value)) == rc


@pytest.mark.parametrize("name", [b"l0.mix.q.norm", b"l0.mix.k.norm", b"l0.mix.v.b", b"l0.mix.o.b", b"l0.mix.sink", b"l0.mlp.gate",
                                  b"l0.norm1", b"l1.mix.left.g", b"l1.mix.left.sink", b"l1.mix.right.f.b", b"l1.mix.right.lower",
                                  b"l1.mix.right.norm", b"l1.mlp.router", b"l1.mlp.e4.gate", b"l2.mix.left.k.b", b"l2.mix.left.out",
                                  b"l2.mix.right.out", b"l2.mix.right.z.b", b"l2.mix.right.g", b"l2.mix.right.o", b"final.norm", b"head"])
def test_missing_tensors(eng, tmp_path, name):
    assert _rc(eng, tmp_path, tensor=(b'"' + name + b'"', b'"' + name[:-1] + b'#"')) == E.WR_ERR_FORMAT
