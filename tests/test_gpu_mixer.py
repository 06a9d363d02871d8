"""Mixer-stack models on the device against the plain implementation of
tests/mixer_oracle.py: every test makes its own small model with random weights."""
import numpy as np
import pytest

from tests import mixer_oracle as O
from tests.mixer_util import Case, run_cut
from wayruntime_amd import engine as E, hipattn, mix_writer as mw

pytestmark = pytest.mark.gpu

@pytest.fixture(scope="module")
def eng():
    hipattn.shutdown()              # the engine owns the device library in this module
    e = E.Engine(E.HOST_SO)
    e.lib.wrh_debug_poison_scratch(1)
    yield e
    e.lib.wrh_debug_poison_scratch(0)
    e.close()


@pytest.fixture(params=["f32", "bf16"])
def prec(request):
    return request.param


LIGHT = mw.lightning(3, 24, 40, decay=[0.5, 0.95, 0.999])
LATENT = mw.latent_attention(5, 24, 40, q_rank=48, kv_rank=72, rot_dim=12, window=50, base=5000.0, scale=0.2)
WIDTH, VOCAB = 104, 211            # neither a multiple of 16

ONE_LAYER = {
    "lightning": [(LIGHT, None)],
    "lightning_odd": [(mw.lightning(3, 20, 44, decay=[0.5, 0.95, 0.999]), None)],
    "lightning_dim48": [(mw.lightning(4, 48, 64), None)],
    "lightning_dim72": [(mw.lightning(2, 72, 136, decay=[0.8, 0.9999]), None)],
    "lightning_dim128": [(mw.lightning(2, 128, 128), None)],
    "lightning_dim160": [(mw.lightning(2, 160, 24, decay=[0.9, 1.0]), None)],
    "lightning_wide_v": [(mw.lightning(1, 16, 200, decay=[0.97]), None)],
    "latent": [(LATENT, None)],
    "latent_rank512": [(mw.latent_attention(3, 32, 32, 64, 500, 64, window=70), None)],
    "latent_rank256": [(mw.latent_attention(20, 16, 16, 32, 250, 32, window=33), None)],
    "latent_rank64_33heads": [(mw.latent_attention(33, 8, 8, 32, 40, 40, window=1), None)],
    "latent_rank600": [(mw.latent_attention(2, 16, 48, 32, 600, 16, window=40), None)],
    "latent_rot80": [(mw.latent_attention(2, 16, 16, 32, 64, 80, window=1000), None)],
    "latent_no_rotation": [(mw.latent_attention(2, 16, 16, 32, 64, 0, window=30), None)],
    "dense": [(LIGHT, mw.dense(72))],
    "moe": [(LIGHT, mw.moe(7, 3, 40))],
    "moe_top1": [(LIGHT, mw.moe(5, 1, 24))],
    "moe_all": [(LATENT, mw.moe(4, 4, 32))],
    "moe_one": [(LATENT, mw.moe(1, 1, 32))],
}


@pytest.mark.parametrize("name", sorted(ONE_LAYER))
def test_one_mechanism(eng, tmp_path, prec, name):
    # whole prompt (chunked recurrence, matrix-core attention) and token by token
    case = Case(eng, tmp_path, mw.config(WIDTH, VOCAB, ONE_LAYER[name], eps=1e-5, logit_scale=0.7), prec)
    t = case.tokens(150)
    margins = []
    want = O.forward(case.cfg, case.w, t, np.float64, margins=margins)
    clear = np.ones(len(t), dtype=bool)
    if prec == "bf16" and margins:                         # (the experts come last here: a close call stays in its row)
        clear = margins[0] > 0.1
        assert clear.mean() > 0.7
    case.check(run_cut(case, t, [150])[clear], want[clear], name + " whole")
    case.check(run_cut(case, t, [83, 1])[clear], want[clear], name + " decoded")
    case.close()


def test_wide_rows(eng, tmp_path, prec):
    # more features than the row steps hold in registers; one expert's rows fill whole tiles
    cfg = mw.config(4200, 50, [(mw.lightning(1, 8, 8, decay=[0.9]), mw.moe(2, 1, 8)), (mw.lightning(1, 8, 8, decay=[0.9]), None)],
                    loop=(0, 2, 2))
    case = Case(eng, tmp_path, cfg, "f32" if prec == "f32" else "bf16")
    t = case.tokens(140)
    margins = []
    want = O.forward(case.cfg, case.w, t, np.float64, margins=margins)
    if prec == "bf16":                                     # up to the first close call
        close = np.flatnonzero(np.min(margins, axis=0) < 0.05)
        t = t[:close[0]] if close.size else t
        assert len(t) >= 5
    case.check(run_cut(case, t, [len(t)]), want[:len(t)], "wide whole")
    case.check(run_cut(case, t, [max(1, len(t) - 9), 1]), want[:len(t)], "wide decoded")
    case.close()


def stack(prec):
    """Several layers, part of them looped.  In bfloat16 every expert is used: a choice among random experts
    now and then hangs on less than bfloat16 resolves."""
    top = 2 if prec == "f32" else 6
    return mw.config(WIDTH, VOCAB, [(LIGHT, mw.dense(72)), (LATENT, mw.moe(6, top, 40)),
                                    (mw.lightning(2, 16, 48, decay=[0.7, 0.99]), None),
                                    (mw.latent_attention(4, 16, 24, 32, 64, 16, window=17, base=100.0), mw.dense(40))],
                     loop=(1, 3, 3), eps=1e-5, logit_scale=0.5)


def test_residual_after_every_layer_run(eng, tmp_path, prec):
    case = Case(eng, tmp_path, stack(prec), prec)
    t = case.tokens(21)
    cap = []
    O.forward(case.cfg, case.w, t, np.float64, cap)
    got = np.zeros((len(cap), len(t), WIDTH), dtype=np.float32)
    s = case.m.session()
    case.m.capture_residual(got)
    E.mixed_step([(s, t, [])])
    case.m.capture_residual(None)
    for i, want in enumerate(cap):
        case.check(got[i], want, f"run {i}", deep=True)
    s.close()
    case.close()


@pytest.mark.parametrize("cuts", [[2], [3, 5, 2, 1], [16, 17, 1, 64, 2], [63, 2, 65], [64], [100, 1], [17]])
def test_portions(eng, tmp_path, prec, cuts):
    case = Case(eng, tmp_path, stack(prec), prec)
    t = case.tokens(190)
    case.check(run_cut(case, t, cuts), case.oracle(t), f"cuts {cuts}", deep=True)
    case.close()


def test_loop_of_one_and_whole_stack(eng, tmp_path, prec):
    for loop in ((0, 2, 2), (1, 2, 1), (1, 1, 4), None):
        cfg = mw.config(64, 80, [(LIGHT, mw.dense(32)), (LATENT, None)], loop=loop)
        case = Case(eng, tmp_path, cfg, prec)
        t = case.tokens(40)
        case.check(run_cut(case, t, [30, 1]), case.oracle(t), f"loop {loop}")
        case.close()


def test_mixed_batches_and_reuse(eng, tmp_path, prec):
    # unequal requests side by side, portions beside single tokens, in a pool that
    # only holds the live ones: pages and slots are used again and again
    case = Case(eng, tmp_path, stack(prec), prec, pool=640, slots=3)
    rng = np.random.default_rng(5)
    todo = [case.tokens(n, seed=100 + i) for i, n in enumerate((150, 7, 90, 1, 130, 64, 65, 33, 170, 12))]
    want = [case.oracle(t) for t in todo]
    live, got, nxt = {}, [[] for _ in todo], 0
    while nxt < len(todo) or live:
        while nxt < len(todo) and len(live) < 3 and sum(-(-len(todo[i]) // 64) * 64 for i in [*live, nxt]) <= 640:
            live[nxt] = [case.m.session(), 0]
            nxt += 1
        entries, who = [], []
        for i, (s, at) in live.items():
            if len(live) > 1 and rng.random() < 0.2:
                continue                                   # left out of this step
            n = min(int(rng.choice([1, 1, 2, 5, 16, 17, 40, 70])), len(todo[i]) - at)
            entries.append((s, todo[i][at:at + n], list(range(n))))
            who.append((i, n))
        if not entries:
            continue
        rc, lg = E.mixed_step(entries)
        assert rc == sum(n for _, n in who)
        for (i, n), rows in zip(who, lg):
            got[i].append(rows)
            live[i][1] += n
            if live[i][1] == len(todo[i]):
                live.pop(i)[0].close()
    for i, t in enumerate(todo):
        case.check(np.concatenate(got[i]), want[i], f"request {i}", deep=True)
    case.close()


def _sharp(bits, cfg, query, key, gain):
    """Makes token `query` ask loudly for token `key`: the embeddings of both carry a feature of their own,
    the query latent picks one up and the shared rotated-free part of the key the other."""
    m = cfg["layers"][0]["mixer"]
    H, D, r = m["heads"], m["dim"], m["rot_dim"]
    f = {k: O.bf16_to_f32(v).copy() for k, v in bits.items()}
    f["embed"][:, :2] = 0
    f["embed"][query, 0] = f["embed"][key, 1] = 12.0
    f["l0.mix.dq"][0] = 0
    f["l0.mix.dq"][0, 0] = 1.0                             # query latent 0: "I am the query token"
    f["l0.mix.dkv"][0] = 0
    f["l0.mix.dkv"][0, 1] = 1.0                            # kv latent 0: "I am the key token"
    uq = f["l0.mix.uq"].reshape(H, D + r, -1)
    uk = f["l0.mix.uk"].reshape(H, D, -1)
    uq[:, 0] = 0
    uq[:, 0, 0] = gain
    uk[:, 0] = 0
    uk[:, 0, 0] = gain
    for k, v in f.items():
        bits[k] = O.f32_to_bf16(v)


@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 63, 64, 65, 97, 128, 150])
def test_window_edges(eng, tmp_path, prec, window):
    # one key that stands out, just inside and just outside the window of a row
    # that asks for it; queries in a prompt and decoded, the key on and beside page borders
    cfg = mw.config(64, 90, [(mw.latent_attention(3, 16, 16, 32, 48, 16, window=window, scale=0.5), None)])
    case = Case(eng, tmp_path, cfg, prec, edit=lambda b: _sharp(b, cfg, 7, 9, 3.0))
    for key_at in (0, 1, 62, 63, 64, 65):
        t = case.tokens(key_at + window + 4)
        t[(t == 7) | (t == 9)] = 11
        t[key_at] = 9
        inside, outside = key_at + window - 1, key_at + window
        if inside > key_at:
            t[inside] = 7
        t[outside] = t[outside + 1] = 7
        want = case.oracle(t)
        # the key really matters: without it the row that sees it changes
        if inside > key_at:
            u = t.copy()
            u[key_at] = 11
            far = case.oracle(u)
            assert np.abs(want[inside] - far[inside]).max() > 0.05 * np.abs(want[inside]).max()
            assert np.abs(want[outside] - far[outside]).max() < 1e-9
        case.check(run_cut(case, t, [len(t)]), want, f"window {window} key at {key_at} prompt")
        case.check(run_cut(case, t, [max(1, inside), 1]), want, f"window {window} key at {key_at} decoded")
        case.check(run_cut(case, t, [max(2, key_at + 1), 2]), want, f"window {window} key at {key_at} pairs")
    case.close()


@pytest.mark.parametrize("dist", [1, 15, 16, 17, 63, 64, 65, 200, 400])
def test_far_state(eng, tmp_path, prec, dist):
    # a token that writes loudly into a slow state and one that reads it far away
    cfg = mw.config(64, 90, [(mw.lightning(2, 16, 16, decay=[0.999, 0.3]), None)])

    def edit(bits):
        f = {k: O.bf16_to_f32(v).copy() for k, v in bits.items()}
        f["embed"][:, 0] = 0
        f["embed"][9, 0] = 10.0
        f["l0.mix.k"][0] = 0
        f["l0.mix.k"][0, 0] = 2.0                          # head 0, state row 0: written by token 9 alone
        for k, v in f.items():
            bits[k] = O.f32_to_bf16(v)

    case = Case(eng, tmp_path, cfg, prec, edit=edit)
    t = case.tokens(dist + 3)
    t[t == 9] = 11
    t[1] = 9
    u = t.copy()
    u[1] = 11
    want, without = case.oracle(t), case.oracle(u)
    assert np.abs(want[1 + dist] - without[1 + dist]).max() > 0.02 * np.abs(want[1 + dist]).max()
    for cuts in ([len(t)], [2, 1], [len(t) - 2, 1], [2, 70]):
        case.check(run_cut(case, t, cuts), want, f"distance {dist} cuts {cuts}")
    case.close()


def test_long_decoding(eng, tmp_path, prec):
    case = Case(eng, tmp_path, stack(prec), prec)
    t = case.tokens(420)
    case.check(run_cut(case, t, [3, 1]), case.oracle(t), "417 decoded tokens", deep=True)
    case.close()


def test_prompt_longer_than_one_pass(eng, tmp_path, prec):
    # more rows than one device pass takes (4096): the step runs in passes
    cfg = mw.config(32, 64, [(mw.lightning(2, 8, 8, decay=[0.9, 0.9999]), None),
                             (mw.latent_attention(2, 8, 8, 16, 32, 8, window=40), mw.moe(4, 2, 16))])
    case = Case(eng, tmp_path, cfg, prec, pool=8192)
    t = case.tokens(4500)
    s, other = case.m.session(), case.m.session()
    places = [0, 1, 4000, 4094, 4095, 4096, 4097, 4163, 4499]
    rc, lg = E.mixed_step([(s, t[:4400], [p for p in places if p < 4400]), (other, t[:30], [29])])
    assert rc == 9
    want = case.oracle(t)
    case.check(lg[0], want[[p for p in places if p < 4400]], "passes")
    case.check(lg[1], want[[29]], "beside it")
    rc, lg = E.mixed_step([(s, t[4400:], [99])])
    case.check(lg[0], want[[4499]], "after the passes")
    s.close()
    other.close()
    case.close()


def test_greedy_generation(eng, tmp_path):
    # wr_prefill, wr_step and wr_batch_step against the oracle's own greedy streams (32-bit: no ties to lose)
    case = Case(eng, tmp_path, stack("f32"), "f32")
    prompts = [case.tokens(n, seed=n) for n in (5, 40, 70)]
    want = []
    for p in prompts:
        t = list(p)
        for _ in range(12):
            t.append(int(case.oracle(t)[-1].argmax()))
        want.append(t[len(p):])
    s = case.m.session()
    assert s.prefill(prompts[1][:-1]) == 39
    tok, got = int(prompts[1][-1]), []
    for _ in range(12):
        tok = int(s.step(tok).argmax())
        got.append(tok)
    assert got == want[1]
    s.close()
    ss = [case.m.session() for _ in prompts]
    for x, p in zip(ss, prompts):
        assert x.prefill(p[:-1]) == len(p) - 1
    feed, got = [int(p[-1]) for p in prompts], []
    for _ in range(12):
        rc, lg = E.batch_step(ss, feed)
        assert rc == 3
        feed = [int(x.argmax()) for x in lg]
        got.append(feed)
    assert [list(x) for x in zip(*got)] == want
    assert [x.pos for x in ss] == [len(p) + 11 for p in prompts]
    for x in ss:
        x.close()
    case.close()


def test_failed_step_changes_nothing(eng, tmp_path, prec):
    case = Case(eng, tmp_path, stack(prec), prec)
    t = case.tokens(100)
    want = case.oracle(t)
    s = case.m.session()
    rc, a = E.mixed_step([(s, t[:60], range(60))])
    for run in (0, 3, 7):
        s.lib.wrh_debug_fail_attention_at(run)
        rc, _ = E.mixed_step([(s, t[60:90], [0])])
        assert rc == E.WR_ERR_INTERNAL and s.pos == 60 and s.status == E.WR_ERR_INTERNAL
    rc, b = E.mixed_step([(s, t[60:], range(40))])
    assert rc == 40
    case.check(np.concatenate([a[0], b[0]]), want, "after failures", deep=True)
    s.close()
    case.close()
