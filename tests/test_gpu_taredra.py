"""Pre-norm mixer-stack models (architecture "Taredra") on the device against the plain
implementation of tests/mixer_oracle.py: every test makes its own small model with
random weights."""
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


def f32_edit(change):
    """An edit of a model's tensors as floats."""
    def edit(bits):
        f = {k: O.bf16_to_f32(v).copy() for k, v in bits.items()}
        change(f)
        for k, v in f.items():
            bits[k] = O.f32_to_bf16(v)
    return edit


WIDTH, VOCAB = 104, 211            # neither a multiple of 16
PAR = mw.window_and_delta(6, 3, 24, 40, window=37, right_heads=3, right_dim=20, rot_dims=12, base=5000.0, scale=0.3,
                          left_scale=0.8, right_scale=1.3)


def par(left=None, right=(2, 16), **kw):
    """Attention (heads, kv_heads, dim, vdim, window) beside a recurrence (heads, dim)."""
    h, g, d, v, w = left or (2, 1, 16, 16, 25)
    return mw.window_and_delta(h, g, d, v, window=w, right_heads=right[0], right_dim=right[1], **kw)


LEFT = dict(left_scale=1.0, right_scale=0.0)
RIGHT = dict(left_scale=0.0, right_scale=1.0)
ONE_LAYER = {
    "wkv_dim16": [(mw.wkv(5, 16), None)],
    "wkv_dim7": [(mw.wkv(3, 7), None)],
    "wkv_dim20": [(mw.wkv(3, 20), None)],
    "wkv_dim32": [(mw.wkv(1, 32), None)],
    "wkv_dim48": [(mw.wkv(3, 48), None)],
    "wkv_dim64": [(mw.wkv(2, 64), None)],
    "wkv_dim100": [(mw.wkv(2, 100), None)],
    "wkv_dim128": [(mw.wkv(2, 128), None)],
    "wkv_dim160": [(mw.wkv(1, 160), None)],
    "wkv_dim256": [(mw.wkv(1, 256), None)],
    "delta_dim8": [(par(right=(4, 8), **RIGHT), None)],
    "delta_dim20": [(par(right=(3, 20), **RIGHT), None)],
    "delta_dim32": [(par(right=(2, 32), **RIGHT), None)],
    "delta_dim45": [(par(right=(2, 45), **RIGHT), None)],
    "delta_dim64": [(par(right=(1, 64), **RIGHT), None)],
    "delta_dim96": [(par(right=(2, 96), **RIGHT), None)],
    "delta_dim128": [(par(right=(2, 128), **RIGHT), None)],
    "delta_dim200": [(par(right=(1, 200), **RIGHT), None)],
    "window": [(par((6, 3, 24, 40, 37), rot_dims=12, scale=0.3, **LEFT), None)],
    "window_no_rotation": [(par((4, 2, 32, 32, 50), rot_dims=0, **LEFT), None)],
    "window_one_head": [(par((1, 1, 10, 6, 64), rot_dims=4, **LEFT), None)],
    "window_every_head_its_own": [(par((3, 3, 64, 64, 65), **LEFT), None)],
    "window_20_heads_on_one": [(par((20, 1, 16, 24, 33), **LEFT), None)],
    "window_40_heads_on_two": [(par((80, 2, 8, 8, 1000), **LEFT), None)],
    "window_dim128": [(par((4, 2, 128, 100, 90), rot_dims=64, **LEFT), None)],
    "window_dim100_v30": [(par((4, 1, 100, 30, 40), **LEFT), None)],
    "window_dim30_v128": [(par((2, 1, 30, 128, 40), **LEFT), None)],
    "window_dim160": [(par((2, 1, 160, 24, 40), **LEFT), None)],
    "window_v200": [(par((2, 2, 16, 200, 40), **LEFT), None)],
    "window_of_one": [(par((4, 2, 16, 16, 1), **LEFT), None)],
    "both": [(PAR, None)],
    "dense": [(par(left_scale=0.1, right_scale=0.1), mw.dense(72))],
    "wkv_dense": [(mw.wkv(2, 16), mw.dense(40))],
}


@pytest.mark.parametrize("name", sorted(ONE_LAYER))
def test_one_mechanism(eng, tmp_path, prec, name):
    # whole prompt (chunked recurrence, matrix-core attention) and token by token
    case = Case(eng, tmp_path, mw.prenorm_config(WIDTH, VOCAB, ONE_LAYER[name], eps=1e-5, embed_scale=3.0), prec)
    t = case.tokens(150)
    want = case.oracle(t)
    case.check(run_cut(case, t, [150]), want, name + " whole")
    case.check(run_cut(case, t, [83, 1]), want, name + " decoded")
    case.close()


def test_wide_rows(eng, tmp_path, prec):
    # more features than the row steps hold in registers
    cfg = mw.prenorm_config(4200, 50, [(mw.wkv(1, 8), mw.dense(8)), (par(), None), (mw.wkv(1, 8), None)])
    case = Case(eng, tmp_path, cfg, prec)
    t = case.tokens(100)
    want = case.oracle(t)
    case.check(run_cut(case, t, [100]), want, "wide whole")
    case.check(run_cut(case, t, [91, 1]), want, "wide decoded")
    case.close()


def stack():
    return mw.prenorm_config(WIDTH, VOCAB, [(PAR, mw.dense(72)), (mw.wkv(3, 24), None), (mw.wkv(2, 16), mw.dense(40)),
                                            (par((4, 2, 16, 32, 17), right=(2, 40), base=100.0), None),
                                            (par((8, 1, 64, 64, 70), right=(1, 64), left_scale=1.2, right_scale=0.7), mw.dense(64))],
                             eps=1e-5)


@pytest.mark.parametrize("first", [0, 1, 3])
def test_residual_after_every_layer(eng, tmp_path, prec, first):
    # layers of both kinds ahead of and behind each other, a different one first each time
    cfg = stack()
    cfg["layers"] = cfg["layers"][first:] + cfg["layers"][:first]
    case = Case(eng, tmp_path, cfg, prec)
    t = case.tokens(21)
    cap = []
    O.forward(case.cfg, case.w, t, np.float64, cap)
    got = np.zeros((len(cap), len(t), WIDTH), dtype=np.float32)
    s = case.m.session()
    case.m.capture_residual(got)
    E.mixed_step([(s, t, [])])
    case.m.capture_residual(None)
    for i, want in enumerate(cap):
        case.check(got[i], want, f"layer {i}")
    s.close()
    case.check(run_cut(case, t, [21]), case.oracle(t), "logits")
    case.close()


@pytest.mark.parametrize("cuts", [[2], [3, 5, 2, 1], [16, 17, 1, 64, 2], [63, 2, 65], [64], [100, 1], [17], [33, 31, 18, 2]])
def test_portions(eng, tmp_path, prec, cuts):
    case = Case(eng, tmp_path, stack(), prec)
    t = case.tokens(190)
    case.check(run_cut(case, t, cuts), case.oracle(t), f"cuts {cuts}")
    case.close()


def test_mixed_batches_and_reuse(eng, tmp_path, prec):
    # unequal requests side by side, portions beside single tokens, in a pool that
    # only holds the live ones: pages and slots are used again and again
    case = Case(eng, tmp_path, stack(), prec, pool=640, slots=3)
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
        case.check(np.concatenate(got[i]), want[i], f"request {i}")
    case.close()


def _sharp(cfg, query, key, gain):
    """Makes token `query` ask loudly for token `key`: the embeddings of both carry a feature of their own, which the
    unrotated last dimension of every query and key picks up."""
    m = cfg["layers"][0]["mixer"]["left"]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]

    def change(f):
        f["embed"][:, :2] = 0
        f["embed"][query, 0] = f["embed"][key, 1] = 1.5
        q, k = f["l0.mix.left.q"].reshape(H, D, -1), f["l0.mix.left.k"].reshape(G, D, -1)
        q[:, -1] = k[:, -1] = 0
        q[:, -1, 0] = k[:, -1, 1] = gain
    return f32_edit(change)


@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 63, 64, 65, 97, 128, 150])
def test_window_edges(eng, tmp_path, prec, window):
    # one key that stands out, just inside and just outside the window of a row
    # that asks for it; queries in a prompt and decoded, the key on and beside page borders
    cfg = mw.prenorm_config(64, 90, [(par((4, 2, 16, 16, window), rot_dims=8, scale=0.5, left_scale=2.0), None)])
    case = Case(eng, tmp_path, cfg, prec, edit=_sharp(cfg, 7, 9, 3.0))
    for key_at in (0, 1, 62, 63, 64, 65):
        t = case.tokens(key_at + window + 4)
        t[(t == 7) | (t == 9)] = 11
        t[key_at] = 9
        inside, outside = key_at + window - 1, key_at + window
        if inside > key_at:
            t[inside] = 7
        t[outside] = t[outside + 1] = 7
        want = case.oracle(t)
        if inside > key_at:
            # the key really matters to the row that sees it, through the attention
            cut = {**case.cfg, "layers": [{**case.cfg["layers"][0], "mixer": {**case.cfg["layers"][0]["mixer"], "right_scale": 0.0}}]}
            u = t.copy()
            u[key_at] = 11
            a, b = O.forward(cut, case.w, t, np.float64), O.forward(cut, case.w, u, np.float64)
            assert np.abs(a[inside] - b[inside]).max() > 0.05 * np.abs(a[inside]).max()
            assert np.abs(a[outside] - b[outside]).max() < 1e-9
        case.check(run_cut(case, t, [len(t)]), want, f"window {window} key at {key_at} prompt")
        case.check(run_cut(case, t, [max(1, inside), 1]), want, f"window {window} key at {key_at} decoded")
        case.check(run_cut(case, t, [max(2, key_at + 1), 2]), want, f"window {window} key at {key_at} pairs")
    case.close()


@pytest.mark.parametrize("sink", [-30.0, 0.0, 6.0, 40.0])
def test_sinks(eng, tmp_path, prec, sink):
    # from no weight at all to nearly all of it; windows long and short, more heads than one tile
    cfg = mw.prenorm_config(64, 90, [(par((20, 1, 16, 16, 300), scale=1.0, left_scale=2.0), None), (par((2, 2, 16, 16, 3)), None)])

    def change(f):
        f["l0.mix.left.sink"][:] = sink + np.linspace(-1, 1, 20)
        f["l1.mix.left.sink"][:] = sink
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(260)
    want = case.oracle(t)
    if sink == 6.0:                                        # leaving it out would show
        bare = O.forward(cfg, {k: v - 100 if k.endswith("sink") else v for k, v in case.w.items()}, t, np.float64)
        assert np.median(np.abs(bare - want).max(axis=1) / np.abs(want).max(axis=1)) > 0.1
    case.check(run_cut(case, t, [260]), want, f"sink {sink} prompt")
    case.check(run_cut(case, t, [130, 1]), want, f"sink {sink} decoded")
    case.close()


@pytest.mark.parametrize("kind", ["wkv", "delta"])
@pytest.mark.parametrize("dist", [1, 2, 15, 16, 17, 63, 64, 65, 200, 400])
def test_far_state(eng, tmp_path, prec, kind, dist):
    # a token that writes loudly into a channel that keeps it, and one that reads it far away
    mixer = mw.wkv(2, 16) if kind == "wkv" else par((1, 1, 8, 8, 1), right=(2, 16), left_scale=0.1)
    cfg = mw.prenorm_config(64, 90, [(mixer, None)])
    p = "l0.mix." if kind == "wkv" else "l0.mix.right."

    def change(f):
        f["embed"][:, 0] = 0
        f["embed"][9, 0] = 3.0
        f[p + "k"][0] = 0
        f[p + "k"][0, 0] = 4.0                             # head 0, channel 0: written by token 9 alone
        f[p + "w0"][0] = -9.0                              # and kept
        f[p + "w2"][0] = 0
        f[p + "r"][0] *= 4.0
        f[p + "o"][:] *= 3.0
        if kind == "delta":
            f[p + "a.b"][:16] = -9.0
        else:
            f["l0.mix.mu.k"][:] = 0.0
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(dist + 3)
    t[t == 9] = 11
    t[1] = 9
    u = t.copy()
    u[1] = 11
    want, without = case.oracle(t), case.oracle(u)
    shown = [np.abs(want[p] - without[p]).max() / np.abs(want[p]).max() for p in (dist, 1 + dist, 2 + dist)]
    assert max(shown) > 0.02, shown
    for cuts in ([len(t)], [2, 1], [len(t) - 2, 1], [2, 70]):
        case.check(run_cut(case, t, cuts), want, f"{kind} distance {dist} cuts {cuts}")
    case.close()


@pytest.mark.parametrize("w0", [-14.0, -6.0, 0.0, 2.0, 5.0])
def test_decays_from_none_to_all(eng, tmp_path, prec, w0):
    # wkv decays from 1 - 1e-6 down to exp(-exp(5)), neighbouring channels far apart
    cfg = mw.prenorm_config(64, 90, [(mw.wkv(2, 32), None), (par(right=(2, 32)), None)])

    def change(f):
        f["l0.mix.w0"][:] = w0
        f["l0.mix.w0"][::3] = -w0
        f["l1.mix.right.w0"][:] = w0
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(230)
    want = case.oracle(t)
    case.check(run_cut(case, t, [230]), want, f"w0 {w0} prompt")
    case.check(run_cut(case, t, [40, 50, 3, 1]), want, f"w0 {w0} cut")
    case.close()


@pytest.mark.parametrize("dim", [12, 32, 60, 100, 128])
@pytest.mark.parametrize("kind", ["wkv", "delta"])
def test_long_prompts_walked_in_segments(eng, tmp_path, prec, kind, dim):
    # prompts long enough for several segments, unequal ones side by side, and one that goes on from a state;
    # decays slow enough for every segment to matter to the last
    mixer = mw.wkv(2, dim) if kind == "wkv" else par((1, 1, 8, 8, 1), right=(2, dim), left_scale=0.1)
    cfg = mw.prenorm_config(48, 90, [(mixer, None)])

    def change(f):
        p = "l0.mix." if kind == "wkv" else "l0.mix.right."
        f[p + "w0"][:] = -7.0 + np.linspace(0, 3, 2 * dim)
        if kind == "delta":
            f[p + "a.b"][:] = np.linspace(-6, 1, 2 * dim)
    case = Case(eng, tmp_path, cfg, prec, pool=2048, edit=f32_edit(change))
    t, u = case.tokens(900), case.tokens(330, seed=8)
    want, other = case.oracle(t), case.oracle(u)
    a, b = case.m.session(), case.m.session()
    rc, lg = E.mixed_step([(a, t[:617], range(617)), (b, u, range(330))])
    assert rc == 947
    case.check(lg[0], want[:617], f"{kind} {dim} beside a shorter one")
    case.check(lg[1], other, f"{kind} {dim} the shorter one")
    rc, lg = E.mixed_step([(a, t[617:], range(283))])
    case.check(lg[0], want[617:], f"{kind} {dim} going on")
    a.close()
    b.close()
    case.check(run_cut(case, t, [880, 1]), want, f"{kind} {dim} decoded behind it")
    case.close()


def test_repeated_keys_are_removed(eng, tmp_path, prec):
    # the same few tokens over and over: unit keys repeat, removal and unit norms carry the outcome;
    # one token's key is all but zero
    cfg = mw.prenorm_config(64, 30, [(par((1, 1, 8, 8, 1), right=(2, 24), left_scale=0.1, right_scale=2.0), None)])

    def change(f):
        f["l0.mix.right.a.b"][:] = 3.0
        f["embed"][:, 5] = 0
        f["embed"][3] = 0
        f["embed"][3, 5] = 1.0
        f["l0.mix.right.k"][:, 5] = 1e-5                   # token 3: |k| of the unit norm's own epsilon
        f["l0.mix.right.w0"][:] = -8.0
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = np.resize([4, 7, 3, 4, 4, 9], 200)
    want = case.oracle(t)
    for cuts in ([200], [50, 1], [16, 17, 30]):
        case.check(run_cut(case, t, cuts), want, f"repeats, cuts {cuts}")
    case.close()


def test_token_shift_over_every_border(eng, tmp_path, prec):
    # mixes that take the previous token alone: a border that loses it shows at once
    cfg = mw.prenorm_config(72, 90, [(mw.wkv(2, 16), None), (mw.wkv(2, 16), None)])

    def change(f):
        for n in "rkvgw":
            f["l0.mix.mu." + n][:] = 1.0
            f["l1.mix.mu." + n][:] = 1.0
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(140)
    want = case.oracle(t)
    for cuts in ([140], [1], [2], [64], [65, 63, 2], [17, 1, 16]):
        case.check(run_cut(case, t, cuts), want, f"cuts {cuts}")
    case.close()


def test_long_decoding(eng, tmp_path, prec):
    case = Case(eng, tmp_path, stack(), prec)
    t = case.tokens(420)
    case.check(run_cut(case, t, [3, 1]), case.oracle(t), "417 decoded tokens")
    case.close()


def test_long_window_decoding_splits_its_keys(eng, tmp_path):
    # one decoded row over thousands of keys: many shares, the sink in the first alone
    cfg = mw.prenorm_config(32, 64, [(par((4, 2, 16, 16, 3000), scale=1.0), None)])
    case = Case(eng, tmp_path, cfg, "bf16", pool=4096)
    t = case.tokens(3400)
    s = case.m.session()
    assert s.prefill(t[:3390]) == 3390
    got = np.stack([s.step(int(x)) for x in t[3390:]])
    s.close()
    case.check(got, case.oracle(t)[3390:], "decoded behind 3390")
    case.close()


def test_prompt_longer_than_one_pass(eng, tmp_path, prec):
    # more rows than one device pass takes (4096): the step runs in passes
    cfg = mw.prenorm_config(32, 64, [(mw.wkv(2, 8), None), (par((2, 1, 8, 8, 40), right=(2, 8)), mw.dense(16))])
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


def test_sixteen_requests(eng, tmp_path, prec):
    case = Case(eng, tmp_path, stack(), prec, pool=4096, slots=16)
    todo = [case.tokens(n, seed=n) for n in range(5, 165, 10)]
    ss = [case.m.session() for _ in todo]
    E.mixed_step([(s, t[:-3], []) for s, t in zip(ss, todo)])
    for k in (-3, -2, -1):
        rc, lg = E.batch_step(ss, [int(t[k]) for t in todo])
        assert rc == 16
        for t, row in zip(todo, lg):
            case.check(row[None], case.oracle(t)[[k]], f"request of {len(t)}")
    for s in ss:
        s.close()
    case.close()


def test_greedy_generation(eng, tmp_path):
    # wr_prefill, wr_step and wr_batch_step against the oracle's own greedy streams (32-bit: no ties to lose)
    case = Case(eng, tmp_path, stack(), "f32")
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
    for x in ss:
        x.close()
    case.close()


def test_failed_step_changes_nothing(eng, tmp_path, prec):
    case = Case(eng, tmp_path, stack(), prec)
    t = case.tokens(100)
    want = case.oracle(t)
    s = case.m.session()
    rc, a = E.mixed_step([(s, t[:60], range(60))])
    for run in (0, 2, 4):
        s.lib.wrh_debug_fail_attention_at(run)
        rc, _ = E.mixed_step([(s, t[60:90], [0])])
        assert rc == E.WR_ERR_INTERNAL and s.pos == 60 and s.status == E.WR_ERR_INTERNAL
    rc, b = E.mixed_step([(s, t[60:], range(40))])
    assert rc == 40
    case.check(np.concatenate([a[0], b[0]]), want, "after failures")
    s.close()
    case.close()
