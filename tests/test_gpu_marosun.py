"""Mixer-stack models whose layers' mixers and feed-forward read one norm (architecture
"Marosun") on the device against the plain implementation of tests/mixer_oracle.py: every
test makes its own small model with random weights."""
import numpy as np
import pytest

from tests import mixer_oracle as O
from tests.mixer_util import Case, f32_edit, run_cut
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


def differs(a, b, least=0.05):
    """Most rows of two sets of logits differ by at least that much of their largest element."""
    return np.median(np.abs(a - b).max(axis=1) / np.abs(a).max(axis=1)) > least


WIDTH, VOCAB = 104, 211            # neither a multiple of 16
T, C, G = mw.turned_values, mw.chunks_and_forget, mw.one_more_and_gru
SOLO = {
    "turned": T(6, 3, 24, 36, rot_dims=12, base=5000.0, scale=0.3, scaling=(3.0, 64, 4.0, 0.5)),
    "turned_not_scaled": T(4, 2, 32, 32, scaling=None),
    "turned_no_rotation": T(4, 2, 32, 30, rot_dims=0),
    "turned_all_rotated": T(4, 4, 40, 40, scale=1.0, scaling=(8.0, 100, 8.0, 1.0)),
    "turned_one_head": T(1, 1, 10, 6, rot_dims=4),
    "turned_20_heads_on_one": T(20, 1, 16, 24, rot_dims=2),
    "turned_dim100_v90": T(4, 2, 100, 90, rot_dims=50),
    "turned_dim128": T(2, 1, 128, 128),
    "turned_dim160_v20": T(2, 1, 160, 20, rot_dims=70),
    "turned_v2": T(3, 3, 8, 2),
    "turned_v200": T(2, 1, 16, 200),
    "chunks": C(6, 3, 24, 36, 37, 3, 10, 14, scale=0.3, left_scale=0.7, right_scale=1.3),
    "chunks_one_head": C(1, 1, 10, 5, 64, 1, 1, 1),
    "chunks_of_one": C(4, 2, 16, 16, 1, 2, 16, 16),
    "chunks_of_everything": C(4, 1, 64, 64, 1000, 2, 32, 32, right_scale=0.5),
    "chunks_20_heads_on_one": C(20, 1, 16, 24, 50, 5, 7, 40),
    "chunks_dim128_v96": C(2, 2, 128, 96, 70, 2, 64, 100, left_scale=-1.0),
    "chunks_dim160_v7": C(2, 1, 160, 7, 33, 2, 100, 30),
    "forget_128x128": C(1, 1, 8, 8, 9, 2, 128, 128),
    "forget_130x20": C(1, 1, 8, 8, 9, 2, 130, 20),
    "forget_20x130": C(1, 1, 8, 8, 9, 2, 20, 130),
    "forget_250x256": C(1, 1, 8, 8, 9, 1, 250, 256),
    "forget_40x200": C(1, 1, 8, 8, 9, 3, 40, 200),
    "forget_left_off": C(2, 1, 8, 8, 9, 2, 24, 20, left_scale=0.0, right_scale=2.0),
    "gru": G(6, 3, 24, 36, 70, rot_dims=12, base=5000.0, scale=0.3),
    "gru_one": G(1, 1, 10, 6, 1, rot_dims=4),
    "gru_32": G(4, 4, 32, 32, 32),
    "gru_wider": G(4, 2, 64, 64, 300),
    "gru_no_rotation": G(4, 2, 16, 30, 33, rot_dims=0),
    "gru_dim160": G(2, 1, 160, 20, 40, rot_dims=100),
    "gru_20_heads_on_one": G(20, 1, 16, 24, 50, rot_dims=2),
}


@pytest.mark.parametrize("name", sorted(SOLO))
def test_one_mixer(eng, tmp_path, prec, name):
    # whole prompt, token by token behind a prompt, and in portions
    case = Case(eng, tmp_path, mw.joint_config(WIDTH, VOCAB, [(SOLO[name], None)], eps=1e-5), prec)
    t = case.tokens(150)
    want = case.oracle(t)
    for cuts in ([150], [83, 1], [40, 2, 17, 5, 64]):
        # (a norm over one element is its sign: small sums may turn it in bfloat16)
        case.check(run_cut(case, t, cuts), want, f"{name} cuts {cuts}", deep=name in ("chunks_one_head", "gru_one"))
    case.close()


CHEAP = T(2, 1, 8, 8)
MLPS = {
    "dense": mw.clamped_dense(72, 1.0),
    "dense_tight": mw.clamped_dense(8, 0.1),
    "dense_wide_open": mw.clamped_dense(300, 50.0),
    "dense_one": mw.clamped_dense(1, 0.7),
    "top_one": mw.moe(6, 1, 40),
    "some": mw.moe(7, 3, 24),
    "one_expert": mw.moe(1, 1, 24),
    "all": mw.moe(5, 5, 8),
    "many": mw.moe(150, 9, 8),
}


def check_clear(case, t, name, cuts_list):
    """Compares rows whose expert choice is no close call (in bfloat16 a close call may fall either way, and the experts
    come last here, so it stays in its row)."""
    margins = []
    want = O.forward(case.cfg, case.w, t, np.float64, margins=margins)
    clear = np.ones(len(t), dtype=bool)
    if case.prec == "bf16" and margins:
        clear = margins[-1] > 0.06
        assert clear.mean() > 0.2, clear.mean()
    for cuts in cuts_list:
        case.check(run_cut(case, t, cuts)[clear], want[clear], f"{name} cuts {cuts}")


@pytest.mark.parametrize("beside", ["attention", "parallel", "parallel_2"])
@pytest.mark.parametrize("name", sorted(MLPS))
def test_one_feed_forward(eng, tmp_path, prec, name, beside):
    # every feed-forward beside every mixer: they share products, and what joins the residual differs
    mixer = {"attention": CHEAP, "parallel": C(2, 1, 8, 8, 9, 2, 8, 6), "parallel_2": G(2, 1, 8, 8, 20)}[beside]
    case = Case(eng, tmp_path, mw.joint_config(WIDTH, VOCAB, [(mixer, MLPS[name])], eps=1e-5), prec)
    check_clear(case, case.tokens(120), name, ([120], [83, 1], [30, 20, 7, 2]))
    case.close()


def test_feed_forward_tiles(eng, tmp_path, prec):
    # enough rows that every expert's fill whole tiles in bfloat16, one expert without any
    cfg = mw.joint_config(96, VOCAB, [(CHEAP, mw.moe(6, 3, 72))])

    def change(f):
        f["embed"][:, 0] = 2.0                             # a feature that every token has keeps expert 2 out
        f["l0.mlp.router"][:, 0] = 0.0
        f["l0.mlp.router"][2, 0] = -2.5
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    check_clear(case, case.tokens(520), "tiles", ([520], [300, 220], [455, 65]))
    case.close()


@pytest.mark.parametrize("kind", ["weight_on_the_output", "renormed", "softmax", "gate_not_clamped", "up_not_clamped", "no_plus_one"])
def test_feed_forward_details_show(eng, tmp_path, prec, kind, monkeypatch):
    # what each mistake there would do, made in the plain implementation, is far from what the device gives
    dense = kind in ("gate_not_clamped", "up_not_clamped", "no_plus_one")
    cfg = mw.joint_config(64, 90, [(CHEAP, mw.clamped_dense(40, 0.5) if dense else mw.moe(6, 2, 40))])

    def change(f):
        for k in f:
            if k.endswith("down"):
                f[k] *= 3
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(110)
    want = case.oracle(t)
    with monkeypatch.context() as mp:
        if dense:
            def unit(h, w, limit):
                g, u = h @ w["gate"].T, h @ w["up"].T
                if kind != "gate_not_clamped":
                    g = np.minimum(g, limit)
                if kind != "up_not_clamped":
                    u = np.clip(u, -limit, limit)
                return (g * O.sigmoid(1.702 * g) * (u + (kind != "no_plus_one"))) @ w["down"].T
            mp.setattr(O, "clamped_expert", unit)
        elif kind == "weight_on_the_output":
            def outside(h, w, cfg):
                out = np.zeros_like(h)
                for i in range(len(h)):
                    for e, s in zip(*O.logistic_choice(w["router"] @ h[i], 2)):
                        out[i] += s * O.dense_mlp(h[i], O._sub(w, f"e{e}."))
                return out
            mp.setattr(O, "weighted_input_moe", outside)
        else:
            right = O.logistic_choice

            def other(z, top):
                chosen, s = right(z, top)
                if kind == "renormed":
                    return chosen, s / s.sum()
                return chosen, (np.exp(z) / np.exp(z).sum())[chosen]
            mp.setattr(O, "logistic_choice", other)
        wrong = O.forward(cfg, case.w, t, np.float64)
    assert differs(want, wrong)
    check_clear(case, t, kind, ([110], [50, 1]))
    case.close()


def test_wide_rows(eng, tmp_path, prec):
    # more features than the row steps hold in registers
    cfg = mw.joint_config(4200, 50, [(G(2, 1, 8, 8, 40), mw.moe(3, 3, 8)), (G(1, 1, 8, 8, 9), mw.clamped_dense(16)),
                                     (CHEAP, mw.moe(2, 2, 8)), (G(1, 1, 8, 8, 9), None)])
    case = Case(eng, tmp_path, cfg, prec)
    t = case.tokens(100)
    want = case.oracle(t)
    case.check(run_cut(case, t, [100]), want, "wide whole", deep=True)
    case.check(run_cut(case, t, [91, 1]), want, "wide decoded", deep=True)
    case.close()


def stack(prec="f32"):
    """All mixers, several rotations, layers without a feed-forward.  In bfloat16 every expert is chosen: a choice among
    random experts now and then hangs on less than bfloat16 resolves."""
    def moe(experts, top, ff):
        return mw.moe(experts, experts if prec == "bf16" else top, ff)
    s = dict(base=3000.0, scaling=(4.0, 48, 5.0, 0.5))
    return mw.joint_config(WIDTH, VOCAB, [
        (T(4, 2, 24, 40, rot_dims=10, **s), mw.clamped_dense(72, 1.0)),
        (C(6, 2, 32, 24, 50, 2, 20, 36, left_scale=0.8, right_scale=1.1), moe(5, 2, 24)),
        (G(4, 2, 24, 16, 90, rot_dims=8, base=100.0), mw.clamped_dense(40, 0.5)),
        (T(6, 1, 16, 16, base=100.0, scaling=None), moe(4, 1, 40)),
        (G(3, 3, 16, 24, 40, rot_dims=16, base=3000.0), moe(3, 2, 16)),
        (C(2, 1, 16, 40, 70, 4, 48, 8), None),
        (T(2, 2, 40, 24, rot_dims=24, **s), None),
        (C(3, 3, 24, 16, 9, 1, 40, 40, left_scale=1.5, right_scale=0.6), mw.clamped_dense(24, 2.0))], eps=1e-5)


@pytest.mark.parametrize("first", [0, 1, 2])
def test_residual_after_every_layer(eng, tmp_path, prec, first):
    cfg = stack(prec)
    if first:                                              # a different layer ahead of the others
        cfg["layers"] = [cfg["layers"][i] for i in ((1, 4, 0, 7), (2, 5, 3, 1))[first - 1]]
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
        case.check(got[i], want, f"layer {i}", deep=True)
    s.close()
    case.check(run_cut(case, t, [21]), case.oracle(t), "logits", deep=True)
    case.close()


@pytest.mark.parametrize("cuts", [[2], [3, 5, 2, 1], [16, 17, 1, 64, 2], [63, 2, 65], [64], [100, 1], [17], [33, 31, 18, 2]])
def test_portions(eng, tmp_path, prec, cuts):
    case = Case(eng, tmp_path, stack(prec), prec)
    t = case.tokens(190)
    case.check(run_cut(case, t, cuts), case.oracle(t), f"cuts {cuts}", deep=True)
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


def sharp(cfg, query, key, gain):
    """Makes token `query` ask loudly for token `key`: the embeddings of both carry a feature of their own, which the
    last (unrotated) dimension of every query and key picks up."""
    def change(f):
        f["embed"][:, :2] = 0
        f["embed"][query, 0] = f["embed"][key, 1] = 1.5
        for i, c in enumerate(cfg["layers"]):
            p = f"l{i}.mix." if c["type"] == "attention" else f"l{i}.mix.left."
            for n, feature in (("q", 0), ("k", 1)):
                D = (c["mixer"] if c["type"] == "attention" else c["mixer"]["left"])["dim"]
                x = f[p + n].reshape(-1, D, f[p + n].shape[-1])
                x[:, -1] = 0
                x[:, -1, feature] = gain
                if p + n + ".b" in f:
                    f[p + n + ".b"].reshape(-1, D)[:, -1] = 0
    return f32_edit(change)


@pytest.mark.parametrize("chunk", [1, 2, 31, 32, 33, 63, 64, 65, 97, 128, 150])
def test_chunk_edges(eng, tmp_path, prec, chunk):
    # one key that stands out: seen to the end of its chunk and not behind it; queries in a prompt and decoded, chunks on
    # and off page borders, the key first and last of its chunk
    cfg = mw.joint_config(64, 90, [(C(4, 2, 16, 16, chunk, 1, 4, 4, scale=0.7, right_scale=0.1), None)])
    case = Case(eng, tmp_path, cfg, prec, edit=sharp(cfg, 7, 9, 3.0))
    for key_at in sorted({0, chunk - 1, chunk, 2 * chunk - 1, 62, 63, 64, 65}):
        end = (key_at // chunk + 1) * chunk                # the first position that does not see it
        t = case.tokens(end + 3)
        t[(t == 7) | (t == 9)] = 11
        t[key_at] = 9
        t[end] = t[end + 1] = 7
        inside = end - 1
        if inside > key_at:
            t[inside] = 7
            u = t.copy()
            u[key_at] = 11
            a, b = case.oracle(t), case.oracle(u)
            assert np.abs(a[inside] - b[inside]).max() > 0.05 * np.abs(a[inside]).max()
        want = case.oracle(t)
        case.check(run_cut(case, t, [len(t)]), want, f"chunk {chunk} key at {key_at} prompt")
        case.check(run_cut(case, t, [max(1, inside), 1]), want, f"chunk {chunk} key at {key_at} decoded")
        case.check(run_cut(case, t, [max(2, key_at + 1), 2]), want, f"chunk {chunk} key at {key_at} pairs")
    case.close()


@pytest.mark.parametrize("sink", [-30.0, 0.0, 6.0, 40.0])
@pytest.mark.parametrize("kind", ["turned", "chunks"])
def test_sinks(eng, tmp_path, prec, sink, kind):
    # from no weight at all to nearly all of it, not scaled; more heads than one tile
    mixer = T(20, 1, 16, 24, rot_dims=8, scale=0.5) if kind == "turned" else C(20, 1, 16, 24, 90, 1, 8, 8, scale=0.5, right_scale=0.2)
    cfg = mw.joint_config(64, 90, [(mixer, None)])
    name = "l0.mix.sink" if kind == "turned" else "l0.mix.left.sink"

    def change(f):
        f[name][:] = sink + np.linspace(-1, 1, 20)
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(200)
    want = case.oracle(t)
    if sink == 6.0:                                        # leaving it out, or scaling it, would show
        for v in (-100.0, 3.0):
            assert differs(want, O.forward(cfg, dict(case.w, **{name: np.full(20, v, np.float32)}), t, np.float64))
    case.check(run_cut(case, t, [200]), want, f"sink {sink} prompt")
    case.check(run_cut(case, t, [130, 1]), want, f"sink {sink} decoded")
    case.close()


def test_one_more_in_the_denominator(eng, tmp_path, prec, monkeypatch):
    # scores far below zero: the one that is added decides, and the first tokens have little else
    cfg = mw.joint_config(64, 90, [(G(4, 2, 16, 16, 8, rot_dims=8, scale=0.4), None)])

    def change(f):
        f["l0.mix.left.k.b"][:] = -3.0
        f["l0.mix.left.q.b"][:] = 3.0
        f["l0.mix.left.o.b"][:] = 0.0
        f["l0.mix.right.out"][:] *= 0.1
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(90)
    want = case.oracle(t)
    with monkeypatch.context() as mp:
        plain = O.sunk_weights
        mp.setattr(O, "sunk_weights", lambda s, sink: plain(s, -1e9))
        assert differs(want, case.oracle(t), 0.01) or differs(want[:5], case.oracle(t)[:5])
    case.check(run_cut(case, t, [90]), want, "one more prompt")
    case.check(run_cut(case, t, [1]), want, "one more decoded")
    case.close()


@pytest.mark.parametrize("scaling", [None, (8.0, 2048, 32.0, 1.0), (4.0, 40, 3.0, 0.25), (2.0, 64, 1.0, 1.0), (16.0, 7, 1.0, 0.01),
                                     (0.5, 4096, 2.0, 0.5), (1.0, 100, 32.0, 1.0)])
@pytest.mark.parametrize("dims", [2, 16, 24])
def test_scaled_rotations(eng, tmp_path, prec, scaling, dims):
    # pairs that keep their frequency, that are slowed down and on the ramp between; a ramp of no width; a stretch of one
    cfg = mw.joint_config(64, 90, [(T(2, 1, 24, 16, rot_dims=dims, base=500.0, scale=0.9, scaling=scaling), None)])
    case = Case(eng, tmp_path, cfg, prec)
    t = case.tokens(140)
    want = case.oracle(t)
    if scaling and scaling[0] > 1:
        other = mw.joint_config(64, 90, [(T(2, 1, 24, 16, rot_dims=dims, base=500.0, scale=0.9, scaling=None), None)])
        assert differs(want, O.forward(other, case.w, t, np.float64), 0.01)
    case.check(run_cut(case, t, [140]), want, f"{scaling} prompt")
    case.check(run_cut(case, t, [70, 1]), want, f"{scaling} decoded")
    case.close()


def test_values_turn(eng, tmp_path, prec, monkeypatch):
    # a sharp query far from its key: the value arrives turned by the distance, with the rotation's own base and no scaling
    cfg = mw.joint_config(64, 90, [(T(2, 1, 16, 16, rot_dims=8, base=20.0, scale=0.7, scaling=(8.0, 50, 4.0, 0.5)), None)])
    case = Case(eng, tmp_path, cfg, prec, edit=sharp(cfg, 7, 9, 8.0))
    t = case.tokens(120)
    t[(t == 7) | (t == 9)] = 11
    t[[0, 40]] = 9
    t[[5, 63, 64, 90, 119]] = 7
    want = case.oracle(t)
    with monkeypatch.context() as mp:
        right = O.turn_neighbours
        mp.setattr(O, "turn_neighbours", lambda x, pos, f, gain=1.0: x if len(f) == 8 and gain == 1.0 else right(x, pos, f, gain))
        assert differs(want[[5, 63, 64, 90, 119]], case.oracle(t)[[5, 63, 64, 90, 119]])
    for cuts in ([120], [60, 1], [2]):
        case.check(run_cut(case, t, cuts), want, f"cuts {cuts}")
    case.close()


@pytest.mark.parametrize("lower", [0.0, 0.5, 1.0])
@pytest.mark.parametrize("bias", [-60.0, -5.0, 0.0, 8.0])
def test_forget_gates(eng, tmp_path, prec, lower, bias):
    # gates shut (everything is written and forgotten at once), open (nothing is), and a bound that decides; some
    # channels differ, so that fast and slow ones stand beside each other
    cfg = mw.joint_config(64, 90, [(C(1, 1, 8, 8, 5, 2, 24, 20, left_scale=0.3), None)])

    def change(f):
        f["l0.mix.right.lower"][:] = lower
        f["l0.mix.right.lower"][::5] = 0.9
        f["l0.mix.right.f.b"][:] = bias
        f["l0.mix.right.f.b"][::3] = 3.0
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(150)
    want = case.oracle(t)
    for cuts in ([150], [70, 1], [17, 2, 30]):
        case.check(run_cut(case, t, cuts), want, f"lower {lower} bias {bias} cuts {cuts}")
    case.close()


@pytest.mark.parametrize("kind", ["forget", "gru"])
def test_states_remember(eng, tmp_path, prec, kind):
    # one token long ago is still in the state: across chunks, segments, portions and decoded tokens
    if kind == "forget":
        mixer = C(1, 1, 8, 8, 3, 2, 16, 16, left_scale=0.1)
    else:
        mixer = G(1, 1, 8, 8, 40)
    cfg = mw.joint_config(48, 90, [(mixer, None)])

    def change(f):
        f["embed"][:, 0] = 0
        f["embed"][9, 0] = 40.0                            # what opens the gates
        if kind == "forget":
            f["l0.mix.right.lower"][:] = 0.0
            f["l0.mix.right.f"][:] *= 0.1
            f["l0.mix.right.f"][:, 0] = -3.0
            f["l0.mix.right.f.b"][:] = 9.0
        else:
            f["l0.mix.right.z"][:] *= 0.1
            f["l0.mix.right.z"][:, 0] = 3.0
            f["l0.mix.right.z.b"][:] = -9.0
            f["l0.mix.left.out"][:] *= 0.1
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change), pool=2048)
    t = case.tokens(900)
    t[t == 9] = 11
    t[3] = 9
    u = t.copy()
    u[3] = 11
    want = case.oracle(t)
    assert differs(want[600:], case.oracle(u)[600:])
    # (rows that 32-bit sums resolve: a head's sum over nine hundred tokens may nearly cancel ahead of its norm)
    d = O.forward(cfg, case.w, t, np.float32) - want
    calm = np.sqrt((d ** 2).mean(1)) < 1e-5 * np.sqrt((want ** 2).mean(1))
    assert calm[600:].mean() > 0.9
    for cuts in ([900], [500, 17, 300, 1], [65, 64, 2]):
        case.check(run_cut(case, t, cuts)[calm], want[calm], f"{kind} cuts {cuts}", deep=True)
    case.close()


@pytest.mark.parametrize("heads,dim,vdim", [(1, 16, 16), (2, 32, 50), (1, 64, 32), (3, 48, 130), (2, 100, 30), (1, 128, 128)])
def test_long_prompts_in_segments(eng, tmp_path, prec, heads, dim, vdim):
    # so few heads that a prompt's recurrence is walked in segments side by side, beside a short request and a long one
    cfg = mw.joint_config(48, 90, [(C(1, 1, 8, 8, 3, heads, dim, vdim, left_scale=0.3), None)])
    case = Case(eng, tmp_path, cfg, prec, pool=4096)
    t, u, v = case.tokens(1210), case.tokens(333, seed=8), case.tokens(9, seed=9)
    want = [case.oracle(x) for x in (t, u, v)]
    case.check(run_cut(case, t, [1100, 1, 109]), want[0], "alone")
    ss = [case.m.session() for _ in range(3)]
    rc, lg = E.mixed_step([(s, x, range(len(x))) for s, x in zip(ss, (t, u, v))])
    for got, w, n in zip(lg, want, (1210, 333, 9)):
        case.check(got, w, f"{n} rows of three requests")
    for s in ss:
        s.close()
    case.close()


@pytest.mark.parametrize("size", [33, 512])
def test_gru_extremes(eng, tmp_path, prec, size):
    # candidates far on both sides of zero and at it, gates shut and open
    cfg = mw.joint_config(64, 90, [(G(1, 1, 8, 8, size), None)])

    def change(f):
        f["l0.mix.right.x"][:] *= 3
        f["l0.mix.right.x"][0] = f["l0.mix.right.x.b"][0] = 0        # u = 0: one half from either branch
        f["l0.mix.right.x.b"][1:4] = [-40, 40, -100]
        f["l0.mix.right.z.b"][::4] = -50
        f["l0.mix.right.z.b"][1::4] = 50
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(300)
    want = case.oracle(t)
    for cuts in ([300], [130, 1], [17, 60, 2, 200]):
        case.check(run_cut(case, t, cuts), want, f"size {size} cuts {cuts}")
    case.close()


@pytest.mark.parametrize("kind", ["turned", "chunks", "gru"])
def test_positions_far_out(eng, tmp_path, prec, kind):
    # angles of far positions, slow and fast pairs, and a key thousands of positions back
    mixer = {"turned": T(2, 1, 16, 16, rot_dims=12, base=50.0, scale=1.0, scaling=(4.0, 512, 16.0, 1.0)),
             "chunks": C(2, 1, 16, 16, 2600, 1, 8, 8, scale=1.0, right_scale=0.3), "gru": G(2, 1, 16, 16, 24, rot_dims=12, scale=1.0)}[kind]
    cfg = mw.joint_config(32, 64, [(mixer, None)])
    case = Case(eng, tmp_path, cfg, prec, pool=4096, edit=sharp(cfg, 7, 9, 8.0))
    t = case.tokens(2900)
    t[(t == 7) | (t == 9)] = 11
    t[3] = t[2601] = 9
    t[[2502, 2599, 2600, 2889, 2890]] = 7
    want = case.oracle(t)
    s = case.m.session()
    places = [0, 1, 2, 63, 64, 1000, 2502, 2598, 2599, 2600, 2601]
    rc, lg = E.mixed_step([(s, t[:2880], places)])
    case.check(lg[0], want[places], kind + " prompt")
    got = np.stack([s.step(int(x)) for x in t[2880:]])
    s.close()
    case.check(got, want[2880:], kind + " decoded behind 2880")
    case.close()


@pytest.mark.parametrize("kind", ["turned", "chunks"])
@pytest.mark.parametrize("dim", [8, 40, 100])
def test_prompts_that_fill_the_device(eng, tmp_path, dim, kind):
    # so many heads and rows that a wave of the prompt's attention takes twice the rows; an unequal request beside it
    mixer = T(96, 48, dim, dim, scale=0.5) if kind == "turned" else C(96, 48, dim, dim + 2, 130, 2, 8, 8, scale=0.5)
    cfg = mw.joint_config(64, 90, [(mixer, None)])
    case = Case(eng, tmp_path, cfg, "bf16", pool=2048)
    t, u = case.tokens(1090), case.tokens(77, seed=8)
    want, other = case.oracle(t), case.oracle(u)
    a, b = case.m.session(), case.m.session()
    rc, lg = E.mixed_step([(a, t[:1050], range(1050)), (b, u, range(77))])
    assert rc == 1127
    case.check(lg[0], want[:1050], f"dim {dim} prompt")
    case.check(lg[1], other, f"dim {dim} beside it")
    rc, lg = E.mixed_step([(a, t[1050:], range(40))])
    case.check(lg[0], want[1050:], f"dim {dim} going on")
    a.close()
    b.close()
    case.close()


def test_long_decoding(eng, tmp_path, prec):
    case = Case(eng, tmp_path, stack(prec), prec)
    t = case.tokens(420)
    case.check(run_cut(case, t, [3, 1]), case.oracle(t), "417 decoded tokens", deep=True)
    case.close()


def test_prompt_longer_than_one_pass(eng, tmp_path, prec):
    # more rows than one device pass takes (4096): the step runs in passes
    cfg = mw.joint_config(32, 64, [(C(2, 1, 8, 8, 100, 2, 8, 12), mw.moe(3, 3, 16)), (G(2, 1, 8, 8, 24), mw.clamped_dense(16)),
                                   (C(2, 2, 8, 8, 4099, 1, 16, 4), None)])
    case = Case(eng, tmp_path, cfg, prec, pool=8192)
    t = case.tokens(4500)
    s, other = case.m.session(), case.m.session()
    places = [0, 1, 4000, 4094, 4095, 4096, 4097, 4098, 4099, 4163, 4499]
    rc, lg = E.mixed_step([(s, t[:4400], [p for p in places if p < 4400]), (other, t[:30], [29])])
    assert rc == 11
    want = case.oracle(t)
    case.check(lg[0], want[[p for p in places if p < 4400]], "passes")
    case.check(lg[1], want[[29]], "beside it")
    rc, lg = E.mixed_step([(s, t[4400:], [99])])
    case.check(lg[0], want[[4499]], "after the passes")
    s.close()
    other.close()
    case.close()


def test_sixteen_requests(eng, tmp_path, prec):
    case = Case(eng, tmp_path, stack(prec), prec, pool=4096, slots=16)
    todo = [case.tokens(n, seed=n) for n in range(5, 165, 10)]
    ss = [case.m.session() for _ in todo]
    E.mixed_step([(s, t[:-3], []) for s, t in zip(ss, todo)])
    got = []
    for k in (-3, -2, -1):
        rc, lg = E.batch_step(ss, [int(t[k]) for t in todo])
        assert rc == 16
        got.append(lg)
    case.check(np.concatenate([np.stack([g[i] for g in got]) for i in range(16)]),
               np.concatenate([case.oracle(t)[-3:] for t in todo]), "sixteen requests", deep=True)
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
    case = Case(eng, tmp_path, stack(prec), prec)
    t = case.tokens(100)
    want = case.oracle(t)
    s = case.m.session()
    rc, a = E.mixed_step([(s, t[:60], range(60))])
    for run in (0, 2, 6):
        s.lib.wrh_debug_fail_attention_at(run)
        rc, _ = E.mixed_step([(s, t[60:90], [0])])
        assert rc == E.WR_ERR_INTERNAL and s.pos == 60 and s.status == E.WR_ERR_INTERNAL
    rc, b = E.mixed_step([(s, t[60:], range(40))])
    assert rc == 40
    case.check(np.concatenate([a[0], b[0]]), want, "after failures", deep=True)
    s.close()
    case.close()
