"""Mixer-stack models of differential and keys-as-values attention with grouped expert
routing (architecture "Fedirax") on the device against the plain implementation of
tests/mixer_oracle.py: every test makes its own small model with random weights."""
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


WIDTH, VOCAB = 104, 211            # neither a multiple of 16
SOLO = {
    "keys": mw.keys_as_values(6, 3, 24, 37, rot_dims=12, base=5000.0, scale=0.3, softcap=4.0),
    "keys_no_cap": mw.keys_as_values(4, 2, 32, 50, softcap=None),
    "keys_tight_cap": mw.keys_as_values(4, 4, 40, 70, scale=1.0, softcap=0.7),
    "keys_no_rotation": mw.keys_as_values(4, 2, 32, 50, rot_dims=0),
    "keys_one_head": mw.keys_as_values(1, 1, 10, 64, rot_dims=4),
    "keys_20_heads_on_one": mw.keys_as_values(20, 1, 16, 33, rot_dims=2),
    "keys_dim100": mw.keys_as_values(4, 2, 100, 90, rot_dims=50),
    "keys_dim128": mw.keys_as_values(2, 1, 128, 1000),
    "keys_dim160": mw.keys_as_values(2, 1, 160, 40, rot_dims=70),
    "keys_window_of_one": mw.keys_as_values(4, 2, 16, 1),
    "diff": mw.difference(6, 3, 24, 40, 37, rot_dims=14, base=5000.0, scale=0.3, diff=0.3),
    "diff_half_rotated": mw.difference(4, 1, 64, 128, 70, rot_dims=32, diff=0.8),
    "diff_no_rotation": mw.difference(4, 2, 32, 64, 50, rot_dims=0, diff=0.1),
    "diff_one_head": mw.difference(1, 1, 10, 6, 64, rot_dims=4),
    "diff_every_head_its_own": mw.difference(3, 3, 64, 64, 65),
    "diff_9_heads_on_one": mw.difference(9, 1, 16, 24, 33),
    "diff_40_heads_on_two": mw.difference(40, 2, 8, 8, 1000, scale=1.5),
    "diff_dim128": mw.difference(4, 2, 128, 100, 90, rot_dims=64),
    "diff_dim100_v30": mw.difference(4, 1, 100, 30, 40),
    "diff_dim30_v128": mw.difference(2, 1, 30, 128, 40),
    "diff_dim60_v60": mw.difference(2, 2, 60, 60, 200, scale=1.0),
    "diff_dim128_v32": mw.difference(2, 1, 128, 32, 200),
    "diff_dim160": mw.difference(2, 1, 160, 24, 40, rot_dims=150),
    "diff_v200": mw.difference(2, 2, 16, 200, 40),
    "diff_window_of_one": mw.difference(4, 2, 16, 16, 1),
    "diff_nothing_taken_by_design": mw.difference(4, 2, 16, 16, 30, diff=0.0),
}


@pytest.mark.parametrize("name", sorted(SOLO))
def test_one_mixer(eng, tmp_path, prec, name):
    # whole prompt (matrix-core attention) and token by token
    case = Case(eng, tmp_path, mw.shared_kv_config(WIDTH, VOCAB, [(SOLO[name], None)], eps=1e-5, embed_scale=1.5), prec)
    t = case.tokens(150)
    want = case.oracle(t)
    case.check(run_cut(case, t, [150]), want, name + " whole")
    case.check(run_cut(case, t, [83, 1]), want, name + " decoded")
    case.close()


CHEAP = mw.keys_as_values(2, 1, 8, 20)
MOES = {
    "plain": mw.grouped_moe(6, 2, 40),
    "one_expert": mw.grouped_moe(1, 1, 24),
    "one_of_one_and_input": mw.grouped_moe(1, 1, 24, identity=1, scale=1.7),
    "scaled_shared": mw.grouped_moe(5, 3, 40, scale=2.5, shared=(72, 0.4)),
    "shared_wider": mw.grouped_moe(4, 2, 8, shared=(136, 3.0), limit=0.5),
    "inputs": mw.grouped_moe(4, 4, 24, identity=5, scale=0.7),
    "groups": mw.grouped_moe(12, 3, 24, groups=(4, 2), limit=0.8),
    "groups_of_one": mw.grouped_moe(7, 2, 24, identity=1, groups=(8, 3)),
    "one_group": mw.grouped_moe(6, 3, 24, groups=(1, 1)),
    "every_group": mw.grouped_moe(6, 3, 24, identity=3, groups=(3, 3)),
    "groups_inputs_shared": mw.grouped_moe(10, 4, 24, identity=4, groups=(7, 3), scale=1.3, limit=1.5, shared=(40, 0.9)),
    "all_of_the_kept": mw.grouped_moe(9, 6, 24, identity=3, groups=(4, 2), scale=3.0),
    "all": mw.grouped_moe(6, 8, 24, identity=2, scale=2.0),
    "many": mw.grouped_moe(150, 9, 8, identity=10, groups=(16, 5), shared=(8, 1.0)),
}


def check_clear(case, t, name, cuts_list):
    """Compares rows whose expert choice is no close call (in bfloat16 a close call may fall either way, and the experts
    come last here, so it stays in its row)."""
    margins = []
    want = O.forward(case.cfg, case.w, t, np.float64, margins=margins)
    clear = np.ones(len(t), dtype=bool)
    if case.prec == "bf16":
        clear = margins[-1] > 0.06
        assert clear.mean() > 0.4, clear.mean()
    for cuts in cuts_list:
        case.check(run_cut(case, t, cuts)[clear], want[clear], f"{name} cuts {cuts}")


@pytest.mark.parametrize("name", sorted(MOES))
def test_one_feed_forward(eng, tmp_path, prec, name):
    # experts by tiles of rows and by slots of sixteen, one token alone
    case = Case(eng, tmp_path, mw.shared_kv_config(WIDTH, VOCAB, [(CHEAP, MOES[name])], eps=1e-5, embed_scale=1.5), prec,
                edit=f32_edit(lambda f: f["l0.mix.o"].__imul__(0.3)))
    check_clear(case, case.tokens(150), name, ([150], [83, 1], [30, 20, 7, 2]))
    case.close()


def test_feed_forward_tiles(eng, tmp_path, prec):
    # enough rows that every expert's fill whole tiles in bfloat16, some experts without any
    cfg = mw.shared_kv_config(96, VOCAB, [(CHEAP, mw.grouped_moe(6, 3, 72, identity=2, groups=(4, 3), shared=(40, 1.0)))])

    def change(f):
        f["l0.mlp.correction"][2] = -5.0                   # hardly ever chosen; its whole group neither
        f["l0.mlp.correction"][3] = -5.0
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    check_clear(case, case.tokens(520), "tiles", ([520], [300, 220], [455, 65]))
    case.close()


@pytest.mark.parametrize("kind", ["negative", "inputs", "no_inputs", "correction_decides", "closed_gate", "open_gate", "clamps"])
def test_routing_branches(eng, tmp_path, prec, kind, monkeypatch):
    moe = mw.grouped_moe(6, 3, 24, identity=2, groups=(4, 2), scale=1.5, limit=0.25 if kind == "clamps" else 2.0,
                         shared=(40, 0.25 if kind == "clamps" else 1.0))
    cfg = mw.shared_kv_config(64, 90, [(CHEAP, moe)])

    def change(f):
        c = f["l0.mlp.correction"]
        if kind == "negative":                             # every choice value below zero
            c -= 2.0
        elif kind == "inputs":                             # only outputs that pass the input on
            c[6:] += 3.0
        elif kind == "no_inputs":
            c[6:] -= 3.0
        elif kind == "correction_decides":                 # the choice is the correction's, the weights are not
            c[:] = [3, -3, 2.5, 2, -3, -3, -3, -3]
        elif kind == "closed_gate":
            f["l0.mlp.shared.sg"] *= 8.0
        elif kind == "open_gate":
            f["l0.mlp.shared.sg"] *= 0.0
        f["l0.mlp.shared.down"] *= 2.0
        f["l0.mix.o"] *= 0.3
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(120)
    if kind in ("negative", "correction_decides", "clamps"):     # what a mistake there would do shows
        bad, cfg2 = dict(case.w), cfg
        a = case.oracle(t)
        if kind == "negative":                             # left-out groups at zero lie above every choice value

            def zeroed(z, correction, top, groups):
                s = np.exp(z - z.max()) / np.exp(z - z.max()).sum()
                v = s + correction
                kept = v.reshape(groups["count"], -1).max(1)
                out = np.argsort(-kept, kind="stable")[groups["keep"]:]
                v[np.isin(np.arange(len(z)) * groups["count"] // len(z), out)] = 0
                return np.argsort(-v, kind="stable")[:top], s
        elif kind == "clamps":
            cfg2 = dict(cfg, layers=[dict(cfg["layers"][0], mlp=dict(moe, expert=dict(moe["expert"], limit=9.0),
                                                                      shared=dict(moe["shared"], limit=9.0)))])
        else:
            bad["l0.mlp.correction"] = 0 * case.w["l0.mlp.correction"]
        with monkeypatch.context() as mp:
            if kind == "negative":
                mp.setattr(O, "grouped_choice", zeroed)
            b = O.forward(cfg2, bad, t, np.float64)
        assert np.median(np.abs(a - b).max(1) / np.abs(a).max(1)) > 0.05
    check_clear(case, t, kind, ([120], [50, 1], [64, 3]))
    case.close()


def test_wide_rows(eng, tmp_path, prec):
    # more features than the row steps hold in registers
    cfg = mw.shared_kv_config(4200, 50, [(CHEAP, mw.grouped_moe(3, 4, 8, identity=1, shared=(8, 1.0))), (mw.difference(2, 1, 8, 8, 9), None)])
    case = Case(eng, tmp_path, cfg, prec)
    t = case.tokens(100)
    want = case.oracle(t)
    case.check(run_cut(case, t, [100]), want, "wide whole")
    case.check(run_cut(case, t, [91, 1]), want, "wide decoded")
    case.close()


def stack(prec="f32"):
    """Both mixers, keys and values shared forwards (past other layers, with windows wider and narrower than their
    owner's, by more query heads), layers without a feed-forward.  In bfloat16 every output is chosen: a choice among random experts now and
    then hangs on less than bfloat16 resolves."""
    def moe(experts, top, ff, identity, groups, **kw):
        if prec == "bf16":
            return mw.grouped_moe(experts, experts + identity, ff, identity, (groups[0], groups[0]), **kw)
        return mw.grouped_moe(experts, top, ff, identity, groups, **kw)
    d = dict(rot_dims=10, base=3000.0, diff=0.4)
    return mw.shared_kv_config(WIDTH, VOCAB, [
        (mw.difference(4, 2, 24, 40, 50, **d), moe(7, 2, 40, 1, (4, 2), shared=(24, 1.0), scale=1.4, limit=1.5)),
        (mw.keys_as_values(4, 2, 32, 17, base=100.0, softcap=5.0), None),
        (mw.difference(6, 3, 16, 16, 70, rot_dims=16), None),
        (mw.difference(4, 2, 24, 40, 90, **d, kv_from=0), moe(5, 3, 24, 1, (2, 1))),
        (mw.difference(6, 3, 16, 16, 23, rot_dims=16, scale=0.7, kv_from=2), None),
        (mw.keys_as_values(6, 1, 16, 65), moe(4, 2, 24, 2, (3, 2), shared=(40, 2.0))),
        (mw.difference(8, 2, 24, 40, 33, **d, kv_from=0), None)], eps=1e-5)


@pytest.mark.parametrize("first", [0, 2])
def test_residual_after_every_layer(eng, tmp_path, prec, first):
    cfg = stack(prec)
    if first:                                              # a different layer ahead of the others
        cfg["layers"] = [cfg["layers"][1], cfg["layers"][0], cfg["layers"][5]]
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
    unrotated last dimension of every query and key (of the first map alone) picks up."""
    layer = cfg["layers"][0]
    m = layer["mixer"]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    maps = 2 if layer["type"] == "attention_2" else 1

    def change(f):
        f["embed"][:, :2] = 0
        f["embed"][query, 0] = f["embed"][key, 1] = 1.5
        for i, c in enumerate(cfg["layers"]):
            if c["type"] != layer["type"]:
                continue
            q = f[f"l{i}.mix.q"].reshape(c["mixer"]["heads"], maps, D, -1)
            q[:, 0, -1] = 0
            q[:, 0, -1, 0] = gain
            if f"l{i}.mix.k" in f:
                k = f[f"l{i}.mix.k"].reshape(G, maps, D, -1)
                k[:, 0, -1] = 0
                k[:, 0, -1, 1] = gain
            if maps == 1:
                f[f"l{i}.mix.q.b"].reshape(H, D)[:, -1] = 0
                f[f"l{i}.mix.k.b"].reshape(G, D)[:, -1] = 0
    return f32_edit(change)


def plant(case, key_at, inside, outside):
    """Tokens with the loud key and the two rows that ask for it; the key matters to the one inside alone."""
    t = case.tokens(outside + 3)
    t[(t == 7) | (t == 9)] = 11
    t[key_at] = 9
    if inside > key_at:
        t[inside] = 7
    t[outside] = t[outside + 1] = 7
    if inside > key_at and len(case.cfg["layers"]) == 1:
        u = t.copy()
        u[key_at] = 11
        a, b = case.oracle(t), case.oracle(u)
        assert np.abs(a[inside] - b[inside]).max() > 0.05 * np.abs(a[inside]).max()
        assert np.abs(a[outside] - b[outside]).max() < 1e-9
    return t


@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 63, 64, 65, 97, 128, 150])
@pytest.mark.parametrize("kind", ["keys", "diff"])
def test_window_edges(eng, tmp_path, prec, kind, window):
    # one key that stands out, just inside and just outside the window of a row
    # that asks for it; queries in a prompt and decoded, the key on and beside page borders
    mixer = (mw.keys_as_values(4, 2, 16, window, rot_dims=8, scale=0.5, softcap=40.0) if kind == "keys" else
             mw.difference(4, 2, 16, 16, window, rot_dims=8, scale=0.7))
    cfg = mw.shared_kv_config(64, 90, [(mixer, None)])
    case = Case(eng, tmp_path, cfg, prec, edit=sharp(cfg, 7, 9, 3.0))
    for key_at in (0, 1, 62, 63, 64, 65):
        inside, outside = key_at + window - 1, key_at + window
        t = plant(case, key_at, inside, outside)
        want = case.oracle(t)
        case.check(run_cut(case, t, [len(t)]), want, f"window {window} key at {key_at} prompt")
        case.check(run_cut(case, t, [max(1, inside), 1]), want, f"window {window} key at {key_at} decoded")
        case.check(run_cut(case, t, [max(2, key_at + 1), 2]), want, f"window {window} key at {key_at} pairs")
    case.close()


@pytest.mark.parametrize("own,borrowed", [(30, 64), (64, 30), (1, 65), (100, 1), (33, 33)])
def test_window_of_borrowed_keys(eng, tmp_path, prec, own, borrowed):
    # a layer that reads another's keys sees them through its own window
    cfg = mw.shared_kv_config(64, 90, [(mw.difference(2, 1, 16, 24, own, rot_dims=8, scale=0.7), None),
                                       (mw.difference(6, 1, 16, 24, borrowed, rot_dims=8, scale=0.7, diff=0.2, kv_from=0), None)])
    case = Case(eng, tmp_path, cfg, prec, edit=sharp(cfg, 7, 9, 3.0))
    for key_at in (0, 63):
        for window in (own, borrowed):
            t = plant(case, key_at, key_at + window - 1, key_at + window)
            want = case.oracle(t)
            for cuts in ([len(t)], [key_at + 1, 1], [key_at + 1, 2, 17]):
                case.check(run_cut(case, t, cuts), want, f"windows {own} {borrowed} key at {key_at} cuts {cuts}")
    case.close()


@pytest.mark.parametrize("sink", [-30.0, 0.0, 6.0, 40.0])
def test_sinks(eng, tmp_path, prec, sink):
    # from no weight at all to nearly all of it, neither scaled nor capped; windows long and short, more heads than one tile
    cfg = mw.shared_kv_config(64, 90, [(mw.keys_as_values(20, 1, 16, 300, scale=1.0, softcap=3.0), None), (mw.keys_as_values(2, 2, 16, 3), None)])

    def change(f):
        f["l0.mix.sink"][:] = sink + np.linspace(-1, 1, 20)
        f["l1.mix.sink"][:] = sink
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(260)
    want = case.oracle(t)
    if sink == 6.0:                                        # leaving it out, or capping it, would show
        for v in (-100, 3 * np.tanh(2.0)):
            other = O.forward(cfg, {k: np.full_like(x, v) if k.endswith("sink") else x for k, x in case.w.items()}, t, np.float64)
            assert np.median(np.abs(other - want).max(axis=1) / np.abs(want).max(axis=1)) > 0.05
    case.check(run_cut(case, t, [260]), want, f"sink {sink} prompt")
    case.check(run_cut(case, t, [130, 1]), want, f"sink {sink} decoded")
    case.close()


@pytest.mark.parametrize("cap", [0.5, 2.0, 50.0])
def test_capped_scores(eng, tmp_path, prec, cap):
    # products far beyond the cap and far inside it
    cfg = mw.shared_kv_config(64, 90, [(mw.keys_as_values(4, 2, 32, 200, scale=2.0, softcap=cap), None)])
    case = Case(eng, tmp_path, cfg, prec)
    t = case.tokens(170)
    want = case.oracle(t)
    if cap < 10:
        free = O.forward(mw.shared_kv_config(64, 90, [(mw.keys_as_values(4, 2, 32, 200, scale=2.0, softcap=None), None)]), case.w, t, np.float64)
        assert np.median(np.abs(free - want).max(axis=1) / np.abs(want).max(axis=1)) > 0.1
    case.check(run_cut(case, t, [170]), want, f"cap {cap} prompt")
    case.check(run_cut(case, t, [90, 1]), want, f"cap {cap} decoded")
    case.close()


@pytest.mark.parametrize("taken", [-1.5, 0.0, 0.9, 3.0])
def test_how_much_the_second_map_takes(eng, tmp_path, prec, taken):
    # the weight is made of two products of vectors: from one that adds to one that turns the output round
    cfg = mw.shared_kv_config(64, 90, [(mw.difference(4, 2, 16, 32, 100, diff=0.5, scale=1.0), None)])

    def change(f):
        for n in ("lq1", "lk1", "lq2", "lk2"):
            f["l0.mix." + n][:] = 0
        f["l0.mix.lq1"][3] = f["l0.mix.lq2"][5] = 1.0
        more = taken - 0.5
        f["l0.mix.lk1"][3] = np.log1p(max(more, 0))
        f["l0.mix.lk2"][5] = np.log1p(max(-more, 0))
    case = Case(eng, tmp_path, cfg, prec, edit=f32_edit(change))
    t = case.tokens(140)
    want = case.oracle(t)
    assert abs(O.differential_weight(O._sub(case.w, "l0.mix."), 0.5) - taken) < 0.02
    case.check(run_cut(case, t, [140]), want, f"weight {taken} prompt", deep=taken == 0.9)
    case.check(run_cut(case, t, [70, 1]), want, f"weight {taken} decoded", deep=taken == 0.9)
    case.close()


@pytest.mark.parametrize("kind", ["keys", "diff"])
def test_positions_far_out(eng, tmp_path, prec, kind):
    # angles of far positions, slow and fast pairs, and a key thousands of positions back
    mixer = (mw.keys_as_values(2, 1, 16, 2500, base=50.0, scale=1.0) if kind == "keys" else
             mw.difference(2, 1, 16, 16, 2500, base=50.0, scale=1.0))
    cfg = mw.shared_kv_config(32, 64, [(mixer, None)])
    case = Case(eng, tmp_path, cfg, prec, pool=4096, edit=sharp(cfg, 7, 9, 3.0))
    t = case.tokens(2900)
    t[(t == 7) | (t == 9)] = 11
    t[3] = t[390] = 9
    t[2502] = t[2503] = t[2889] = t[2890] = 7
    want = case.oracle(t)
    s = case.m.session()
    places = [0, 1, 2, 63, 64, 1000, 2499, 2500, 2501, 2502, 2503]
    rc, lg = E.mixed_step([(s, t[:2880], places)])
    case.check(lg[0], want[places], kind + " prompt")
    got = np.stack([s.step(int(x)) for x in t[2880:]])
    s.close()
    case.check(got, want[2880:], kind + " decoded behind 2880")
    case.close()


@pytest.mark.parametrize("dim", [8, 40, 100])
def test_prompts_that_fill_the_device(eng, tmp_path, dim):
    # so many heads and rows that a wave of the prompt's attention takes twice the rows; an unequal request beside it
    cfg = mw.shared_kv_config(64, 90, [(mw.keys_as_values(96, 48, dim, 130, scale=0.5), None)])
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
    cfg = mw.shared_kv_config(32, 64, [(mw.difference(2, 1, 8, 8, 40), None),
                                       (mw.difference(2, 1, 8, 8, 60, kv_from=0), mw.grouped_moe(3, 4, 16, identity=1)),
                                       (mw.keys_as_values(2, 2, 8, 30), None)])
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
