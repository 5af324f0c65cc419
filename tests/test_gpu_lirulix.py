"""The Lirulix session on the GPU against the plain implementation of the tests: every
mechanism, prompts and decoding, portions, sequences one after the other, far keys and
window edges, loops, and generation through the framework's own entry points."""
import copy
import json
import os
import subprocess
from pathlib import Path

import numpy as np
import pytest

import buddy_mlir_amd as bma
import lirulix_models as M
import lirulix_oracle as L
from buddy_mlir_amd import BuddyHipError
from buddy_mlir_amd.session import FolderSession, Sampler

pytestmark = pytest.mark.gpu

ROOT = Path(__file__).resolve().parent.parent
# f32: rounding of sums only.  bfloat16: 2^-9 per stored activation, a dozen of them
# on the way through a few layers.
BOUND = {"float32": 2e-5, "bfloat16": 4e-2}
DTYPES = ("float32", "bfloat16")


def tokens_for(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.int32)


def check(got, want, dtype, what=""):
    """Every row within the bound.  Of many bfloat16 rows a few may lie above it: where
    the two maps of a head all but cancel, the norm behind them scales up their rounding."""
    e = M.row_errors(got, want)
    assert np.isfinite(got).all()
    if dtype == "bfloat16" and len(e) >= 20 and e.max() < 3 * BOUND[dtype]:
        assert np.mean(e > BOUND[dtype]) < 0.04, (what, float(np.mean(e > BOUND[dtype])))
        return
    assert e.max() < BOUND[dtype], (what, int(e.argmax()), float(e.max()), float(np.median(e)))


def all_rows(s, tokens, start=0):
    return s.prefill_rows(tokens, np.arange(len(tokens)), start)


def feed(s, tokens, cuts):
    """The sequence in portions of the given sizes (1 = a decode step), its logits."""
    out, at = [], 0
    for n in cuts:
        part = tokens[at:at + n]
        if n == 1:
            out.append(s.decode(int(part[0]), at)[1][None])
        else:
            out.append(all_rows(s, part, at))
        at += n
    assert at == len(tokens)
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(M.SIZES))
def test_prompt_and_decoding_match_the_oracle(tmp_path, name, dtype):
    cfg = M.SIZES[name]
    folder, t = M.build(tmp_path, cfg, seed=len(name), rank=(16, 24) if name == "even" else None)
    tokens = tokens_for(cfg, 90)
    want = L.forward(cfg, t, tokens)
    s = FolderSession(folder, dtype, max_len=128)
    assert s.vocab == cfg["vocab"] and s.architecture == "Lirulix"
    check(all_rows(s, tokens), want, dtype, "prompt")
    check(feed(s, tokens, [1] * 90), want, dtype, "decoding")
    check(feed(s, tokens, [70] + [1] * 20), want, dtype, "prompt, then decoding")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompt_at_real_head_sizes(tmp_path, dtype):
    cfg = M.LARGE
    folder, t = M.build(tmp_path, cfg, rank=(128, 64))
    tokens = tokens_for(cfg, 1100)
    want = L.forward(cfg, t, tokens)
    s = FolderSession(folder, dtype, max_len=1200)
    check(all_rows(s, tokens), want, dtype, "prompt")
    got = feed(s, tokens, [700, 384] + [1] * 16)
    check(got, want, dtype, "portions, then decoding")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("what", ["full", "diff", "delta", "feed_forward", "loop"])
def test_mechanism_alone(tmp_path, what, dtype):
    """One layer, the head an identity: the logits are the normed residual."""
    layer = {"full": M.full(ff=None), "diff": M.diff(ff=None), "delta": M.delta(),
             "feed_forward": M.full(ff=33), "loop": M.full(ff=None)}[what]
    cfg = M.config([layer], width=56, vocab=64, loop=(0, 1, 3 if what == "loop" else 1))

    def edit(t):
        t["head"] = np.eye(64, 56)
        if what in ("feed_forward", "loop"):
            t["l0.mix.o"] *= 0.0          # the feed-forward, or the steps, alone
    folder, t = M.build(tmp_path, cfg, 3, edit)
    tokens = tokens_for(cfg, 70)
    want = L.forward(cfg, t, tokens)
    s = FolderSession(folder, dtype, max_len=80)
    check(all_rows(s, tokens), want, dtype, "prompt")
    check(feed(s, tokens, [3] + [1] * 67), want, dtype, "decoding")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("block", [0, 16, 80])
def test_portions_do_not_matter(tmp_path, dtype, block):
    """Cuts anywhere, down to two tokens and one, also where a portion is longer than
    the block in which it goes through the layers and the ring of cache rows wraps."""
    cfg = M.SIZES["mixed"]
    folder, t = M.build(tmp_path, cfg)
    tokens = tokens_for(cfg, 205, 7)
    want = L.forward(cfg, t, tokens)
    s = FolderSession(folder, dtype, max_len=256, prefill_block=block)
    rng = np.random.default_rng(8)
    for cuts in ([205], [2] * 102 + [1], [3, 64, 1, 2, 63, 65, 1, 1, 5], None, None):
        if cuts is None:
            cuts = []
            while sum(cuts) < 205:
                cuts.append(int(min(rng.choice([1, 2, 3, 17, 37, 64, 130]), 205 - sum(cuts))))
        check(feed(s, tokens, cuts), want, dtype, cuts)


@pytest.mark.parametrize("dtype", DTYPES)
def test_sequences_one_after_the_other(tmp_path, dtype):
    """What an earlier sequence left in caches, rings and states is not seen, whether
    it was ended or simply overtaken by position 0."""
    cfg = M.SIZES["mixed"]
    folder, t = M.build(tmp_path, cfg)
    s = FolderSession(folder, dtype, max_len=160)
    reqs = [tokens_for(cfg, n, n) for n in (150, 1, 2, 23, 97)]
    fresh = [feed(FolderSession(folder, dtype, max_len=160), r, [len(r)]) for r in reqs]
    for r, f in zip(reqs, fresh):
        check(f, L.forward(cfg, t, r), dtype)
    for end in (True, False):
        for i in (0, 1, 3, 0, 2, 4, 1, 0):
            np.testing.assert_array_equal(feed(s, reqs[i], [len(reqs[i])]), fresh[i])
            if end:
                s.reset()
    # decoding from position 0 over what a long prompt left
    feed(s, reqs[0], [150])
    check(feed(s, reqs[3], [1] * 23), L.forward(cfg, t, reqs[3]), dtype)


def needle_tokens(cfg, n, seed, places):
    tokens = np.random.default_rng(seed).integers(6, cfg["vocab"], n).astype(np.int32)
    for at, token in places.items():
        tokens[at] = token
    return tokens


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
def test_window_edges(tmp_path, dtype, decoded):
    """A key whose score stands out, just inside and just outside the window, from the
    first tokens on and after the ring of cache rows has wrapped."""
    window = 24
    cfg, t = M.needle_model("diff", window)
    folder = L.write_model(tmp_path, cfg, t)
    s = FolderSession(folder, dtype, max_len=512, prefill_block=16)   # ring of 64 rows
    for at in (0, 1, 15, 16, 39, 40, 63, 64, 127, 200):
        for gap in (1, window - 1, window):
            n = at + gap + 1
            tokens = needle_tokens(cfg, n, at + gap, {at: M.NEEDLE, n - 1: M.ASK})
            want = L.forward(cfg, t, tokens)[-1]
            seen = want[M.FOUND] > 1.0
            assert seen == (gap < window)              # the oracle tells them apart
            if decoded:
                s.prefill(tokens[:-1], 0)
                got = s.decode(M.ASK, n - 1)[1]
            else:
                got = s.prefill(tokens, 0)[1]
            assert (got[M.FOUND] > 1.0) == seen
            check(got[None], want[None], dtype, (at, gap))


@pytest.mark.parametrize("dtype", DTYPES)
def test_window_passes_over_decoded_tokens(tmp_path, dtype):
    cfg, t = M.needle_model("diff", 9)
    folder = L.write_model(tmp_path, cfg, t)
    s = FolderSession(folder, dtype, max_len=256)
    tokens = needle_tokens(cfg, 30, 3, {11: M.NEEDLE, 12: M.ASK, 19: M.ASK, 20: M.ASK, 28: M.ASK})
    want = L.forward(cfg, t, tokens)                   # gaps 1, 8: visible; 9, 17: not
    assert (want[[12, 19, 20, 28], M.FOUND] > 1.0).tolist() == [True, True, False, False]
    for cuts in ([10] + [1] * 20, [30], [11, 2, 7, 1, 9], [19, 2, 9]):
        check(feed(s, tokens, cuts), want, dtype, cuts)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["full", "diff"])
@pytest.mark.parametrize("length", [1030, 4500])
def test_far_keys(tmp_path, dtype, kind, length):
    """One key among thousands decides, in prompts and in decoding; chunks of a step
    take more than one tile of keys in the longer one."""
    cfg, t = M.needle_model(kind, 5000, heads=1)
    folder = L.write_model(tmp_path, cfg, t)
    s = FolderSession(folder, dtype, max_len=5100)
    asked = [64, 100, 1022, 1023, length - 7, length - 3, length - 1]
    tokens = needle_tokens(cfg, length, 5, {3: M.NEEDLE, **{p: M.ASK for p in asked}})
    want = L.forward(cfg, t, tokens)
    rows = np.unique([2, 3, 4, 64, 100, 1022, length - 8])
    got = s.prefill_rows(tokens[:-7], rows)
    check(got, want[rows], dtype, "prompt")
    assert (got[np.isin(rows, asked), M.FOUND] > 1.0).all()
    for p in range(length - 7, length):
        got = s.decode(int(tokens[p]), p)[1]
        check(got[None], want[p][None], dtype, p)
        assert (got[M.FOUND] > 1.0) == (tokens[p] == M.ASK)


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_takes_the_weight_that_no_key_earns(tmp_path, dtype):
    """With a sink between the ordinary scores and the needle's, what is found depends
    on the sink alone: nothing without the needle, all of it with."""
    cfg, t = M.needle_model("full", heads=2, sink=9.0)
    folder = L.write_model(tmp_path, cfg, t)
    s = FolderSession(folder, dtype, max_len=300)
    for n, places in ((1, {}), (70, {}), (70, {2: M.NEEDLE, 69: M.ASK}), (200, {2: M.NEEDLE, 199: M.ASK})):
        tokens = needle_tokens(cfg, n, n, places)
        want = L.forward(cfg, t, tokens)
        if not places:      # the common part of the values is all but lost to the sink
            without = dict(t, **{"l0.mix.sink": t["l0.mix.sink"] - 60})
            assert abs(want[-1][4]) < 0.3 < L.forward(cfg, without, tokens)[-1][4]
        check(feed(s, tokens, [n]), want, dtype, n)
        check(feed(s, tokens, [1] * n), want, dtype, n)


@pytest.mark.parametrize("dtype", DTYPES)
def test_strong_and_weak_decays(tmp_path, dtype):
    """One loud token: what later tokens still hear of it, across the chunks of a prompt
    and in decoding, with decays per channel from none to a factor e^-30 a token."""
    cfg = M.config([M.delta(heads=3, kv=1, dim=16, vdim=16, taps=1)], width=40, vocab=48)

    def edit(t):
        t["embed.norm"] *= 0.0
        t["l0.mix.v"] *= 3.0
        t["l0.mix.a2"] *= 0.3
        t["l0.mix.A_log"] = np.array([0.0, 1.0, -6.0])
        t["l0.mix.dt_bias"] = np.concatenate([np.linspace(-9, 12, 16)] * 3)
        t["head"] = np.eye(48, 40)
    folder, t = M.build(tmp_path, cfg, 1, edit)
    for at in (0, 14, 15, 16, 62, 63, 64):
        tokens = tokens_for(cfg, 260, at)
        tokens[tokens == 5] = 6
        tokens[at] = 5
        want = L.forward(cfg, t, tokens)
        s = FolderSession(folder, dtype, max_len=300, prefill_block=128)
        check(all_rows(s, tokens), want, dtype, at)
        check(feed(s, tokens, [66, 2, 60] + [1] * 132), want, dtype, at)


@pytest.mark.parametrize("dtype", DTYPES)
def test_repeated_keys_are_overwritten(tmp_path, dtype):
    """The same few tokens over and over, full steps and hardly any decay: every write
    meets what the same key wrote before, within a chunk and across chunks."""
    cfg = M.config([M.delta(heads=2, kv=1, dim=20, vdim=12, taps=1)], width=40, vocab=48)

    def edit(t):
        t["l0.mix.b"] *= 4.0
        t["l0.mix.dt_bias"] = t["l0.mix.dt_bias"] * 0.0 - 8.0
        t["head"] = np.eye(48, 40)
    folder, t = M.build(tmp_path, cfg, 2, edit)
    tokens = (tokens_for(cfg, 300) % 3).astype(np.int32)
    want = L.forward(cfg, t, tokens)
    s = FolderSession(folder, dtype, max_len=300)
    check(all_rows(s, tokens), want, dtype, "prompt")
    check(feed(s, tokens, [131, 2, 64, 3] + [1] * 100), want, dtype, "portions")


@pytest.mark.parametrize("dtype", DTYPES)
def test_passes_of_a_loop_do_not_share_their_state(tmp_path, dtype):
    """Every pass with a cache of its own: the first pass differs from the others only by
    its step, and a model unrolled by hand gives the same logits."""
    body = [M.full(), M.diff(), M.delta(ff=20)]
    cfg = M.config(body, loop=(0, 3, 2))
    folder, t = M.build(tmp_path / "a", cfg, 4)
    flat = M.config(body + copy.deepcopy(body), loop=(0, 1, 1))
    u = {k: v for k, v in t.items() if not k.startswith("l")}
    for k, v in t.items():
        if k.startswith("l") and k != "loop.step":
            i, rest = int(k[1:k.index(".")]), k[k.index("."):]
            u[f"l{i}{rest}"] = u[f"l{i + 3}{rest}"] = v
    t = dict(t, **{"loop.step": np.stack([t["loop.step"][0], 0 * t["loop.step"][1]])})
    u["loop.step"] = t["loop.step"][:1]
    L.write_model(tmp_path / "a", cfg, t)
    L.write_model(tmp_path / "b", flat, u)
    tokens = tokens_for(cfg, 100)
    a, b = (FolderSession(tmp_path / x, dtype, max_len=128) for x in "ab")
    for cuts in ([100], [60] + [1] * 40):
        got = feed(a, tokens, cuts)
        np.testing.assert_array_equal(got, feed(b, tokens, cuts))
        check(got, L.forward(cfg, t, tokens), dtype, cuts)


def test_configuration_without_a_loop(tmp_path):
    cfg = M.config([M.full(), M.delta()])
    t = L.random_tensors(cfg, 6)
    t["loop.step"] *= 0.0
    want = L.forward(cfg, t, tokens_for(cfg, 40))
    del t["loop.step"]
    for loop in ("none", "null"):
        c = {k: v for k, v in cfg.items() if k != "loop"} if loop == "none" else {**cfg, "loop": None}
        s = FolderSession(L.write_model(tmp_path / loop, c, t), "float32", max_len=64)
        check(feed(s, tokens_for(cfg, 40), [30] + [1] * 10), want, "float32")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_by_the_greedy_entry_point(tmp_path, dtype):
    """300 greedy steps on the device (captured steps, replayed) against the oracle on
    the tokens they chose, and the same tokens from single steps, captured or not."""
    cfg = M.SIZES["mixed"]
    folder, t = M.build(tmp_path, cfg)
    s = FolderSession(folder, dtype, max_len=400)
    prompt = tokens_for(cfg, 12)
    first, _ = s.prefill(prompt, 0)
    out = s.decode_greedy(first, 12, 300)
    seq = np.concatenate([prompt, [first], out]).astype(np.int32)
    want = L.forward(cfg, t, seq)
    # the chosen logit is the largest, up to the format's rounding
    spread = want.std(-1)
    for p, tok in zip(range(11, 312), seq[12:]):
        assert want[p, tok] > want[p].max() - BOUND[dtype] * 4 * spread[p]
    for graph in (True, False):
        s.use_graph(graph)
        s.prefill(prompt, 0)
        logits = []
        for i in range(300):
            nxt, lg = s.decode(int(seq[12 + i]), 12 + i)
            assert nxt == seq[13 + i]
            logits.append(lg)
        check(np.stack(logits), want[12:312], dtype, graph)


def test_captured_steps_equal_launched_ones_bit_for_bit(tmp_path):
    cfg = M.SIZES["even"]
    folder, _ = M.build(tmp_path, cfg)
    tokens = tokens_for(cfg, 40)
    s = FolderSession(folder, "bfloat16", max_len=64)
    runs = []
    for graph in (True, False, True):
        s.use_graph(graph)
        runs.append(feed(s, tokens, [8] + [1] * 32))
    np.testing.assert_array_equal(runs[0], runs[1])
    np.testing.assert_array_equal(runs[0], runs[2])


def test_sampling_entry_points(tmp_path):
    """temperature 0 is the greedy choice; a seeded sampler repeats itself."""
    cfg = M.SIZES["mixed"]
    folder, _ = M.build(tmp_path, cfg)
    s = FolderSession(folder, "bfloat16", max_len=128)
    prompt = tokens_for(cfg, 9)
    first, _ = s.prefill(prompt, 0)
    greedy = s.decode_greedy(first, 9, 20)

    def run(**kw):
        sampler = Sampler(**kw)
        s.prefill(prompt, 0)
        out = [first]
        for i in range(20):
            out.append(s.decode_sample(sampler, out[-1], 9 + i, out))
        return out[1:]
    assert run(temperature=0.0) == greedy.tolist()
    a = run(temperature=1.2, top_k=20, seed=11)
    assert a == run(temperature=1.2, top_k=20, seed=11) and a != greedy.tolist()


def test_positions_that_do_not_follow_are_refused(tmp_path):
    cfg = M.SIZES["mixed"]
    folder, _ = M.build(tmp_path, cfg)
    s = FolderSession(folder, "bfloat16", max_len=64)
    s.prefill(tokens_for(cfg, 10), 0)
    for bad in (lambda: s.decode(1, 9), lambda: s.decode(1, 11), lambda: s.prefill([1, 2], 12),
                lambda: s.decode_greedy(1, 10, 60), lambda: s.prefill(tokens_for(cfg, 60), 10),
                lambda: s.decode(cfg["vocab"], 10)):
        with pytest.raises(BuddyHipError):
            bad()
    s.decode(1, 10)


@pytest.mark.parametrize("edit,text", [
    (lambda c: c["layers"][0].update(type="other"), "other"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=2), "kv_heads"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "moe"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=22), "rotation"),
    (lambda c: c["layers"][2]["mixer"].pop("diff"), "diff"),
    (lambda c: c["loop"].update(stop=9), "loop"),
    (lambda c: c.update(width=47), "expected BF16"),
    (lambda c: c["loop"].update(times=3), "loop.step"),
    (lambda c: c["layers"].append(c["layers"][0]), "l4."),
])
def test_configurations_that_do_not_fit_are_refused(tmp_path, edit, text):
    cfg = copy.deepcopy(M.SIZES["mixed"])
    folder, _ = M.build(tmp_path, cfg)
    edit(cfg)
    (folder / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(BuddyHipError, match=text):
        FolderSession(folder)


def test_command_line_runner_generates_the_same(tmp_path):
    cfg = M.SIZES["mixed"]
    folder, _ = M.build(tmp_path, cfg)
    prompt = tokens_for(cfg, 11).tolist()
    runner = bma.library_path().parent / "buddy_hip_run"
    for dtype in DTYPES:
        s = FolderSession(folder, dtype, max_len=128)
        first, _ = s.prefill(prompt, 0)
        want = [first] + s.decode_greedy(first, 11, 24).tolist()
        s.close()
        r = subprocess.run([str(runner), "--model", str(folder), "--dtype", dtype, "--max-new", "25",
                            "--tokens", ",".join(map(str, prompt))],
                           capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr
        ids = [line for line in r.stdout.splitlines() if line.startswith("[Output ids]")][0]
        assert [int(x) for x in ids.split("]")[1].split()] == want


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(tmp_path, dtype):
    """Two sequences one after the other, in portions, through the replay program."""
    cfg = M.SIZES["odd"]
    folder, t = M.build(tmp_path / "m", cfg)
    out = tmp_path / "out"
    out.mkdir()
    a, b = tokens_for(cfg, 50, 1), tokens_for(cfg, 20, 2)
    steps = [("a", a[:30], [29, 0, 7]), ("a", a[30:31], [0]), ("a", a[31:33], []), ("a", a[33:], [16, 2]),
             ("b", b[:1], [0]), ("b", b[1:], [18])]
    lines = [json.dumps({"step": i, "entries": [{"id": n, "tokens": x.tolist(), "want": w}],
                         "end": ["a"] if i == 3 else ["b"] if i == 5 else []})
             for i, (n, x, w) in enumerate(steps)]
    r = subprocess.run([str(ROOT / "bin" / "trace_run"), "--model", str(folder), "--dtype", dtype,
                        "--out", str(out), "--max-tokens", "50"], input="\n".join(lines) + "\n",
                       capture_output=True, text=True, timeout=110, env=dict(os.environ))
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(6)]
    full = {"a": L.forward(cfg, t, a), "b": L.forward(cfg, t, b)}
    at = {"a": 0, "b": 0}
    for i, (n, x, w) in enumerate(steps):
        path = out / f"{i}.f32"
        assert path.exists() == bool(w)
        if w:
            got = np.fromfile(path, "<f4").reshape(len(w), cfg["vocab"])
            check(got, full[n][at[n] + np.array(w)], dtype, i)
        at[n] += len(x)
