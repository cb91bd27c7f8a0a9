"""Models of layer lists on the GPU against the plain float64 oracle (oracle/layered.py): every mechanism alone, prompts
in one pass, in portions and token by token, window edges, long decoding, reuse of the cache and the states, odd sizes,
and greedy generation through the framework's entry points."""
import os
import subprocess
import sys

import numpy as np
import pytest

from mongoose_amd import configs as C
from mongoose_amd import engine as E
from oracle import layered as O
from tests import layered_models as M

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# float32: what reordered fp32 sums leave; bfloat16: what bf16 activations and cache rows leave on these small models
TOL = {"float32": 1e-4, "bfloat16": 0.05}


def with_ff(layer, ff):
    return {**layer, **ff}


MIXED = [with_ff(M.latent(window=37), C.dense_ff(100)),
         with_ff(M.latent(window=20, scale=0.6), C.moe_ff(40, 10, 3, 72)),
         with_ff(M.delta(), C.moe_ff(24, 7, 2)),
         M.latent(heads=2, window=50, kv_from=1, dim=64, vdim=33),
         with_ff(M.delta(heads=2, dim=32, decay_rank=70), C.dense_ff(64)),
         with_ff(M.latent(heads=5, window=0, kv_from=0, rope_base=10000.0), C.moe_ff(33, 66, 5, 10))]

MECHANISMS = {
    "latent": [M.latent()],
    "latent_window": [M.latent(window=9)],
    "latent_part_rotated": [M.latent(rope_dims=16)],
    "latent_one_head": [M.latent(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, q_rank=1)],
    "latent_wide": [M.latent(heads=4, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=192, scale=0.1, window=30)],
    "latent_wider": [M.latent(heads=2, dim=160, rot_dim=72, vdim=200, kv_rank=600, q_rank=96, scale=0.1)],
    "latent_beyond_variants": [M.latent(heads=2, dim=250, rot_dim=16, vdim=130, kv_rank=200, q_rank=96, scale=0.1, window=25)],
    "latent_shared": [M.latent(window=12), M.latent(window=31, kv_from=0, heads=4, dim=96, vdim=64)],
    "delta": [M.delta()],
    "delta_small": [M.delta(heads=1, dim=5, decay_rank=1)],
    "delta_64": [M.delta(heads=4, dim=64, decay_rank=32)],
    "delta_128": [M.delta(heads=2, dim=128, decay_rank=65)],
    "delta_200": [M.delta(heads=2, dim=200, decay_rank=40)],
    "dense": [with_ff(M.delta(), C.dense_ff(77))],
    "moe": [with_ff(M.delta(), C.moe_ff(50, 9, 4))],
    "moe_shared": [with_ff(M.latent(window=5), C.moe_ff(64, 70, 6, 130))],
    "moe_all": [with_ff(M.latent(window=5), C.moe_ff(16, 4, 4, 8))],
    "one_expert": [with_ff(M.delta(), C.moe_ff(31, 1, 1))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_each_mechanism_alone(hip, name, dtype):
    """70 tokens: one pass (matrix forms of attention and recurrence), token by token, and small portions."""
    p = M.Pair(M.model(MECHANISMS[name]), seed=3, eng=hip, dtype=dtype, maxSeq=128)
    toks = p.tokens(70)
    want = p.oracle_logits(toks)
    for sizes in ([70], [1], [33, 2]):
        e = M.errors(M.run_portions(p.hip, toks, sizes), want)
        assert e.max() < TOL[dtype], (name, sizes, int(e.argmax()), float(e.max()))
    p.close()


def all_experts(layers):
    """The same layers with every expert chosen: in bf16 two router scores closer than rounding pick another expert,
    which is no fault but would need tolerances that hide faults (the choice itself is tested alone)."""
    return [{**L, "experts": L["top"]} if L.get("mlp") == C.MLP_MOE else L for L in layers]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width, vocab", [(70, 37), (65, 1), (130, 131), (320, 257), (1100, 70)])
def test_other_widths(hip, dtype, width, vocab):
    """Widths and vocabularies that are no multiple of anything the kernels work in."""
    layers = [with_ff(M.latent(window=11, heads=2), C.dense_ff(width // 2 + 1)), with_ff(M.delta(), C.moe_ff(9, 3, 3, 5)),
              M.latent(kv_from=0, window=23, heads=3, vdim=20, q_rank=31)]
    p = M.Pair(M.model(layers, width=width, vocab=vocab, alpha=3.1, eps=1e-3), seed=8, eng=hip, dtype=dtype, maxSeq=128)
    toks = p.tokens(90)
    want = p.oracle_logits(toks)
    for sizes in ([90], [1], [50, 2]):
        got = M.run_portions(p.hip, toks, sizes)
        if vocab == 1:
            assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max()
            continue
        e = M.errors(got, want)
        assert e.max() < TOL[dtype], (sizes, int(e.argmax()), float(e.max()))
    p.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("w0, ab", [(9.0, 9.0), (-9.0, 9.0), (9.0, -9.0), (-9.0, -9.0)])
def test_delta_rule_at_the_ends_of_its_gates(hip, dtype, w0, ab):
    """Fastest and slowest decay, full and no removal, over several chunks of the many-row form and a ragged end."""
    p = M.Pair(M.model([M.delta(heads=2, dim=64, decay_rank=8)]), seed=6, eng=hip, dtype=dtype, maxSeq=256,
               tweak={"l0.mix.w0": lambda a: 0.1 * a + w0, "l0.mix.a.b": lambda a: 0.1 * a + ab})
    toks = p.tokens(215)
    want = p.oracle_logits(toks)
    for sizes in ([215], [64], [100, 3], [1]):
        e = M.errors(M.run_portions(p.hip, toks, sizes), want)
        assert e.max() < TOL[dtype], (sizes, int(e.argmax()), float(e.max()))
    p.close()


@pytest.fixture(scope="module", params=["float32", "bfloat16"])
def mixed(request, hip):
    layers = MIXED if request.param == "float32" else all_experts(MIXED)
    p = M.Pair(M.model(layers), seed=5, eng=hip, dtype=request.param, maxSeq=400)
    p.dtype = request.param
    p.toks = p.tokens(330)
    p.want = p.oracle_logits(p.toks)
    yield p
    p.close()


def test_residual_after_every_layer(mixed):
    p = mixed
    toks = p.toks[:40]
    p.orc.reset()
    trail = []
    for t in toks:
        p.orc.step(int(t))
        trail.append(p.orc.trail)
    for end in range(1, len(MIXED) + 1):
        rc, x = p.hip.PrefillHidden(toks, 0, end)
        assert rc == 0, E.last_error()
        want = np.stack([t[end - 1] for t in trail])
        err = np.abs(x - want).max() / np.abs(want).max()
        assert err < (1e-5 if p.dtype == "float32" else 0.05), (end, err)
    assert p.hip.ResetKV() == 0


@pytest.mark.parametrize("sizes", [[330], [2], [3, 64, 2, 17], [100, 1, 1, 31], [16], [15], [64], [65, 63]])
def test_portions(mixed, sizes):
    p = mixed
    e = M.errors(M.run_portions(p.hip, p.toks, sizes), p.want)
    assert e.max() < TOL[p.dtype], (sizes, int(e.argmax()), float(e.max()))


def test_prompt_then_long_decoding(mixed):
    p = mixed
    assert p.hip.ResetKV() == 0
    rc, _ = p.hip.PrefillLogits(p.toks[:30], 0, [])
    assert rc == 0
    out = np.empty(p.s.vocab, np.float32)
    got = []
    for pos in range(30, len(p.toks)):
        rc, nxt = p.hip.DecodeToken(int(p.toks[pos]), pos, out)
        assert rc == 0, E.last_error()
        assert nxt == int(out.argmax())
        got.append(out.copy())
    e = M.errors(np.stack(got), p.want[30:])
    assert e.max() < TOL[p.dtype], (int(e.argmax()) + 30, float(e.max()))


def test_cache_and_states_are_reused_cleanly(mixed):
    """Another request between two runs of the same one, and a restart at position 0 without a reset."""
    p = mixed
    first = M.run_portions(p.hip, p.toks[:80], [80])
    other = p.tokens(200, salt=9)
    M.run_portions(p.hip, other, [200])
    rc, again = p.hip.PrefillLogits(p.toks[:80], 0, list(range(80)))
    assert rc == 0
    assert np.array_equal(first, again)
    M.run_portions(p.hip, other, [1])
    out, rows = np.empty(p.s.vocab, np.float32), []
    for pos in range(20):
        rc, _ = p.hip.DecodeToken(int(p.toks[pos]), pos, out)
        assert rc == 0
        rows.append(out.copy())
    assert M.errors(np.stack(rows), p.want[:20]).max() < TOL[p.dtype]


def test_wanted_rows_do_not_change_with_the_selection(mixed):
    p = mixed
    assert p.hip.ResetKV() == 0
    rc, some = p.hip.PrefillLogits(p.toks[:60], 0, [59, 0, 7])
    assert rc == 0
    rc, rows = p.hip.PrefillLogits(p.toks[:60], 0, list(range(60)))
    assert rc == 0
    assert np.abs(some - rows[[59, 0, 7]]).max() <= 1e-5 * np.abs(rows).max()
    rc, nxt, last, ms = p.hip.Prefill(p.toks[:60], 0, True)
    assert rc == 0 and ms > 0 and nxt == int(last.argmax())
    assert M.errors(last[None], p.want[59:60]).max() < TOL[p.dtype]


# ---------------------------------------------------------------------------
# edges of the window
# ---------------------------------------------------------------------------
def needle_model(window, vocab=61, width=128):
    """One latent layer whose scores single out a needle token (vocab - 1): its key points one way, every query looks
    there, and nothing else comes near."""
    layer = M.latent(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=32, q_rank=48, scale=0.1, window=window)
    s = M.model([layer], width=width, vocab=vocab, alpha=1.0)
    rng = np.random.default_rng(8)
    mark = rng.standard_normal(width)
    mark /= np.linalg.norm(mark)

    def embed(a):
        a = a - np.outer(a @ mark, mark)                  # no token carries the mark ...
        a[:, 0] = 2.0                                     # ... all carry a constant first entry
        a[-1] += 14 * mark                                # ... but the needle
        return a

    def dq(a):                                            # queries: the constant, through latent entry 0
        a = 0.05 * a
        a[0, :] = 0
        a[0, 0] = 1.0
        return a

    def dkv(a):                                           # latent entry 0: the mark
        a[0] = 4 * mark
        return a

    def uq(a):
        a = 0.1 * a
        a[[0, 48], 0] = 3.0                               # dim 0 of both heads
        return a

    def uk(a):
        a = 0.1 * a
        a[[0, 32], 0] = 3.0
        return a
    pre = "l0.mix."
    return s, {"embed": embed, pre + "dq": dq, pre + "dkv": dkv, pre + "uq": uq, pre + "uk": uk,
               pre + "o": lambda a: 3 * a}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window", [2, 31, 32, 33, 64, 65, 100])
def test_needle_just_inside_and_outside_the_window(hip, window, dtype):
    s, tweak = needle_model(window)
    p = M.Pair(s, seed=11, eng=hip, dtype=dtype, maxSeq=300, tweak=tweak)
    toks = p.tokens(250) % (s.vocab - 1)
    at = 70
    toks[at] = s.vocab - 1
    want = p.oracle_logits(toks)
    # the oracle with a window one longer or shorter must be far off at the edge, or this test would see nothing
    for wrong, pos in ((window + 1, at + window), (window - 1, at + window - 1)):
        bad = M.oracle_model(s)
        bad["layers"][0]["mixer"]["window"] = wrong
        assert M.errors(O.Oracle(bad, p.values).run(toks), want)[pos] > 10 * TOL[dtype], (wrong, pos)
    for sizes in ([250], [1], [at + window, 180], [at + window - 1, 2], [64, 2, 7]):
        e = M.errors(M.run_portions(p.hip, toks, sizes), want)
        assert e.max() < TOL[dtype], (window, sizes, int(e.argmax()), float(e.max()))
    p.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_needle_far_away_without_a_window(hip, dtype):
    s, tweak = needle_model(0)
    p = M.Pair(s, seed=12, eng=hip, dtype=dtype, maxSeq=1300, tweak=tweak)
    toks = p.tokens(1200) % (s.vocab - 1)
    toks[3] = s.vocab - 1
    want = p.oracle_logits(toks)
    plain = p.oracle_logits(np.where(toks == s.vocab - 1, 0, toks))
    assert M.errors(plain, want)[4:].min() > 5 * TOL[dtype]
    for sizes in ([1200], [700, 2], [1100] + [1] * 100):
        e = M.errors(M.run_portions(p.hip, toks, sizes), want)
        assert e.max() < TOL[dtype], (sizes, int(e.argmax()), float(e.max()))
    p.close()


def test_large_tiles_agree_with_small_ones(hip):
    """Sizes at which a long prompt takes the large tiles of the matrix products and of the experts: one pass against
    portions of 64 tokens, whose products take the small tiles, and the first tokens against the oracle."""
    layers = [with_ff(M.latent(heads=8, dim=128, rot_dim=64, vdim=128, kv_rank=256, q_rank=512, scale=0.07, window=700), C.dense_ff(5632)),
              with_ff(M.delta(heads=32, dim=64, decay_rank=64), C.moe_ff(512, 3, 3, 256)),
              with_ff(M.latent(heads=4, dim=128, rot_dim=64, vdim=128, kv_rank=256, q_rank=512, scale=0.07, window=0, kv_from=0), C.dense_ff(4096))]
    p = M.Pair(M.model(layers, width=2048, vocab=300, alpha=2.2), seed=17, eng=hip, dtype="bfloat16", maxSeq=2100)
    toks = p.tokens(2050)
    assert p.hip.ResetKV() == 0
    rows = list(range(0, 2050, 7)) + list(range(1980, 2050))
    rc, one = p.hip.PrefillLogits(toks, 0, rows)
    assert rc == 0, E.last_error()
    small = M.run_portions(p.hip, toks, [64])
    e = M.errors(one, small[rows].astype(np.float64))
    assert e.max() < 0.02, (rows[int(e.argmax())], float(e.max()))
    e = M.errors(small[:12], p.oracle_logits(toks[:12]))
    assert e.max() < TOL["bfloat16"], float(e.max())
    p.close()


def test_first_tokens(mixed):
    p = mixed
    for n in (1, 2, 3, 4):
        for sizes in ([n], [1]):
            e = M.errors(M.run_portions(p.hip, p.toks[:n], sizes), p.want[:n])
            assert e.max() < TOL[p.dtype], (n, sizes)


# ---------------------------------------------------------------------------
# generation, graphs, errors
# ---------------------------------------------------------------------------
def assert_greedy(p, prompt, toks, tol):
    """Every token is the oracle's choice on the same history, or within tol of it."""
    p.orc.reset()
    lg = p.orc.run(prompt)[-1]
    for i, t in enumerate(toks):
        assert lg[t] >= lg.max() - tol * np.abs(lg).max(), (i, int(t), int(lg.argmax()))
        lg = p.orc.step(int(t))


def test_greedy_generation(mixed):
    p = mixed
    prompt, n = p.toks[:45], 60
    tol = 1e-4 if p.dtype == "float32" else 0.1
    outs = []
    for run in (lambda: p.hip.Generate(prompt, n, useGraph=True), lambda: p.hip.Generate(prompt, n, useGraph=False),
                lambda: p.hip.GeneratePrefill(prompt, n), lambda: p.hip.Generate(prompt, n, useGraph=True)):
        rc, toks = run()
        assert rc == 0, E.last_error()
        assert_greedy(p, prompt, toks, tol)
        outs.append(toks.tolist())
    assert outs[0] == outs[1] == outs[3]              # graph replays are the eager launches
    if p.dtype == "float32":
        assert outs[2] == outs[0]
    # and the sequence can go on where generation stopped
    pos = len(prompt) - 1 + n
    rc, _ = p.hip.DecodeToken(outs[0][-1], pos)
    assert rc == 0, E.last_error()


def test_graph_replays_match_eager_steps(mixed):
    p = mixed
    assert p.hip.ResetKV() == 0
    out = np.empty(p.s.vocab, np.float32)
    for pos in range(12):
        rc, md = p.hip.ValidateGraph(int(p.toks[pos]), pos)
        assert rc == 0 and md == 0.0, (pos, md, E.last_error())
    rc, _ = p.hip.DecodeToken(int(p.toks[12]), 12, out)
    assert rc == 0
    assert M.errors(out[None], p.want[12:13]).max() < TOL[p.dtype]


def test_timing_calls_and_sizes(mixed):
    p = mixed
    assert p.hip.ResetKV() == 0
    rc, ms = p.hip.TimedDecode(1, 5, 10)
    assert rc == 0 and ms > 0
    rc, cls, n = p.hip.ProfileDecode(1, 5, 4)
    assert rc == 0 and n[6] == 1 and n[2] == len(MIXED) and cls[2] > 0
    assert p.hip.WeightBytesPerToken() > 0 and p.hip.KVBytesAt(100) > p.hip.KVBytesAt(0)
    # the measurement gave the sequence up: it only starts over
    assert p.hip.DecodeToken(1, 15)[0] == -4
    assert p.hip.DecodeToken(1, 0)[0] == 0


def test_a_recurrent_sequence_only_continues_where_it_stopped(mixed):
    p = mixed
    assert p.hip.ResetKV() == 0
    assert p.hip.PrefillLogits(p.toks[:10], 0, [])[0] == 0
    assert p.hip.PrefillLogits(p.toks[:5], 3, [])[0] == -4 and "cannot continue" in E.last_error()
    assert p.hip.PrefillLogits(p.toks[10:15], 10, [])[0] == 0


def test_errors(hip):
    s = M.model([M.latent()])
    m = E.NewHIPLayeredInference(hip, s, 16)
    assert m is not None
    assert m.DecodeToken(0, 0)[0] == -4 and "not set" in E.last_error()
    assert m.SetTensor("nothing", np.zeros(3, np.uint16)) == -2
    assert m.SetTensor("embed", np.zeros(3, np.uint16)) == -2
    assert E.lib.mg_num_weights(m._h) == 0 and E.lib.mg_set_layer_range(m._h, 0, 1) == -5
    m.Close()
    for bad in (M.latent(kv_rank=5000), M.latent(kv_from=0), M.delta(dim=300), with_ff(M.delta(), C.moe_ff(8, 2, 3)),
                M.latent(rot_dim=200)):
        assert E.NewHIPLayeredInference(hip, M.model([bad]), 16) is None
        assert "layer 0" in E.last_error()


def test_position_limits(hip):
    p = M.Pair(M.model([M.latent()]), eng=hip, maxSeq=20)
    toks = p.tokens(20)
    want = p.oracle_logits(toks)
    assert M.errors(M.run_portions(p.hip, toks, [19, 1]), want).max() < TOL["float32"]
    assert p.hip.DecodeToken(1, 20)[0] == -2
    assert p.hip.PrefillLogits(toks[:2], 19, [])[0] == -2
    # an attention-only model may go back over positions it holds
    rc, lg = p.hip.PrefillLogits(toks[12:15], 12, [0, 1, 2])
    assert rc == 0 and M.errors(lg, want[12:15]).max() < TOL["float32"]
    p.close()


def test_trace_run_replays_a_folder(hip, tmp_path):
    s = M.model(MIXED[:3], width=96, vocab=50)
    p = M.Pair(s, seed=21)
    M.write_folder(str(tmp_path / "m"), s, p.bits, M.vadonex_config(s))
    a, b = p.tokens(40, 1), p.tokens(9, 2)
    steps = ['{"step": 0, "entries": [{"id": "a", "tokens": %s, "want": [0, 29]}], "end": []}' % a[:30].tolist(),
             '{"step": 1, "entries": [{"id": "a", "tokens": %s, "want": []}], "end": []}' % a[30:39].tolist(),
             '{"step": 2, "entries": [{"id": "a", "tokens": %s, "want": [0]}], "end": ["a"]}' % a[39:].tolist(),
             '{"step": 3, "entries": [{"id": "b", "tokens": %s, "want": [8]}], "end": ["b"]}' % b.tolist()]
    (tmp_path / "out").mkdir()
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32",
                        "--out", str(tmp_path / "out"), "--max-tokens", "40"], input="\n".join(steps) + "\n", text=True,
                       capture_output=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    wa, wb = p.oracle_logits(a), p.oracle_logits(b)
    for step, want in ((0, wa[[0, 29]]), (2, wa[[39]]), (3, wb[[8]])):
        got = np.fromfile(tmp_path / "out" / f"{step}.f32", "<f4").reshape(-1, s.vocab)
        assert M.errors(got, want).max() < TOL["float32"]
    assert not (tmp_path / "out" / "1.f32").exists()
