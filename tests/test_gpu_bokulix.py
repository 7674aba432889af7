"""Bokulix models on the GPU against the plain oracle (bokulix_ref.py): each mechanism alone, whole models of many shapes,
prompts against token-by-token decoding, portions, batches, reused slots, window edges and far keys, and greedy generation
through the framework's entry points. Both precisions: float32 and 16-bit serving."""
import json

import numpy as np
import pytest

from tests import bokulix_ref as R
from tests.test_stack import write_safetensors

pytestmark = pytest.mark.gpu
TOL = {"float32": 1e-4, "bfloat16": 2e-2}  # of the largest value compared
DTYPES = list(TOL)


def blk(heads=4, dim=16, vdim=24, kv_rank=40, window=17, scale=None, experts=5, top=2, ff=36):
    return dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, window=window, scale=dim ** -0.5 if scale is None else scale,
                experts=experts, top=top, ff=ff if experts else 0)


def stack(*blocks, order=None, vocab=101, width=80, taps=3, eps=1e-6, positions=256):
    return dict(blocks=list(blocks), order=list(range(len(blocks))) if order is None else order, vocab=vocab, width=width,
                taps=taps, eps=eps, positions=positions)


def make(c, t, dtype, max_length=None, batch=1):
    from simplellminference_amd.stack import BlockSpec, StackModel, StackSpec
    spec = StackSpec(c["vocab"], c["width"], tuple(BlockSpec("latent", **b) for b in c["blocks"]), taps=c["taps"], eps=c["eps"],
                     max_length=max_length or c["positions"], arrangement="sequential", positions=c["positions"],
                     runs=tuple(c["order"]))
    m = StackModel(spec, dtype=dtype, batch=batch).init()
    for n, v in t.items():
        m.set_tensor(n, v)
    return m


def tokens(n, vocab=101, seed=0):
    return [int(x) for x in np.random.default_rng(seed).integers(0, vocab, n)]


def close(got, want, dtype, what=""):
    assert np.isfinite(got).all(), what
    err, top = float(np.abs(got - want).max()), float(np.abs(want).max())
    assert err <= TOL[dtype] * top, f"{what}: max|d| {err:.3e} of {top:.3e}"


def pieces(m, ids, cut, slot=0, start=0):
    """ids fed from position `start` in portions that end at the places in cut: logits of every position."""
    out, p = [], 0
    for e in list(cut) + [len(ids)]:
        out.append(m.feed([slot], [start + p], [ids[p:e]], [list(range(e - p))]))
        p = e
    return np.concatenate(out)


MODELS = {
    "two-layers": stack(blk(), blk(window=5, top=3)),
    "shared": stack(blk(), blk(heads=6, dim=20, vdim=12, kv_rank=33, window=70, experts=7, top=1), order=[0, 1, 1, 0, 0]),
    "no-feed-forward": stack(blk(experts=0), blk(), blk(experts=0, window=3), order=[0, 1, 2, 0]),
    "all-without": stack(blk(experts=0, top=0), order=[0, 0]),
    "odd-sizes": stack(blk(heads=5, dim=13, vdim=7, kv_rank=11, window=19, experts=3, top=3, ff=21), blk(heads=1, dim=9, vdim=11),
                       width=37, vocab=53, taps=2),
    "ones": stack(blk(heads=1, dim=1, vdim=1, kv_rank=1, window=1, experts=1, top=1, ff=1), width=3, vocab=5, taps=1),
    "one-of-each": stack(blk(heads=1, window=1), blk(experts=1, top=1), blk(heads=17, dim=8, vdim=8), taps=1),
    "wide-heads": stack(blk(heads=2, dim=96, vdim=128, kv_rank=64), blk(heads=3, dim=160, vdim=48, kv_rank=100, window=40),
                        blk(heads=2, dim=24, vdim=136, window=40)),
    "ranks-to-256": stack(blk(kv_rank=130, window=90), blk(kv_rank=192), blk(kv_rank=256, heads=33, dim=4, vdim=4)),
    "ranks-to-448": stack(blk(kv_rank=320), blk(kv_rank=400, window=66), blk(kv_rank=448, window=100)),
    "ranks-past-512": stack(blk(kv_rank=512, window=70), blk(kv_rank=530, window=80)),
    "ranks-past-1024": stack(blk(kv_rank=1100, window=70)),
    "whole-context": stack(blk(window=0), blk(window=500)),
    "long-taps": stack(blk(), blk(experts=0), taps=7),
    "four-taps": stack(blk(), blk(), taps=4, order=[0, 1, 0]),
    "many-experts": stack(blk(experts=70, top=9, ff=16), blk(experts=300, top=2, ff=8), blk(experts=18, top=18, ff=24), width=96),
    "eps": stack(blk(), blk(), eps=0.3),
}


def ref_model(c):
    """window 0: the whole context"""
    return {**c, "blocks": [{**b, "window": b["window"] or 10 ** 9} for b in c["blocks"]]}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_whole_model_against_oracle(gpu, name, dtype):
    """A prompt at once (every position's logits, the residual after every layer), token by token, and by the engine's own
    step."""
    c = MODELS[name]
    t = R.random_tensors(c, 11)
    ids = tokens(107, c["vocab"], 3)
    want, hid = R.forward(ref_model(c), t, ids)
    m = make(c, t, dtype)
    got, h = m.feed([0], [0], [ids], [list(range(len(ids)))], want_hidden=True)
    assert m.runs == len(c["order"]) == len(h)
    for r in range(len(h)):
        close(h[r], hid[r], dtype, f"residual after layer {r}")
    close(got, want, dtype, "prompt")
    close(pieces(m, ids, range(1, len(ids))), want, dtype, "token by token")
    hs = np.concatenate([m.feed([0], [p], [[i]], want_hidden=True)[1] for p, i in enumerate(ids[:9])], axis=1)
    close(hs, hid[:, :9], dtype, "residual, token by token")
    toks, lg = m.predict(ids, 107, want_logits=True)  # the engine's own step, teacher-forced
    assert toks.tolist() == ids
    close(lg, want, dtype, "predict")
    m.close()


# ---------------------------------------------------------------- windows
def strong_pair(window, n, heads, kv_rank):
    """Tokens 1 (query) and 2 (key): the query's score with the key stands out, every other score is 0. The key's value
    is its own direction."""
    c = stack(blk(heads=heads, dim=24, vdim=16, kv_rank=kv_rank, window=window, scale=1.0, experts=0), vocab=8, width=64,
              taps=1, positions=n)
    t = R.random_tensors(c, 17)
    e = np.zeros((8, 64))
    e[0, 20:30], e[1, 0], e[1, 30], e[2, 1], e[3, 40:50] = 1.0, 3.0, 2.0, 3.0, 1.0
    dkv, uk, wq = np.zeros((kv_rank, 64)), np.zeros((heads * 24, kv_rank)), np.zeros((heads * 24, 64))
    dkv[0, 1], dkv[1, 20:30], dkv[2, 40:50], dkv[3, 30] = 1.0, 0.125, 0.125, 0.5  # a latent direction per token
    uk[::24, 0], wq[::24, 0] = 4.0 / np.sqrt(kv_rank), 1.0
    t.update({"embed": e, "pos": 0 * t["pos"], "l0.canon1": 0 * t["l0.canon1"], "l0.mix.dkv": dkv, "l0.mix.uk": uk,
              "l0.mix.q": wq, "l0.mix.dkv.norm": np.ones(kv_rank), "l0.norm1": np.ones(64)})
    return c, t


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 31, 32, 33, 63, 64, 65, 127, 128, 129, 200, 333])
def test_window_edges(gpu, window, dtype):
    """A key that stands out, just inside and just outside the window of the queries after it, at tile borders and beside
    them: in one prompt, in portions that start between key and query, and decoded."""
    n = 420
    c, t = strong_pair(window, n, 5, 70)
    for place in (0, 1, 31, 32, 62, 64):
        ids = [0] * n
        for p in range(7, n, 13):
            ids[p] = 3
        inside, outside = place + window - 1, place + window
        ids[inside], ids[outside], ids[place] = 1, 1, 2
        ids = ids[:outside + 3]
        want = R.forward(c, t, ids)[0]
        if window > 1:  # the edge shows: the two queries differ in the key only
            assert np.abs(want[inside] - want[outside]).max() > 0.2 * np.abs(want).max()
        m = make(c, t, dtype)
        ask = [inside, outside, outside + 2]
        close(m.feed([0], [0], [ids], [ask]), want[ask], dtype, f"prompt, key at {place}")
        if inside > place + 1:
            got = pieces(m, ids, [place + 1, inside])
            close(got, want, dtype, f"portions, key at {place}")
        k = max(inside, 1)
        m.feed([0], [0], [ids[:k]])
        got = np.concatenate([m.feed([0], [p], [[ids[p]]], [[0]]) for p in range(k, len(ids))])
        close(got, want[k:], dtype, f"decoded, key at {place}")
        m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("place,heads,rank", [(p, 18, 96) for p in (0, 63, 64, 255, 256, 700, 1023, 1024)] +
                         [(p, 3, 500) for p in (0, 64, 1100)])
def test_far_key_in_a_long_window(gpu, place, heads, rank, dtype):
    """One key among many hundred, at tile, split and pass borders, found from a prompt row in a later pass and from
    decoded rows; more heads than one workgroup of the decode attention takes, or a rank so large that the merge of its
    splits takes more than one round of loads."""
    n = 1300
    c, t = strong_pair(n, n, heads, rank)
    t["l0.mix.uk"] = t["l0.mix.uk"] * 2
    ids = [0] * n
    ids[place] = 2
    for p in (place + 1, 1280, 1297, 1299):
        ids[p] = 1
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype)
    ask = [place, place + 1, 1280, 1297, 1298, 1299]
    assert np.abs(want[1297] - want[1298]).max() > 0.2 * np.abs(want).max()
    close(m.feed([0], [0], [ids], [ask]), want[ask], dtype, "prompt")
    m.feed([0], [0], [ids[:1290]])
    got = np.concatenate([m.feed([0], [p], [[ids[p]]], [[0]]) for p in range(1290, n)])
    close(got, want[1290:], dtype, "decoded")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens(gpu, dtype):
    """Fewer tokens than the window and the taps: sequences of one to six tokens, as prompts and decoded."""
    c = MODELS["long-taps"]
    t = R.random_tensors(c, 41)
    m = make(c, t, dtype, batch=6)
    reqs = [tokens(n, c["vocab"], 50 + n) for n in range(1, 7)]
    want = [R.forward(c, t, r)[0] for r in reqs]
    got = m.feed(list(range(6)), [0] * 6, reqs, [list(range(len(r))) for r in reqs])
    close(got, np.concatenate(want), dtype, "prompts")
    for i in (5, 2):
        close(pieces(m, reqs[i], range(1, len(reqs[i])), slot=i), want[i], dtype, "decoded")
    m.close()


# ---------------------------------------------------------------- the other mechanisms alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 9])
def test_input_convolution_alone(gpu, taps, dtype):
    """Portions cut inside the taps' reach, down to two tokens and one."""
    c = stack(blk(experts=0), taps=taps, width=48)
    t = R.random_tensors(c, 7)
    t["l0.canon1"] *= 2.0
    ids = tokens(40, c["vocab"], 8)
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype)
    for cut in ([], [1], [2, 3, 4], [1, 2, 3, 5, 8, 13], range(2, 40, 2)):
        close(pieces(m, ids, cut), want, dtype, f"cut {list(cut)}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top", [(1, 1), (4, 1), (4, 4), (9, 3), (64, 2), (65, 5), (256, 16), (257, 17)])
def test_mixture_alone(gpu, experts, top, dtype):
    """The mixer adds nothing and the router reads every channel of the token's row, so the choice is exact in both
    precisions. One row, a batch, and a prompt whose tokens crowd on a few experts."""
    c = stack(blk(experts=experts, top=top, ff=24), width=64, vocab=40, positions=300)
    t = R.random_tensors(c, 12)
    r = np.random.default_rng(13)
    t.update({"l0.norm1": np.zeros(64), "pos": 0 * t["pos"],
              "l0.mlp.router": (r.standard_normal((experts, 64)) * 0.3).astype(np.float16).astype(np.float64)})
    ids = tokens(160, 40, 1) + [7] * 100
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype, 300, batch=5)
    close(m.feed([0], [0], [ids], [list(range(260))]), want, dtype, "prompt")
    close(pieces(m, ids[:12], range(1, 12)), want[:12], dtype, "one row at a time")
    for p in range(6):
        got = m.feed(list(range(5)), [p] * 5, [[ids[20 * b + p]] for b in range(5)], [[0]] * 5)
        close(got, want[[20 * b + p for b in range(5)]], dtype, "five rows")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_expert_weights_alone(gpu, dtype):
    """Equal logits go to the lower index, one logit far above the others takes all the weight, and the weights of the
    chosen add up to 1 whatever the others' logits are."""
    c = stack(blk(experts=6, top=3, ff=16), width=32, vocab=6)
    t = R.random_tensors(c, 14)
    t.update({"l0.norm1": np.zeros(32), "pos": 0 * t["pos"], "l0.mlp.router": np.zeros((6, 32))})
    m = make(c, t, dtype)
    for bias in (np.zeros(6), np.array([0, 0, 30.0, 0, 0, 0]), np.array([2.0, 2.0, 1.5, 1.5, 1.0, 1.0]),
                 np.array([-3.0, 1.0, -1.0, 1.0, 2.0, -2.0])):
        t["l0.mlp.router.b"] = bias
        m.set_tensor("l0.mlp.router.b", bias)
        want = R.forward(c, t, [0, 1, 2, 3, 4, 5] * 3)[0]
        close(m.feed([0], [0], [[0, 1, 2, 3, 4, 5] * 3], [list(range(18))]), want, dtype, f"prompt {bias}")
        close(m.feed([0], [0], [[0]], [[0]]), want[:1], dtype, f"row {bias}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("gate", [-9.0, 0.0, 9.0])
def test_gated_residual_alone(gpu, gate, dtype):
    """Gates nearly shut, half open and open; a nearly shut gate leaves a result whose norm is all in eps."""
    c = stack(blk(), eps=1e-3)
    t = R.random_tensors(c, 15)
    for n in ("l0.rg1", "l0.rg2"):
        t[n] = t[n] * 0.25
        t[n + ".b"] = t[n + ".b"] + gate
    ids = tokens(40, c["vocab"], 9)
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype)
    close(pieces(m, ids, []), want, dtype, "prompt")
    close(pieces(m, ids, range(1, 40)), want, dtype, "token by token")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_learned_positions_alone(gpu, dtype):
    """The same token everywhere: only the position rows differ; the last position is the table's last row."""
    c = stack(blk(window=3), positions=97)
    t = R.random_tensors(c, 16)
    t["pos"] *= 3.0
    ids = [5] * 97
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype)
    close(pieces(m, ids, [90] + list(range(91, 97))), want, dtype)
    m.close()
    from simplellminference_amd._lib import SliError
    with pytest.raises(SliError):
        make(c, t, dtype, max_length=98)


# ---------------------------------------------------------------- portions, batches, slots
PAIR = stack(blk(heads=8, dim=32, vdim=40, kv_rank=72, window=50, experts=9, top=2, ff=40),
             blk(heads=3, dim=20, vdim=12, kv_rank=30, window=130, experts=4, top=3, ff=24), order=[0, 1, 0], width=96, taps=4,
             positions=640)


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_a_prompt(gpu, dtype):
    t = R.random_tensors(PAIR, 13)
    ids = tokens(530, PAIR["vocab"], 14)
    m = make(PAIR, t, dtype)
    want = R.forward(PAIR, t, ids)[0]
    close(pieces(m, ids, []), want, dtype, "whole")
    for cut in (range(2, 530, 2), [31, 62], [32, 64, 96], [33], [127, 129], [255, 257], [511], [512], [513], [1, 529],
                [49, 50, 51, 129, 130, 131]):
        close(pieces(m, ids, cut), want, dtype, f"cut {list(cut)[:4]}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_prompt_past_one_pass(gpu, dtype):
    """A prompt of several passes, and experts crowded enough for every height of their row blocks."""
    c = stack(blk(window=300, experts=2, top=1, ff=200), blk(window=77, experts=8, top=2, ff=72), width=64, positions=2300, vocab=301)
    t = R.random_tensors(c, 23)
    ids = tokens(2200, c["vocab"], 24)
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype)
    ask = list(range(0, 2200, 9)) + [2198, 2199]
    close(m.feed([0], [0], [ids], [ask]), want[ask], dtype, "whole")
    got = pieces(m, ids, [1000, 1720, 1830, 1920, 1980])
    close(got, want, dtype, "portions")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lens", [(5, 70, 33), (1, 2, 3, 130, 64, 31, 32, 97), tuple(range(3, 14))])
def test_batches_of_unequal_requests(gpu, lens, dtype):
    """Prompts as one batch, decoded together, the shorter ones ending earlier: each as it is alone."""
    t = R.random_tensors(PAIR, 15)
    reqs = [tokens(n + 4 + i, PAIR["vocab"], 20 + i) for i, n in enumerate(lens)]
    one = make(PAIR, t, dtype)
    want = [pieces(one, r, []) for r in reqs]
    one.close()
    m = make(PAIR, t, dtype, batch=len(lens))
    B = len(lens)
    got = m.feed(list(range(B)), [0] * B, [r[:n] for r, n in zip(reqs, lens)], [list(range(n)) for n in lens])
    close(got, np.concatenate([w[:n] for w, n in zip(want, lens)]), dtype, "prompts")
    at = list(lens)
    step = 0
    while any(a < len(r) for a, r in zip(at, reqs)):
        live = [i for i in range(B) if at[i] < len(reqs[i])]
        live = live[step % len(live):] + live[:step % len(live)]  # any order of the entries
        got = m.feed(live, [at[i] for i in live], [[reqs[i][at[i]]] for i in live], [[0]] * len(live))
        close(got, np.stack([want[i][at[i]] for i in live]), dtype, f"decode step {step}")
        for i in live:
            at[i] += 1
        step += 1
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_several_sequences(gpu, dtype):
    """Later portions of sequences at different places in one pass: each keeps its own window of earlier rows."""
    t = R.random_tensors(PAIR, 44)
    reqs = [tokens(n, PAIR["vocab"], 60 + n) for n in (400, 90, 222, 17)]
    want = [R.forward(PAIR, t, r)[0] for r in reqs]
    m = make(PAIR, t, dtype, batch=4)
    cuts = [(0, 0, 0, 0), (333, 1, 64, 2), (335, 51, 65, 4), (390, 52, 200, 10), (400, 90, 222, 17)]
    for a, b in zip(cuts, cuts[1:]):
        got = m.feed([3, 0, 2, 1], list(a), [r[x:y] for r, x, y in zip(reqs, a, b)], [list(range(y - x)) for x, y in zip(a, b)])
        close(got, np.concatenate([w[x:y] for w, x, y in zip(want, a, b)]), dtype, f"{a} .. {b}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_sequences_in_lockstep(gpu, dtype):
    """The engine's own batched step over the most sequences it takes, teacher-forced."""
    t = R.random_tensors(PAIR, 28)
    n = 64
    ids = [tokens(6, PAIR["vocab"], 100 + i) for i in range(n)]
    m = make(PAIR, t, dtype, 16, batch=n)
    lg = np.empty((6, n, PAIR["vocab"]), np.float32)
    for p in range(6):
        for i in range(n):
            m.set_state_seq(i, ids[i][p], p, advance=False)
        m.step()
        lg[p] = m.logits()[0]
    for i in (0, 1, 31, 32, 62, 63):
        close(lg[:, i], R.forward(PAIR, t, ids[i])[0], dtype, f"sequence {i}")
    m.close()


def test_more_expanded_rows_than_a_pass_holds(gpu):
    """Two-token portions of many long sequences: their windows together exceed what one pass expands, so the batch runs
    as several passes."""
    c = stack(blk(heads=2, dim=8, vdim=8, kv_rank=16, window=0, experts=2, top=1, ff=8), width=32, vocab=40, positions=1100)
    t = R.random_tensors(c, 31)
    B, n = 40, 1064
    ids = [tokens(n, 40, 200 + b) for b in range(B)]
    m = make(c, t, "bfloat16", batch=B)
    m.feed(list(range(B)), [0] * B, [i[:n - 4] for i in ids])
    got = m.feed(list(range(B)), [n - 4] * B, [i[n - 4:n - 2] for i in ids], [[0, 1]] * B)
    last = m.feed(list(range(B)), [n - 2] * B, [i[n - 2:] for i in ids], [[1]] * B)
    for b in (0, 31, 32, 39):
        want = R.forward(ref_model(c), t, ids[b])[0]
        close(got[2 * b:2 * b + 2], want[n - 4:n - 2], "bfloat16", f"sequence {b}")
        close(last[b:b + 1], want[-1:], "bfloat16", f"sequence {b}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_slots_are_reused(gpu, dtype):
    """A slot's next sequence sees nothing of the one before, whatever its length, and other slots go on."""
    t = R.random_tensors(PAIR, 16)
    a, b, c2 = tokens(90, seed=1), tokens(40, seed=2), tokens(60, seed=3)
    want = {n: R.forward(PAIR, t, s)[0] for n, s in (("a", a), ("b", b), ("c", c2))}
    m = make(PAIR, t, dtype, batch=3)
    m.feed([1, 2], [0, 0], [a, c2[:50]])
    got = pieces(m, b, [3, 20, 21, 22], slot=1)
    close(got, want["b"], dtype, "after a longer sequence")
    got = m.feed([1], [0], [[a[0]]], [[0]])
    close(got, want["a"][:1], dtype, "first token in a used slot")
    got = m.feed([2], [50], [c2[50:]], [list(range(10))])
    close(got, want["c"][50:], dtype, "the slot beside it")
    for p in range(40):  # decoding from position 0 in a used slot
        got = m.feed([1, 0], [p, p], [[b[p]], [a[p]]], [[0], [0]])
        close(got, np.stack([want["b"][p], want["a"][p]]), dtype, f"position {p}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, dtype):
    t = R.random_tensors(PAIR, 18)
    ids = tokens(500, PAIR["vocab"], 19)
    want = R.forward(PAIR, t, ids)[0]
    m = make(PAIR, t, dtype)
    close(m.predict(ids, 500, want_logits=True)[1], want, dtype)
    close(pieces(m, ids, [3] + list(range(4, 500))), want, dtype, "feed")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff", [(64, 16000), (4160, 40), (2048, 1100)])
def test_wide_layers(gpu, width, ff, dtype):
    """Expert rows too long, and a model too wide, for the one-row launches; and one that fills them."""
    c = stack(blk(window=9, ff=ff, experts=3), width=width, vocab=600, positions=40)
    t = R.random_tensors(c, 25)
    a, b = tokens(12, c["vocab"], 26), tokens(12, c["vocab"], 27)
    want = [R.forward(c, t, i)[0] for i in (a, b)]
    m = make(c, t, dtype, 40, batch=2)
    close(pieces(m, a, []), want[0], dtype, "prompt")
    close(pieces(m, a, range(1, 12)), want[0], dtype, "token by token")
    m.feed([0, 1], [0, 0], [a[:8], b[:8]])
    for p in range(8, 12):
        got = m.feed([0, 1], [p, p], [[a[p]], [b[p]]], [[0], [0]])
        close(got, np.stack([w[p] for w in want]), dtype, f"batch, position {p}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_passes_repeat_bit_for_bit(gpu, dtype):
    """The same prompt and the same decode steps give the same bits every time, with other work in between."""
    t = R.random_tensors(PAIR, 21)
    ids, other = tokens(300, seed=4), tokens(77, seed=5)
    m = make(PAIR, t, dtype, 512, batch=2)
    ref = None
    for i in range(12):
        got = np.concatenate([m.feed([0], [0], [ids], [list(range(0, 300, 7))]), m.feed([0], [300], [[5]], [[0]])])
        m.feed([1], [0], [other[:1 + 6 * i]])
        ref = got if ref is None else ref
        assert np.array_equal(got.view(np.uint32), ref.view(np.uint32)), i
    m.close()


# ---------------------------------------------------------------- the framework's entry points
@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation(gpu, dtype):
    """predict, predict_prefill, predict_batch and predict_batch_prefill: the oracle's greedy tokens, while its choice is
    not closer than the tolerance."""
    t = R.random_tensors(PAIR, 22)
    prompts = [tokens(n, seed=30 + n) for n in (1, 9, 37)]
    N = 60
    want = [R.greedy(PAIR, t, p, N) for p in prompts]
    sure = []
    for w, p in zip(want, prompts):
        lg = R.forward(PAIR, t, w)[0]
        two = np.sort(lg, axis=1)[:, -2:]
        unsure = np.nonzero(two[:, 1] - two[:, 0] < 4 * TOL[dtype] * np.abs(lg).max())[0]
        unsure = [u for u in unsure if u >= len(p) - 1]
        sure.append(min(unsure[0] + 1, N) if unsure else N)
    one = make(PAIR, t, dtype, 64)
    for p, w, n in zip(prompts, want, sure):
        assert one.predict(p, N).tolist()[:n] == w[:n]
        assert one.predict_prefill(p, N).tolist()[:n] == w[:n]
    one.close()
    m = make(PAIR, t, dtype, 64, batch=3)
    for got in (m.predict_batch(prompts, N), m.predict_batch_prefill(prompts, N)):
        for g, w, n in zip(got, want, sure):
            assert g.tolist()[:n] == w[:n]
    m.close()


def bokulix_folder(path, c, t):
    """c as a config.json of the Bokulix architecture, with its tensors under the names of the layers that own them."""
    layers, first = [], {}
    for i, k in enumerate(c["order"]):
        b = c["blocks"][k]
        mlp = {"kind": "moe", "expert": {"ff": b["ff"]}, "router": {"experts": b["experts"], "top": b["top"]}} if b["experts"] else None
        e = {"type": "latent_attention", "mlp": mlp,
             "mixer": {**{n: b[n] for n in ("heads", "dim", "vdim", "kv_rank", "scale")}, "mask": {"size": b["window"]}}}
        if k in first:
            e["weights_of"] = first[k]
        first.setdefault(k, i)
        layers.append(e)
    cfg = {"architecture": "Bokulix", "vocab": c["vocab"], "width": c["width"], "canon": {"taps": c["taps"]},
           "norm": {"eps": c["eps"]}, "max_positions": c["positions"], "layers": layers}
    (path / "config.json").write_text(json.dumps(cfg))
    named = {}
    for n, v in t.items():
        k, dot, leaf = n.partition(".")
        own = dot and k[1:].isdigit()
        named[f"l{first[int(k[1:])]}.{leaf}" if own else n] = v
    write_safetensors(path / "model.safetensors", named)


def bf16(t):
    return {k: ((np.asarray(v, np.float32).view(np.uint32) & 0xFFFF0000).view(np.float32)).astype(np.float64)
            for k, v in t.items()}


@pytest.mark.parametrize("dtype", DTYPES)
def test_folder_trace_and_command_line(gpu, dtype, tmp_path, capsys, monkeypatch):
    """A bfloat16 model folder through the registry, the trace replay and the command line."""
    import io

    from simplellminference_amd import trace
    from simplellminference_amd.__main__ import main
    c = {**PAIR, "order": [1, 1, 0, 1, 0], "positions": 70}
    t = bf16(R.random_tensors(c, 23))
    bokulix_folder(tmp_path, c, t)
    a, b = tokens(50, seed=6), tokens(23, seed=7)
    wa, wb = R.forward(c, t, a)[0], R.forward(c, t, b)[0]
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:48], "want": [0, 47, 20]},
                                     {"id": "y", "tokens": b[:22], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": b[22:], "want": [0]}, {"id": "x", "tokens": a[48:49], "want": [0]}],
              "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": a[49:], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": n, "tokens": b[:5 + i], "want": [4]} for i, n in enumerate("pqr")], "end": list("pqr")}]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    assert trace.main(["--model", str(tmp_path), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "80"]) == 0
    assert capsys.readouterr().out.split() == "done 0 done 1 done 2 done 3".split()
    V = c["vocab"]
    for n, want in ((0, wa[[0, 47, 20]]), (1, np.stack([wb[22], wa[48]])), (2, wa[[49]]), (3, wb[[4, 4, 4]])):
        close(np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, V), want, dtype, f"step {n}")
    argv = ["--model", str(tmp_path), "--dtype", dtype, "--max-length", "12", "--prompt", "3 1 4", "--prompt", "1 5"]
    outs = []
    for extra in ([], ["--no-prefill"]):
        assert main(argv + extra) == 0
        outs.append(capsys.readouterr().out)
    lines = [[int(x) for x in ln.split()] for ln in outs[0].strip().split("\n")]
    assert [len(x) for x in lines] == [12, 12] and lines[0][:3] == [3, 1, 4] and lines[1][:2] == [1, 5]
    if dtype == "float32":
        assert outs[0] == outs[1]


def test_errors_come_from_the_host(gpu):
    from simplellminference_amd._lib import SliError
    from simplellminference_amd.stack import BlockSpec, StackModel, StackSpec
    t = R.random_tensors(PAIR, 24)
    m = make(PAIR, t, "bfloat16", 32, batch=2)
    for args in (([2], [0], [[1]]), ([0, 0], [0, 0], [[1], [1]]), ([0], [32], [[1]]), ([0], [0], [[101]]), ([0], [0], [[1] * 33])):
        with pytest.raises(SliError):
            m.feed(*args)
    for name, v in (("l0.mix.k", np.zeros(3)), ("l0.mix.q", np.zeros(3)), ("l0.mlp.e9.up", np.zeros((40, 96))),
                    ("l2.mix.q", np.zeros(3)), ("l0.norm1", np.full(96, 1e6))):
        with pytest.raises(SliError):
            m.set_tensor(name, v)
    m.close()

    def refused(*blocks, **kw):
        with pytest.raises(SliError):
            StackModel(StackSpec(8, 8, tuple(BlockSpec(*b[0], **b[1]) for b in blocks), **kw)).init()
    good = (("latent", 2, 4, 4), dict(kv_rank=8, experts=2, top=1, ff=4))
    with pytest.raises(SliError, match="not loaded"):
        StackModel(StackSpec(8, 8, (BlockSpec(*good[0], **good[1]),), arrangement="sequential")).init().feed([0], [0], [[1]])
    refused(good)  # latent attention in a parallel block
    for bad in (dict(top=3), dict(experts=0), dict(kv_rank=0), dict(kv_rank=2049), dict(top=0), dict(ff=0), dict(window=-1)):
        refused((good[0], {**good[1], **bad}), arrangement="sequential")
    refused((("attention", 2, 4, 4), dict(kv_heads=1)), arrangement="sequential")
    refused(good, arrangement="sequential", runs=(0, 1))
    refused(good, arrangement="sequential", positions=4, max_length=8)
