"""Block-stack models on the GPU against the plain oracle (stack_ref.py): each mechanism alone, whole models of many
shapes, prompts against token-by-token decoding, portions, batches, reused slots, far keys and edges, and greedy
generation through the framework's entry points. Both precisions: float32 and 16-bit serving."""
import json

import numpy as np
import pytest

from tests import stack_ref as R
from tests.test_stack import write_safetensors

pytestmark = pytest.mark.gpu
TOL = {"float32": 1e-4, "bfloat16": 2e-2}  # of the largest value compared
DTYPES = list(TOL)


def att(heads=4, kv_heads=2, dim=32, vdim=32, scale=None, ff=48, ff_limit=1.2):
    return dict(mixer="attention", heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, ff=ff, ff_limit=ff_limit,
                scale=dim ** -0.5 if scale is None else scale)


def ret(heads=2, dim=32, vdim=24, rot_dims=None, rot_base=1e4, decay=None, ff=48, ff_limit=1.2):
    return dict(mixer="retention", heads=heads, dim=dim, vdim=vdim, rot_dims=dim if rot_dims is None else rot_dims,
                rot_base=rot_base, ff=ff, ff_limit=ff_limit,
                decay=decay or tuple(1.0 - 2.0 ** -(2 + 2 * h) for h in range(heads)))


def stack(*blocks, vocab=101, width=80, taps=4, loop=(0, 0, 1), eps=1e-6, emb_scale=1.5, residual_mult=0.4):
    return dict(blocks=list(blocks), vocab=vocab, width=width, taps=taps, loop=loop, eps=eps, emb_scale=emb_scale,
                residual_mult=residual_mult)


def make(c, t, dtype, max_length=256, batch=1):
    from simplellminference_amd.stack import BlockSpec, StackModel, StackSpec
    blocks = tuple(BlockSpec(**{k: v for k, v in b.items()}) for b in c["blocks"])
    spec = StackSpec(c["vocab"], c["width"], blocks, tuple(c["loop"]), c["taps"], c["eps"], c["emb_scale"],
                     c["residual_mult"], max_length)
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


def pieces(m, ids, cut, slot=0):
    """ids fed in portions that end at the places in cut: logits of every position."""
    out, p = [], 0
    for e in list(cut) + [len(ids)]:
        out.append(m.feed([slot], [p], [ids[p:e]], [list(range(e - p))]))
        p = e
    return np.concatenate(out)


MODELS = {
    "attention": stack(att()),
    "retention": stack(ret()),
    "mixed-loop": stack(ret(), att(), att(heads=6, kv_heads=3, dim=20, vdim=12), ret(heads=3, dim=24, vdim=40, rot_dims=16),
                        loop=(1, 3, 3)),
    "loop-first": stack(att(ff=0), ret(ff=0), loop=(0, 1, 2)),
    "loop-all": stack(ret(ff=20), att(ff=36), loop=(0, 2, 2), taps=3),
    "odd-sizes": stack(att(heads=5, kv_heads=1, dim=13, vdim=7, ff=21), ret(heads=1, dim=17, vdim=9, rot_dims=6, ff=0),
                       width=37, vocab=53, taps=2),
    "ones": stack(att(heads=1, kv_heads=1, dim=1, vdim=1, ff=1), ret(heads=1, dim=2, vdim=1, ff=1), width=3, vocab=5, taps=1),
    "no-rotation": stack(ret(rot_dims=0), ret(rot_dims=2, rot_base=7.0)),
    "wide-heads": stack(att(heads=2, kv_heads=2, dim=96, vdim=128), att(heads=3, kv_heads=1, dim=160, vdim=48),
                        ret(heads=1, dim=130, vdim=70, rot_dims=64)),
    "long-taps": stack(att(), ret(), taps=7),
    "groups": stack(att(heads=12, kv_heads=4), att(heads=16, kv_heads=2, dim=16, vdim=16), att(heads=7, kv_heads=1)),
    "eps": stack(ret(), att(), eps=0.3, residual_mult=1.0, emb_scale=0.1),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_whole_model_against_oracle(gpu, name, dtype):
    """A prompt at once (every position's logits, the residual after every run) and token by token."""
    c = MODELS[name]
    t = R.random_tensors(c, 11)
    ids = tokens(71, c["vocab"], 3)
    want, hid = R.forward(c, t, ids)
    m = make(c, t, dtype)
    got, h = m.feed([0], [0], [ids], [list(range(len(ids)))], want_hidden=True)
    assert m.runs == len(R.order(c)) == len(h)
    for r in range(len(h)):
        close(h[r], hid[r], dtype, f"residual after run {r}")
    close(got, want, dtype, "prompt")
    close(pieces(m, ids, range(1, len(ids))), want, dtype, "token by token")
    toks, lg = m.predict(ids, 71, want_logits=True)  # the engine's own step, teacher-forced
    assert toks.tolist() == ids
    close(lg, want, dtype, "predict")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim", [20, 64, 128])
def test_attention_weights_read_out(gpu, dim, dtype):
    """One head whose values are one-hot per position: the block's output is the row of attention weights itself.
    Bias, sink and one far key that stands out, in a prompt and in decoding."""
    n = 150
    c = stack(dict(att(heads=1, kv_heads=1, dim=dim, vdim=n, ff=0), scale=0.25), vocab=n, width=n, taps=1, eps=0.0,
              emb_scale=1.0, residual_mult=1.0)
    t = R.random_tensors(c, 5)
    t.update({"embed": np.eye(n), "l0.norm1": np.float64(1.0), "l0.canon1": np.zeros((n, 1)), "l0.mix.o": np.eye(n),
              "l0.mix.v": np.eye(n) / 4, "l0.mix.r1": np.array([0.75]), "l0.mix.r2": np.array([0.5]),
              "l0.mix.sink": np.array([1.0])})
    ids = list(range(n))
    h0 = R.rms(np.eye(n), 0.0)
    q, k = h0 @ t["l0.mix.q"].T, h0 @ t["l0.mix.k"].T
    k[3] = 8.0 * q[140] / np.linalg.norm(q[140])  # one query, one far key
    t["l0.mix.k"] = (k / h0[0, 0]).T.astype(np.float16).astype(np.float64)
    _, hid = R.forward(c, t, ids)
    want = (hid[0] - np.eye(n)) / (np.sqrt(n) / 4)
    assert want[140, 3] > 0.2  # the far key shows
    m = make(c, t, dtype)
    _, h = m.feed([0], [0], [ids], want_hidden=True)
    assert np.abs((h[0] - np.eye(n)) / (np.sqrt(n) / 4) - want).max() < (1e-5 if dtype == "float32" else 4e-3)
    rows = []
    for p in ids:
        rows.append(m.feed([0], [p], [[p]], want_hidden=True)[1][0, 0])
    assert np.abs((np.array(rows) - np.eye(n)) / (np.sqrt(n) / 4) - want).max() < (1e-5 if dtype == "float32" else 4e-3)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_with_one_key(gpu, dtype):
    """At the first token the only key shares the softmax with the sink."""
    c = stack(att(heads=2, kv_heads=1, ff=0), taps=1, residual_mult=1.0)
    t = R.random_tensors(c, 6)
    for sink in (-30.0, 0.0, 6.0):
        t["l0.mix.sink"] = np.array([sink, -sink])
        m = make(c, t, dtype)
        close(m.feed([0], [0], [[9]], [[0]]), R.forward(c, t, [9])[0], dtype, f"sink {sink}")
        m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 8])
def test_input_convolution_alone(gpu, taps, dtype):
    """Mixer and feed-forward read convolved rows; portions cut inside the taps' reach, down to one token."""
    c = stack(att(), taps=taps, width=48)
    t = R.random_tensors(c, 7)
    t["l0.canon1"] *= 2.0
    t["l0.canon2"] *= 2.0
    ids = tokens(40, c["vocab"], 8)
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype)
    for cut in ([], [1], [2, 3, 4], [1, 2, 3, 5, 8, 13], range(2, 40, 2)):
        close(pieces(m, ids, cut), want, dtype, f"cut {list(cut)}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_retention_alone_long(gpu, dtype):
    """Slow and fast decays over several chunks and passes, then decoding from the state they left."""
    c = stack(ret(heads=4, dim=48, vdim=33, rot_dims=32, decay=(0.5, 0.9, 0.99, 0.9995), ff=0), width=64)
    t = R.random_tensors(c, 9)
    ids = tokens(620, c["vocab"], 10)
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype, 640)
    close(pieces(m, ids, [600] + list(range(601, 620))), want, dtype, "prompt, then decoding")
    close(pieces(m, ids, [1, 32, 63, 65, 300, 513]), want, dtype, "portions")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_feed_forward_clamp_alone(gpu, dtype):
    c = stack(dict(att(ff=64, ff_limit=0.5)), taps=1)
    t = R.random_tensors(c, 12)
    t["l0.mix.o"] = np.zeros_like(t["l0.mix.o"])
    t["l0.mlp.gate"] *= 3.0
    t["l0.mlp.up"] *= 3.0
    ids = tokens(33, c["vocab"], 1)
    m = make(c, t, dtype)
    close(m.feed([0], [0], [ids], [list(range(33))]), R.forward(c, t, ids)[0], dtype)
    m.close()


PAIR = stack(ret(heads=2, dim=64, vdim=40), att(heads=8, kv_heads=2, dim=64, vdim=64), ret(heads=3, dim=20, vdim=12, rot_dims=10),
             loop=(0, 2, 2), width=96)


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_a_prompt(gpu, dtype):
    t = R.random_tensors(PAIR, 13)
    ids = tokens(530, PAIR["vocab"], 14)
    m = make(PAIR, t, dtype, 600)
    want = pieces(m, ids, [])
    close(want, R.forward(PAIR, t, ids)[0], dtype, "whole")
    for cut in (range(2, 530, 2), [31, 62], [32, 64, 96], [33], [127, 129], [255, 257], [511], [512], [513], [1, 529]):
        close(pieces(m, ids, cut), want, dtype, f"cut {list(cut)[:4]}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_wide_projections(gpu, dtype):
    """Feed-forward and output head wide enough for every GEMM tiling, in passes of 1024, 512, 256, 128 and 96 rows and
    with wanted-row counts that are no multiple of a tile."""
    c = stack(ret(ff=8300), att(ff=40), width=64, vocab=1001)
    t = R.random_tensors(c, 23)
    ids = tokens(1060, c["vocab"], 24)
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype, 1100)
    close(pieces(m, ids, []), want, dtype, "whole")
    for cut in ([500, 720, 830, 920], [213, 300, 400, 550]):
        close(pieces(m, ids, cut), want, dtype, f"cut {cut}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_output_rows(gpu, dtype):
    """An output projection whose input [mixer; feed-forward] is longer than 16384: with and without the shapes that the
    fused batch-1 launches take, alone and as a batch."""
    c = stack(att(ff=16300), ret(vdim=33, ff=16370), ret(vdim=32, ff=16384), width=32, vocab=61)
    t = R.random_tensors(c, 25)
    a, b = tokens(45, c["vocab"], 26), tokens(45, c["vocab"], 27)
    want = [R.forward(c, t, i)[0] for i in (a, b)]
    m = make(c, t, dtype, 64, batch=2)
    close(pieces(m, a, range(1, 45)), want[0], dtype, "token by token")
    m.feed([0, 1], [0, 0], [a[:40], b[:40]])
    for p in range(40, 45):
        got = m.feed([0, 1], [p, p], [[a[p]], [b[p]]], [[0], [0]])
        close(got, np.stack([w[p] for w in want]), dtype, f"batch, position {p}")
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
def test_slots_are_reused(gpu, dtype):
    """A slot's next sequence sees nothing of the one before, whatever its length, and other slots go on."""
    t = R.random_tensors(PAIR, 16)
    a, b, c2 = tokens(90, seed=1), tokens(40, seed=2), tokens(60, seed=3)
    fresh = make(PAIR, t, dtype)
    want = {n: pieces(fresh, s, []) for n, s in (("a", a), ("b", b), ("c", c2))}
    fresh.close()
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
@pytest.mark.parametrize("place", [0, 1, 30, 31, 32, 33, 127, 128, 255, 256, 511, 512, 699])
def test_far_keys_at_edges(gpu, place, dtype):
    """One key, `place`, stands out for the query tokens that follow: found from far away, at tile, split and pass edges,
    from a prompt row and from a decoded one."""
    c = stack(att(heads=8, kv_heads=2, dim=64, vdim=32, ff=0, scale=1.0), taps=1, vocab=8, width=64, residual_mult=1.0)
    t = R.random_tensors(c, 17)
    # q and k along one direction, used by token 1 (query) and token 2 (key) only: every other score is 0
    e = np.zeros((8, 64))
    e[0, 2:10], e[1, 0], e[2, 1], e[3, 10:20] = 1.0, 3.0, 3.0, 1.0
    wq, wk = np.zeros((8 * 64, 64)), np.zeros((2 * 64, 64))
    wq[::64, 0], wk[::64, 1] = 1.0, 0.25
    t.update({"embed": e, "l0.mix.q": wq, "l0.mix.k": wk, "l0.canon1": np.zeros((64, 1)), "l0.norm1": np.float64(1.0),
              "l0.mix.r1": np.full(8, 0.25), "l0.mix.r2": np.full(8, 0.5), "l0.mix.sink": np.linspace(-2, 5, 8)})
    t["l0.mix.r1"][3] = 1.5
    ids = [0] * 720
    ids[place] = 2
    for p in range(place + 1, 720, 97):
        ids[p] = 1
    ids[715] = ids[719] = 1
    ask = sorted({p for p in range(720) if ids[p] == 1} | {place, 719})
    # (only the asked rows: the oracle's attention is quadratic)
    x = e[np.array(ids)] * c["emb_scale"]
    h = R.rms(x, c["eps"])
    want = []
    for i in ask:
        o = []
        for n in range(8):
            k, v = h @ wk[64 * (n // 4):][:64].T, h @ t["l0.mix.v"][32 * (n // 4):][:32].T
            s = (k[:i + 1] @ (wq[64 * n:64 * n + 64] @ h[i])) - t["l0.mix.r1"][n] * np.log(1 + 0.5 * (i - np.arange(i + 1)))
            w = np.exp(s)
            o.append(w @ v[:i + 1] / (w.sum() + np.exp(t["l0.mix.sink"][n])))
        y = x[i] + np.concatenate(o) @ t["l0.mix.o"].T
        want.append((R.rms(y, c["eps"]) * t["final.norm"]) @ t["head"].T)
    want = np.array(want)
    m = make(c, t, dtype, 768)
    close(m.feed([0], [0], [ids], [ask]), want, dtype, "prompt")
    m.feed([0], [0], [ids[:710]])
    got = np.concatenate([m.feed([0], [p], [[ids[p]]], [[0]]) for p in range(710, 720)])
    for j, p in enumerate(ask):
        if p >= 710:
            close(got[p - 710], want[j], dtype, f"decoded {p}")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, dtype):
    c = stack(ret(heads=2, dim=32, vdim=32), att(heads=4, kv_heads=2, dim=64, vdim=64), width=64)
    t = R.random_tensors(c, 18)
    ids = tokens(400, c["vocab"], 19)
    want = R.forward(c, t, ids)[0]
    m = make(c, t, dtype, 2048)  # (several context splits per head, most of them past the live context)
    lg = m.predict(ids, 400, want_logits=True)[1]
    close(lg, want, dtype)
    close(pieces(m, ids, [3] + list(range(4, 400))), want, dtype, "feed")
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
        m.feed([1], [0], [other[:1 + 7 * i]])
        ref = got if ref is None else ref
        assert np.array_equal(got.view(np.uint32), ref.view(np.uint32)), i
    m.close()


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


def rugudra_folder(path, c, t):
    """c as a config.json of the Rugudra architecture, with its tensors."""
    layers = []
    for b in c["blocks"]:
        mlp = {"kind": "dense", "ff": b["ff"], "limit": b["ff_limit"]} if b["ff"] else None
        mx = {k: b[k] for k in ("heads", "dim", "vdim")}
        if b["mixer"] == "attention":
            mx.update(kv_heads=b["kv_heads"], scale=b["scale"])
        else:
            mx.update(decay=list(b["decay"]), rot={"base": b["rot_base"], "dims": b["rot_dims"]})
        layers.append({"type": b["mixer"], "mixer": mx, "mlp": mlp})
    cfg = {"architecture": "Rugudra", "vocab": c["vocab"], "width": c["width"], "canon": {"taps": c["taps"]},
           "embedding": {"scale": c["emb_scale"]}, "norm": {"eps": c["eps"]}, "residual_mult": c["residual_mult"],
           "loop": dict(zip(("start", "stop", "times"), c["loop"])), "layers": layers}
    (path / "config.json").write_text(json.dumps(cfg))
    write_safetensors(path / "model.safetensors", t)


def bf16(t):
    return {k: ((np.asarray(v, np.float32).view(np.uint32) & 0xFFFF0000).view(np.float32)).astype(np.float64)
            for k, v in t.items()}


@pytest.mark.parametrize("dtype", DTYPES)
def test_folder_trace_and_command_line(gpu, dtype, tmp_path, capsys, monkeypatch):
    """A bfloat16 model folder through the registry, the trace replay and the command line."""
    import io

    from simplellminference_amd import trace
    from simplellminference_amd.__main__ import main
    c, t = PAIR, bf16(R.random_tensors(PAIR, 23))
    rugudra_folder(tmp_path, c, t)
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


def test_folder_without_a_feed_forward(gpu, tmp_path):
    """A null feed-forward, with and without the second sublayer's norm and taps in the file."""
    from simplellminference_amd.registry import load_model
    c = stack(att(ff=0), ret(ff=24), width=40)
    t = bf16(R.random_tensors(c, 29))
    ids = tokens(20, c["vocab"], 30)
    want = R.forward(c, t, ids)[0]
    for extra in ({}, {"l0.norm2": np.float64(3.0), "l0.canon2": np.ones((40, 4))}):
        rugudra_folder(tmp_path, c, {**t, **extra})
        m = load_model(str(tmp_path), "float32", 32)
        close(m.feed([0], [0], [ids], [list(range(20))]), want, "float32")
        m.close()


def test_errors_come_from_the_host(gpu):
    from simplellminference_amd._lib import SliError
    t = R.random_tensors(PAIR, 24)
    m = make(PAIR, t, "bfloat16", 32, batch=2)
    for args in (([2], [0], [[1]]), ([0, 0], [0, 0], [[1], [1]]), ([0], [32], [[1]]), ([0], [0], [[101]]), ([0], [0], [[1] * 33])):
        with pytest.raises(SliError):
            m.feed(*args)
    with pytest.raises(SliError):
        m.feed([0], [0], [[1, 2]], [[2]])
    with pytest.raises(SliError):
        m.set_tensor("l0.mix.nothing", np.zeros(3))
    with pytest.raises(SliError):
        m.set_tensor("l0.mix.q", np.zeros(3))
    with pytest.raises(SliError):  # values fp16 weights cannot hold
        m.set_tensor("l0.norm1", np.float32(1e6))
    for call in (lambda: m.set_exec("persist"), lambda: m.kv(0, 0, 1), m.time_families):
        with pytest.raises((SliError, AttributeError, ZeroDivisionError)):
            call()
    m.close()
    from simplellminference_amd.stack import BlockSpec, StackModel, StackSpec
    with pytest.raises(SliError, match="not loaded"):
        StackModel(StackSpec(8, 8, (BlockSpec("attention", 1, 4, 4, kv_heads=1),))).init().feed([0], [0], [[1]])
    with pytest.raises(SliError):
        StackModel(StackSpec(8, 8, (BlockSpec("attention", 3, 4, 4, kv_heads=2),))).init()
