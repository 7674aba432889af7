"""Block-stack models without a GPU: the folder readers, the registry, the slot map, the trace replay's bookkeeping over
a recording stand-in, and the oracle's own mechanisms on cases that can be worked out by hand."""
import json
import struct

import numpy as np
import pytest

from tests import stack_ref as R


def write_safetensors(path, tensors, dtype="BF16"):
    head, data = {"__metadata__": {"format": "pt"}}, b""
    for n, v in tensors.items():
        v = np.asarray(v, np.float32)
        raw = (v.view(np.uint32) >> 16).astype("<u2").tobytes() if dtype == "BF16" else v.astype("<f4").tobytes()
        head[n] = {"dtype": dtype, "shape": list(v.shape), "data_offsets": [len(data), len(data) + len(raw)]}
        data += raw
    h = json.dumps(head).encode()
    path.write_bytes(struct.pack("<Q", len(h)) + h + data)


CFG = {
    "architecture": "Rugudra", "vocab": 31, "width": 24, "embedding": {"scale": 2.0}, "norm": {"eps": 1e-5},
    "residual_mult": 0.5, "canon": {"taps": 3}, "loop": {"start": 1, "stop": 2, "times": 3},
    "layers": [
        {"type": "attention", "mixer": {"heads": 6, "kv_heads": 3, "dim": 10, "vdim": 7, "scale": 0.3}, "mlp": None},
        {"type": "retention", "mixer": {"heads": 3, "dim": 12, "vdim": 5, "decay": [0.9, 0.5, 0.99],
                                        "rot": {"base": 500.0, "dims": 8}},
         "mlp": {"kind": "dense", "ff": 20, "limit": 1.5}},
    ],
}


def test_safetensors_reader(tmp_path):
    from simplellminference_amd.checkpoint import SafeTensors
    want = {"a": np.arange(6, dtype=np.float32).reshape(2, 3) / 4, "s": np.float32(1.5)}
    for dt in ("BF16", "F32"):
        p = tmp_path / f"{dt}.safetensors"
        write_safetensors(p, want, dt)
        st = SafeTensors(str(p))
        assert sorted(st.names()) == ["a", "s"] and st.shape("a") == (2, 3) and st.shape("s") == ()
        for n, v in want.items():
            assert np.array_equal(st.get(n), v)
    p = tmp_path / "bad.safetensors"
    p.write_bytes(b"\xff" * 8)
    with pytest.raises(ValueError):
        SafeTensors(str(p))


def test_config_to_spec():
    from simplellminference_amd.stack import rugudra_spec
    s = rugudra_spec(CFG, 77)
    assert (s.vocab_size, s.width, s.taps, s.max_length, s.loop) == (31, 24, 3, 77, (1, 2, 3))
    assert s.order == [0, 1, 1, 1]
    a, r = s.blocks
    assert (a.mixer, a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.ff) == ("attention", 6, 3, 10, 7, 0.3, 0)
    assert (r.mixer, r.decay, r.rot_dims, r.rot_base, r.ff, r.ff_limit) == ("retention", (0.9, 0.5, 0.99), 8, 500.0, 20, 1.5)
    assert (s.eps, s.emb_scale, s.residual_mult) == (1e-5, 2.0, 0.5)
    no_loop = {k: v for k, v in CFG.items() if k != "loop"}
    assert rugudra_spec(no_loop, 5).order == [0, 1]
    bad = json.loads(json.dumps(CFG))
    bad["layers"][1]["mlp"]["kind"] = "other"
    with pytest.raises(ValueError):
        rugudra_spec(bad, 5)
    bad = json.loads(json.dumps(CFG))
    bad["layers"][0]["type"] = "other"
    with pytest.raises(ValueError):
        rugudra_spec(bad, 5)


def test_registry_names_and_unknown(tmp_path):
    from simplellminference_amd.registry import architectures, load_model
    assert architectures() == ["Bokulix", "Llama", "Rugudra"]
    (tmp_path / "config.json").write_text('{"architecture": "Nothing"}')
    with pytest.raises(ValueError, match="unknown architecture"):
        load_model(str(tmp_path))


def test_slot_map():
    from simplellminference_amd.sequences import SlotMap
    m = SlotMap(2)
    assert m.begin("a") == 0 and m.begin("b") == 1
    with pytest.raises(RuntimeError):
        m.begin("c")
    with pytest.raises(ValueError):
        m.begin("a")
    assert m.advance("a", 5) == (0, 0) and m.advance("a", 1) == (0, 5) and m.advance("b", 2) == (1, 0)
    m.end("a")
    assert "a" not in m and m.begin("c") == 0 and m.advance("c", 3) == (0, 0) and len(m) == 2


def test_trace_runner_bookkeeping(monkeypatch):
    """Slots, positions, wanted rows in the order asked for, and a larger batch once the earlier one has ended."""
    import simplellminference_amd.trace as T
    made, calls = [], []

    class Fake:
        local_vocab = 4

        def __init__(self, batch):
            self.batch = batch

        def feed(self, slots, starts, tokens, want):
            calls.append((list(slots), list(starts), [list(t) for t in tokens], [list(w) for w in want]))
            return np.array([[100 * s + p] * 4 for s, w in enumerate(want) for p in w], np.float32).reshape(-1, 4)

        def close(self):
            pass

    monkeypatch.setattr(T, "load_model", lambda folder, dtype, n, batch: made.append((dtype, n, batch)) or Fake(batch))
    r = T.TraceRunner("x", "float32", 99)
    out = r.step([{"id": "a", "tokens": [1, 2, 3], "want": [2, 0]}], [])
    assert out[:, 0].tolist() == [2, 0] and calls[-1] == ([0], [0], [[1, 2, 3]], [[0, 2]])
    with pytest.raises(RuntimeError):
        r.step([{"id": "b", "tokens": [1], "want": []}], [])
    r.step([{"id": "a", "tokens": [4], "want": []}], ["a"])
    assert calls[-1][1] == [3]
    r.step([{"id": "b", "tokens": [1], "want": []}, {"id": "c", "tokens": [1, 2], "want": [1]}], ["b"])
    assert made == [("float32", 99, 1), ("float32", 99, 2)] and calls[-1][0] == [0, 1]
    r.step([{"id": "c", "tokens": [7], "want": [0]}], ["c"])
    assert calls[-1] == ([1], [2], [[7]], [[0]])


def test_trace_main(monkeypatch, tmp_path, capsys):
    import io

    import simplellminference_amd.trace as T

    class Fake:
        local_vocab = 2

        def feed(self, slots, starts, tokens, want):
            return np.array([[1.0, 2.0] for w in want for _ in w], np.float32).reshape(-1, 2)

    monkeypatch.setattr(T, "load_model", lambda *a: Fake())
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": [1, 2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [3], "want": [0]}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(x) for x in lines) + "\n"))
    assert T.main(["--model", "m", "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "8"]) == 0
    assert capsys.readouterr().out.split("\n")[:2] == ["done 0", "done 1"]
    assert not (tmp_path / "0.f32").exists()
    assert np.fromfile(tmp_path / "1.f32", "<f4").tolist() == [1.0, 2.0]


def test_command_line_arguments():
    from simplellminference_amd.__main__ import main
    with pytest.raises(SystemExit):
        main(["--model", "x"])
    with pytest.raises(SystemExit):
        main(["--model", "x", "--text", "words"])


# ---------------------------------------------------------------- the oracle on cases worked out by hand
def test_oracle_conv_and_norm():
    h = np.array([[1.0], [2.0], [4.0]])
    assert R.causal_conv(h, np.array([[0.5, 3.0]]))[:, 0].tolist() == [3.0, 6.5, 13.0]
    assert np.allclose(R.rms(np.array([3.0, 4.0]), 0.0), np.array([3.0, 4.0]) / np.sqrt(12.5))
    assert np.allclose(R.rms(np.zeros(4), 1e-6), 0.0)


def test_oracle_retention_is_a_decayed_sum():
    r = np.random.default_rng(0)
    q, k, v = r.standard_normal((3, 9, 2, 4))
    dec = np.array([0.5, 0.9])
    o = R.retention(q, k, v, dec)
    for t in range(9):
        for h in range(2):
            want = sum(dec[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert np.allclose(o[t, h], want)


def test_oracle_rotation_keeps_relative_positions():
    r = np.random.default_rng(1)
    a, b = r.standard_normal((2, 6))
    z = np.tile(np.stack([a, b])[None], (20, 1, 1))
    y = R.rotate(z, 4, 100.0)
    assert np.allclose(y[0], z[0]) and np.allclose(y[:, :, 4:], z[:, :, 4:])
    dots = [y[t, 0] @ y[t + 3, 1] for t in range(10)]
    assert np.allclose(dots, dots[0])


def test_oracle_attention_sink_and_bias():
    z = np.zeros((5, 3))
    p = R.attention_weights(z, z, 1.0, 0.0, 1.0, 0.0)  # the sink counts as one more key of score 0
    assert np.allclose(p[4], 1 / 6)
    p = R.attention_weights(z, z, 1.0, 1.0, 1.0, -1e9)  # weights 1 / (1 + distance)
    w = np.array([1 / 5, 1 / 4, 1 / 3, 1 / 2, 1.0])
    assert np.allclose(p[4], w / w.sum())


def test_oracle_feed_forward_clamps():
    one = np.ones((1, 1))
    y = R.feed_forward(np.array([[10.0]]), one, one, one, 2.0)[0, 0]
    assert np.isclose(y, 2.0 * R.sigmoid(3.404) * 3.0)
    y = R.feed_forward(np.array([[-10.0]]), one, one, one, 2.0)[0, 0]  # gate below is not clamped, up is
    assert np.isclose(y, -10.0 * R.sigmoid(-17.02) * -1.0)


# ---------------------------------------------------------------- a fault in any mechanism shows in the logits
def _cfg():
    a = dict(mixer="attention", heads=4, kv_heads=2, dim=16, vdim=12, scale=0.25, ff=20, ff_limit=1.0)
    r = dict(mixer="retention", heads=2, dim=16, vdim=10, rot_dims=8, rot_base=100.0, decay=(0.75, 0.97), ff=20, ff_limit=1.0)
    return dict(blocks=[r, a], vocab=41, width=32, taps=3, loop=(0, 1, 2), eps=1e-6, emb_scale=1.5, residual_mult=0.4)


FAULTS = {
    "sink": lambda mp, c, t: t.update({"l1.mix.sink": t["l1.mix.sink"] - 50.0}),
    "bias": lambda mp, c, t: t.update({"l1.mix.r1": 0 * t["l1.mix.r1"]}),
    "bias distance": lambda mp, c, t: mp.setattr(
        R, "attention_weights", lambda q, k, s, r1, r2, sk, f=R.attention_weights: f(q, k, s, r1, 5.0 * r2, sk)),
    "decay": lambda mp, c, t: c["blocks"][0].update(decay=(0.75, 0.93)),
    "rotation base": lambda mp, c, t: c["blocks"][0].update(rot_base=140.0),
    "rotation dims": lambda mp, c, t: c["blocks"][0].update(rot_dims=6),
    "key scale": lambda mp, c, t: mp.setattr(R, "rms", lambda x, e, f=R.rms: f(x, e) * (1.1 if x.shape[-1] == 10 else 1.0)),
    "gate": lambda mp, c, t: t.update({"l0.mix.g": -t["l0.mix.g"]}),
    "convolution shifted": lambda mp, c, t: mp.setattr(
        R, "causal_conv", lambda h, w, f=R.causal_conv: f(np.vstack([np.zeros_like(h[:1]), h[:-1]]), w)),
    "convolution of one sublayer": lambda mp, c, t: t.update({"l1.canon2": 0 * t["l1.canon2"]}),
    "clamp": lambda mp, c, t: c["blocks"][1].update(ff_limit=1.3),
    "head mapping": lambda mp, c, t: t.update({"l1.mix.k": np.roll(t["l1.mix.k"], 16, 0)}),
    "loop": lambda mp, c, t: c.update(loop=(0, 1, 1)),
    "residual": lambda mp, c, t: c.update(residual_mult=0.5),
    "embedding scale": lambda mp, c, t: c.update(emb_scale=3.0),
}


@pytest.mark.parametrize("fault", list(FAULTS))
def test_a_fault_would_show(monkeypatch, fault):
    """The random models of the GPU tests are sensitive to every mechanism: a fault planted in the oracle moves the logits
    by more than the 16-bit tolerance."""
    c = _cfg()
    t = R.random_tensors(c, 3)
    ids = np.random.default_rng(4).integers(0, 41, 40)
    good = R.forward(c, t, ids)[0]
    FAULTS[fault](monkeypatch, c, t)
    assert np.abs(R.forward(c, t, ids)[0] - good).max() > 0.03 * np.abs(good).max()
