"""Bokulix models without a GPU: config.json to a stack description, the oracle's own mechanisms on cases that can be worked
out by hand, and the random models' sensitivity to a fault in any of them."""
import copy
import json

import numpy as np
import pytest

from tests import bokulix_ref as R


def entry(heads=3, dim=10, vdim=6, kv_rank=14, size=9, scale=0.3, ff=20, experts=5, top=2, **kw):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}} if experts else None
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                                                  "mask": {"size": size}}, "mlp": mlp, **kw}


CFG = {"architecture": "Bokulix", "vocab": 31, "width": 24, "norm": {"eps": 1e-4}, "canon": {"taps": 2}, "max_positions": 60,
       "layers": [entry(), entry(weights_of=0), entry(heads=2, size=4, experts=0), entry(weights_of=2, experts=0),
                  entry(top=5)]}


def test_config_to_spec():
    from simplellminference_amd.stack import bokulix_spec
    s = bokulix_spec(CFG, 50)
    assert (s.vocab_size, s.width, s.taps, s.eps, s.positions, s.max_length) == (31, 24, 2, 1e-4, 60, 50)
    assert bokulix_spec(CFG, 500).max_length == 60  # no context past the learned positions
    assert s.arrangement == "sequential" and s.runs == (0, 0, 1, 1, 2) and s.order == [0, 0, 1, 1, 2]
    a, b, c = s.blocks
    assert (a.mixer, a.heads, a.dim, a.vdim, a.kv_rank, a.window, a.scale) == ("latent", 3, 10, 6, 14, 9, 0.3)
    assert (a.ff, a.experts, a.top) == (20, 5, 2) and (b.ff, b.experts, b.heads, b.window) == (0, 0, 2, 4) and c.top == 5
    # tensors are named by layer, the model's by block; a block without a feed-forward drops its second norm and gate
    assert s.layer_names == (0, 2, 4)
    names = ["embed", "l0.mix.q", "l2.norm1", "l2.norm2", "l2.rg2.b", "l4.mlp.e3.up"]
    assert s.tensor_names(names) == [("embed", "embed"), ("l0.mix.q", "l0.mix.q"), ("l2.norm1", "l1.norm1"),
                                     ("l4.mlp.e3.up", "l2.mlp.e3.up")]
    # a layer's name that is no block's must not land in another block
    assert s.tensor_names(["l1.mix.q"]) == [("l1.mix.q", "l3.mix.q")]


def test_weights_of_chains_and_errors():
    from simplellminference_amd.stack import bokulix_spec
    c = copy.deepcopy(CFG)
    c["layers"] = [entry(), entry(weights_of=0), entry(weights_of=1), entry(weights_of=4), entry(heads=2)]
    s = bokulix_spec(c, 50)
    assert s.runs == (0, 0, 0, 1, 1) and s.layer_names == (0, 4)
    for bad in ([entry(weights_of=0)], [entry(weights_of=1), entry(weights_of=0)], [entry(weights_of=7)]):
        with pytest.raises(ValueError):
            bokulix_spec({**CFG, "layers": bad}, 50)
    for key, value in (("type", "other"), ("mlp", {"kind": "other"})):
        c = json.loads(json.dumps(CFG))
        c["layers"][0][key] = value
        with pytest.raises(ValueError):
            bokulix_spec(c, 50)


def test_rugudra_tensor_names_stay():
    from simplellminference_amd.stack import BlockSpec, StackSpec
    s = StackSpec(8, 8, (BlockSpec("attention", 1, 4, 4, kv_heads=1), BlockSpec("attention", 1, 4, 4, kv_heads=1, ff=4)))
    names = ["embed", "l0.norm1", "l0.norm2", "l0.canon2", "l1.norm2", "l1.canon2"]
    assert [a for a, _ in s.tensor_names(names)] == ["embed", "l0.norm1", "l1.norm2", "l1.canon2"]
    assert all(a == b for a, b in s.tensor_names(names)) and s.order == [0, 1]


# ---------------------------------------------------------------- the oracle on cases worked out by hand
def test_oracle_window_and_softmax():
    z = np.zeros((6, 3))
    assert np.allclose(R.attention_weights(z, z, 1.0, 3)[5], [0, 0, 0, 1 / 3, 1 / 3, 1 / 3])
    assert np.allclose(R.attention_weights(z, z, 1.0, 1), np.eye(6))
    assert np.allclose(R.attention_weights(z, z, 1.0, 99)[2], [1 / 3, 1 / 3, 1 / 3, 0, 0, 0])
    q, k = np.array([[0.0], [2.0]]), np.array([[3.0], [1.0]])
    e = np.exp([2 * 3 * 0.5, 2 * 1 * 0.5])
    assert np.allclose(R.attention_weights(q, k, 0.5, 9)[1], e / e.sum())


def test_oracle_convolution_and_latent():
    h = np.array([[1.0], [2.0], [4.0]])
    assert R.convolved(h, np.array([[0.5, 3.0]]))[:, 0].tolist() == [1 + 3.0, 2 + 6.5, 4 + 13.0]
    assert np.allclose(R.convolved(h, np.array([[0.25]])), 1.25 * h)
    c = R.latent(np.array([[3.0, 4.0]]), np.eye(2), np.array([1.0, 2.0]), 0.0)
    assert np.allclose(c, np.array([[3.0, 8.0]]) / np.sqrt(12.5))


def test_oracle_mixture():
    idx, p = R.route(np.array([[1.0]]), np.array([[1.0], [5.0], [3.0], [5.0]]), np.array([0.0, 0.0, 3.0, 0.0]), 3)
    assert idx.tolist() == [[2, 1, 3]]
    e = np.exp([6.0, 5.0, 5.0])
    assert np.allclose(p[0], e / e.sum())
    one = np.ones((1, 1))
    assert np.isclose(R.expert(np.array([[2.0]]), one, 3 * one, one)[0, 0], 2 * R.sigmoid(2.0) * 6)


def test_oracle_gated_residual():
    x, y = np.array([[1.0, -1.0]]), np.array([[3.0, 4.0]])
    got = R.residual(x, y, np.zeros((2, 2)), np.array([0.0, 50.0]), np.array([1.0, 2.0]), 0.0)
    v = np.array([1.5, 4.0])
    assert np.allclose(got, x + v / np.sqrt((v * v).mean()) * [1, 2])


# ---------------------------------------------------------------- a fault in any mechanism shows in the logits
def model(**kw):
    b = dict(heads=4, dim=12, vdim=10, kv_rank=20, window=9, scale=0.5, experts=6, top=2, ff=20)
    return {**dict(vocab=41, width=32, taps=3, eps=1e-6, positions=64, blocks=[dict(b), {**b, "window": 5, "top": 3}],
                   order=[0, 1, 0]), **kw}


def swap(name, make):
    return lambda mp, c, t: mp.setattr(R, name, make(getattr(R, name)))


FAULTS = {
    "window one short": swap("visible", lambda f: lambda n, w: f(n, w - 1)),
    "window one long": swap("visible", lambda f: lambda n, w: f(n, w + 1)),
    "scale": lambda mp, c, t: [b.update(scale=0.6) for b in c["blocks"]],
    "latent norm": lambda mp, c, t: t.update({"l0.mix.dkv.norm": t["l0.mix.dkv.norm"] ** 0}),
    "key heads": lambda mp, c, t: t.update({"l0.mix.uk": np.roll(t["l0.mix.uk"], 12, 0)}),
    "value heads": lambda mp, c, t: t.update({"l1.mix.uv": np.roll(t["l1.mix.uv"], 10, 0)}),
    "output gate": lambda mp, c, t: t.update({"l0.mix.g": 0 * t["l0.mix.g"]}),
    "output gate's input": swap("latent_attention", lambda f: lambda h, w, b, e: f(h, {**w, "g": 0.7 * w["g"]}, b, e)),
    "convolution shifted": swap("convolved", lambda f: lambda h, w: h + f(np.vstack([0 * h[:1], h[:-1]]), w)),
    "convolution without its input": swap("convolved", lambda f: lambda h, w: f(h, w) - h),
    "residual gate": lambda mp, c, t: t.update({"l1.rg1": 0 * t["l1.rg1"]}),
    "residual gate bias": lambda mp, c, t: t.update({"l0.rg2.b": -t["l0.rg2.b"]}),
    "gates swapped": lambda mp, c, t: t.update({"l0.rg1": t["l0.rg2"], "l0.rg2": t["l0.rg1"]}),
    "norm gains": lambda mp, c, t: t.update({"l0.norm2": np.roll(t["l0.norm2"], 1)}),
    "gate after the norm": swap("residual", lambda f: lambda x, y, g, b, n, e: x + R.rms(y, e) * n * R.sigmoid(x @ g.T + b)),
    "fewer experts": lambda mp, c, t: c["blocks"][1].update(top=2),
    "equal expert weights": swap("route", lambda f: lambda h, w, b, k: (f(h, w, b, k)[0], np.full((len(h), k), 1 / k))),
    "router bias": lambda mp, c, t: t.update({"l0.mlp.router.b": 0 * t["l0.mlp.router.b"]}),
    "expert order": lambda mp, c, t: t.update({"l0.mlp.e0.up": t["l0.mlp.e1.up"], "l0.mlp.e1.up": t["l0.mlp.e0.up"]}),
    "positions": lambda mp, c, t: t.update({"pos": np.roll(t["pos"], 1, 0)}),
    "shared layer": lambda mp, c, t: c.update(order=[0, 1, 1]),
    "final norm": lambda mp, c, t: t.update({"final.norm": np.roll(t["final.norm"], 3)}),
}


@pytest.mark.parametrize("fault", list(FAULTS))
def test_a_fault_would_show(monkeypatch, fault):
    """The random models of the GPU tests are sensitive to every mechanism: a fault planted in the oracle moves the logits
    by more than the 16-bit tolerance."""
    c = model()
    t = R.random_tensors(c, 3)
    ids = np.random.default_rng(4).integers(0, 41, 40)
    good = R.forward(c, t, ids)[0]
    FAULTS[fault](monkeypatch, c, t)
    assert np.abs(R.forward(c, t, ids)[0] - good).max() > 0.03 * np.abs(good).max()
