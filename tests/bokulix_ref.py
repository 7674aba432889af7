"""A plain, slow restatement of Bokulix models in float64 numpy, one function per mechanism: the oracle of
test_bokulix.py and test_gpu_bokulix.py. It shares no code with the package; a model is a dict of settings
(``vocab, width, taps, eps, positions``, ``blocks`` and ``order``, the block of every layer) and a dict of tensors."""
import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softmax(z):
    e = np.exp(z - z.max())
    return e / e.sum()


def embedding(t, ids):
    """token rows + the row of each position."""
    return t["embed"][np.asarray(ids)] + t["pos"][np.arange(len(ids))]


def convolved(h, w):
    """h [T, C], w [C, taps]: h[t] + sum_j w[:, j] h[t - taps + 1 + j], zeros before the start."""
    taps = w.shape[1]
    padded = np.vstack([np.zeros((taps - 1, h.shape[1])), h])
    return h + sum(w[:, j] * padded[j:j + len(h)] for j in range(taps))


def latent(h, w_down, w_norm, eps):
    """The cached row of every token: [T, kv_rank]."""
    return rms(h @ w_down.T, eps) * w_norm


def visible(n, window):
    """[query, key]: the query itself and the window - 1 tokens before it."""
    d = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (d >= 0) & (d < window)


def attention_weights(q, k, scale, window):
    """One head: q, k [T, dim] -> [T, T]."""
    s, see = (q @ k.T) * scale, visible(len(q), window)
    p = np.zeros_like(s)
    for i in range(len(q)):
        p[i, see[i]] = softmax(s[i, see[i]])
    return p


def latent_attention(h, w, b, eps):
    T, H = len(h), b["heads"]
    c = latent(h, w["dkv"], w["dkv.norm"], eps)
    q = (h @ w["q"].T).reshape(T, H, b["dim"])
    k = (c @ w["uk"].T).reshape(T, H, b["dim"])
    v = (c @ w["uv"].T).reshape(T, H, b["vdim"])
    o = np.stack([attention_weights(q[:, n], k[:, n], b["scale"], b["window"]) @ v[:, n] for n in range(H)], axis=1)
    return (o.reshape(T, -1) * sigmoid(h @ w["g"].T)) @ w["o"].T


def route(h, w_router, bias, top):
    """[T, top] experts in order of their logits, and their weights."""
    z = h @ w_router.T + bias
    idx = np.argsort(-z, axis=1, kind="stable")[:, :top]
    return idx, np.stack([softmax(z[i, idx[i]]) for i in range(len(z))])


def expert(h, gate, up, down):
    g = h @ gate.T
    return (g * sigmoid(g) * (h @ up.T)) @ down.T


def mixture(h, w, b):
    idx, p = route(h, w["router"], w["router.b"], b["top"])
    y = np.zeros_like(h)
    for i in range(len(h)):
        for e, a in zip(idx[i], p[i]):
            y[i] += a * expert(h[i], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
    return y


def residual(x, y, gate_w, gate_b, norm, eps):
    """x + the gated result of a sublayer that read x, normed."""
    return x + rms(y * sigmoid(x @ gate_w.T + gate_b), eps) * norm


def part(t, prefix):
    return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}


def layer(x, c, t, i):
    b, w, eps = c["blocks"][i], part(t, f"l{i}."), c["eps"]
    y = latent_attention(convolved(x, w["canon1"]), part(w, "mix."), b, eps)
    x = residual(x, y, w["rg1"], w["rg1.b"], w["norm1"], eps)
    if b["experts"]:
        x = residual(x, mixture(x, part(w, "mlp."), b), w["rg2"], w["rg2.b"], w["norm2"], eps)
    return x


def forward(c, t, ids):
    """logits [T, vocab], residual after every layer [layers, T, width]."""
    x = embedding(t, ids)
    hidden = []
    for i in c["order"]:
        x = layer(x, c, t, i)
        hidden.append(x)
    return (rms(x, c["eps"]) * t["final.norm"]) @ t["head"].T, np.array(hidden)


def greedy(c, t, prompt, length):
    ids = [int(i) for i in prompt]
    while len(ids) < length:
        ids.append(int(np.argmax(forward(c, t, ids)[0][-1])))
    return ids


def shapes(c):
    D = c["width"]
    out = {"embed": (c["vocab"], D), "pos": (c["positions"], D), "head": (c["vocab"], D), "final.norm": (D,)}
    for i, b in enumerate(c["blocks"]):
        p, q, v, R = f"l{i}.", b["heads"] * b["dim"], b["heads"] * b["vdim"], b["kv_rank"]
        out.update({p + "norm1": (D,), p + "canon1": (D, c["taps"]), p + "rg1": (D, D), p + "rg1.b": (D,),
                    p + "mix.q": (q, D), p + "mix.dkv": (R, D), p + "mix.dkv.norm": (R,), p + "mix.uk": (q, R),
                    p + "mix.uv": (v, R), p + "mix.g": (v, D), p + "mix.o": (D, v)})
        if b["experts"]:
            out.update({p + "norm2": (D,), p + "rg2": (D, D), p + "rg2.b": (D,), p + "mlp.router": (b["experts"], D),
                        p + "mlp.router.b": (b["experts"],)})
            for e in range(b["experts"]):
                out.update({p + f"mlp.e{e}.gate": (b["ff"], D), p + f"mlp.e{e}.up": (b["ff"], D),
                            p + f"mlp.e{e}.down": (D, b["ff"])})
    return out


def random_tensors(c, seed):
    """Random weights on which every mechanism shows: scores of a few units, gates on both sides of one half, norm gains
    away from 1. fp16-exact values, so both precisions hold the same model. The routers read the first quarter of the
    channels, which no sublayer adds to (norm gains 0, no position rows): the choice of experts follows from the token,
    and no rounding of the residual stream turns a close call into another expert."""
    r = np.random.default_rng(seed)
    t, own = {}, max(1, c["width"] // 4)
    for name, s in shapes(c).items():
        leaf = name.split(".")[-1]
        if "norm" in name:
            v = 0.6 + 0.8 * r.random(s)
            if leaf in ("norm1", "norm2"):
                v[:own] = 0.0
        elif leaf == "canon1":
            v = 0.35 * r.standard_normal(s)
        elif leaf in ("embed", "pos"):
            v = (1.0 if leaf == "embed" else 0.5) * r.standard_normal(s)
            if leaf == "pos":
                v[:, :own] = 0.0
        elif leaf == "router":
            v = np.zeros(s)
            v[:, :own] = 1.5 * r.standard_normal((s[0], own)) / np.sqrt(own)
        elif len(s) == 1:
            v = 0.7 * r.standard_normal(s)
        else:
            gain = {"q": 1.5, "uk": 1.5, "gate": 1.2, "up": 1.2, "head": 1.0}.get(leaf, 0.9)
            v = gain * r.standard_normal(s) / np.sqrt(s[-1])
        t[name] = np.asarray(v).astype(np.float16).astype(np.float64)
    return t
