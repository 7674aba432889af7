"""A plain, slow restatement of block-stack models in float64 numpy, one function per mechanism: the oracle of
test_gpu_stack.py. It shares no code with the package; a model is a dict of settings and a dict of tensors."""
import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def causal_conv(h, w):
    """h [T, C], w [C, taps]: y[t] = sum_j w[:, j] h[t - taps + 1 + j], zeros before the start."""
    T, taps = h.shape[0], w.shape[1]
    y = np.zeros_like(h)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * h[s]
    return y


def rotate(z, dims, base):
    """z [T, H, D]: pairs (i, i + dims / 2) of the first dims turned by position * base^(-2 i / dims)."""
    half = dims // 2
    out = z.copy()
    for i in range(half):
        ang = np.arange(z.shape[0]) * float(base) ** (-2.0 * i / dims)
        c, s = np.cos(ang)[:, None], np.sin(ang)[:, None]
        u, v = z[:, :, i], z[:, :, i + half]
        out[:, :, i], out[:, :, i + half] = u * c - v * s, v * c + u * s
    return out


def retention(q, k, v, decay):
    """q, k [T, H, D], v [T, H, E]; S <- decay S + k v^T, o = S^T q, token by token."""
    T, H, D = q.shape
    o = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        S = np.zeros((D, v.shape[2]))
        for t in range(T):
            S = decay[h] * S + np.outer(k[t, h], v[t, h])
            o[t, h] = S.T @ q[t, h]
    return o


def retention_mixer(h, w, b, eps):
    T, H = h.shape[0], b["heads"]
    q = (h @ w["q"].T).reshape(T, H, b["dim"])
    k = (h @ w["k"].T).reshape(T, H, b["dim"])
    v = (h @ w["v"].T).reshape(T, H, b["vdim"])
    if b["rot_dims"]:
        q, k = rotate(q, b["rot_dims"], b["rot_base"]), rotate(k, b["rot_dims"], b["rot_base"])
    o = rms(retention(q, k * b["dim"] ** -0.5, v, b["decay"]), eps).reshape(T, -1)
    g = h @ w["g"].T
    return (o * g * sigmoid(g)) @ w["o"].T


def attention_weights(q, k, scale, r1, r2, sink):
    """One head: q, k [T, D] -> weights [T, T] over the keys (they sum to less than 1: the sink takes the rest)."""
    T = q.shape[0]
    p = np.zeros((T, T))
    for i in range(T):
        s = np.array([scale * (q[i] @ k[j]) - r1 * np.log(1.0 + r2 * (i - j)) for j in range(i + 1)])
        m = max(s.max(), sink)
        e = np.exp(s - m)
        p[i, :i + 1] = e / (e.sum() + np.exp(sink - m))
    return p


def attention_mixer(h, w, b, eps):
    T, H, G = h.shape[0], b["heads"], b["kv_heads"]
    q = (h @ w["q"].T).reshape(T, H, b["dim"])
    k = (h @ w["k"].T).reshape(T, G, b["dim"])
    v = (h @ w["v"].T).reshape(T, G, b["vdim"])
    o = np.zeros((T, H, b["vdim"]))
    for n in range(H):
        kv = n // (H // G)
        o[:, n] = attention_weights(q[:, n], k[:, kv], b["scale"], w["r1"][n], w["r2"][n], w["sink"][n]) @ v[:, kv]
    return o.reshape(T, -1) @ w["o"].T


def feed_forward(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def block(x, c, t, i):
    b, p = c["blocks"][i], f"l{i}."
    w = {k[len(p) + 4:]: v for k, v in t.items() if k.startswith(p + "mix.")}
    h1 = rms(x, c["eps"]) * t[p + "norm1"]
    h1 = h1 + causal_conv(h1, t[p + "canon1"])
    y = (attention_mixer if b["mixer"] == "attention" else retention_mixer)(h1, w, b, c["eps"])
    if b["ff"]:
        h2 = rms(x, c["eps"]) * t[p + "norm2"]
        h2 = h2 + causal_conv(h2, t[p + "canon2"])
        y = y + feed_forward(h2, t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"], b["ff_limit"])
    return x + c["residual_mult"] * y


def order(c):
    a, b, n = c["loop"]
    return list(range(a)) + list(range(a, b)) * n + list(range(b, len(c["blocks"])))


def forward(c, t, tokens):
    """logits [T, vocab], residual after every block run [runs, T, width]."""
    x = t["embed"][np.asarray(tokens)] * c["emb_scale"]
    hidden = []
    for i in order(c):
        x = block(x, c, t, i)
        hidden.append(x)
    return (rms(x, c["eps"]) * t["final.norm"]) @ t["head"].T, np.array(hidden)


def greedy(c, t, prompt, length):
    ids = [int(i) for i in prompt]
    while len(ids) < length:
        ids.append(int(np.argmax(forward(c, t, ids)[0][-1])))
    return ids


def shapes(c):
    D = c["width"]
    out = {"embed": (c["vocab"], D), "head": (c["vocab"], D), "final.norm": ()}
    for i, b in enumerate(c["blocks"]):
        p, att = f"l{i}.", b["mixer"] == "attention"
        kv = b["kv_heads"] if att else b["heads"]
        out.update({p + "norm1": (), p + "canon1": (D, c["taps"]), p + "mix.q": (b["heads"] * b["dim"], D),
                    p + "mix.k": (kv * b["dim"], D), p + "mix.v": (kv * b["vdim"], D),
                    p + "mix.o": (D, b["heads"] * b["vdim"])})
        if att:
            out.update({p + "mix." + n: (b["heads"],) for n in ("r1", "r2", "sink")})
        else:
            out[p + "mix.g"] = (b["heads"] * b["vdim"], D)
        if b["ff"]:
            out.update({p + "norm2": (), p + "canon2": (D, c["taps"]), p + "mlp.gate": (b["ff"], D),
                        p + "mlp.up": (b["ff"], D), p + "mlp.down": (D, b["ff"])})
    return out


def random_tensors(c, seed):
    """Random weights on which every mechanism shows: scores of a few units, biases and sinks that matter, gains away
    from 1, feed-forward inputs on both sides of the clamp. fp16-exact values, so both precisions hold the same model."""
    r = np.random.default_rng(seed)
    t = {}
    for name, s in shapes(c).items():
        leaf = name.split(".")[-1]
        if "norm" in name:
            v = 0.8 + 0.5 * r.random()
        elif leaf in ("canon1", "canon2"):
            v = 0.35 * r.standard_normal(s)
        elif leaf == "r1":
            v = 0.3 + 1.5 * r.random(s)
        elif leaf == "r2":
            v = 0.05 + 0.5 * r.random(s)
        elif leaf == "sink":
            v = 2.0 * r.standard_normal(s)
        elif leaf == "embed":
            v = r.standard_normal(s)
        else:
            gain = {"q": 1.4, "k": 1.4, "gate": 1.2, "up": 1.2}.get(leaf, 0.8)
            v = gain * r.standard_normal(s) / np.sqrt(s[-1])
        t[name] = np.asarray(v).astype(np.float16).astype(np.float64)
    return t
