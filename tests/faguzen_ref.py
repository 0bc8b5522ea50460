"""Plain, slow restatement of the Faguzen design (test infrastructure only).

One function per mechanism, float64 numpy, whole sequences at once (no cache, no state
object): recurrences are walked token by token from a zero state, attention rows see every
earlier position. Nothing here is shared with the product path; the tests compare the HIP
engine against these functions on small random models.

A model is (cfg, w): cfg the parsed config.json dict, w a dict name -> float64 array under
the checkpoint's tensor names.

The design in short. x = E[token]. Every layer is a parallel block with two norms of the same
stream, both results scaled by one number: x += m (mix(n1(x)) + ff(n2(x))) (the feed-forward may
be absent). The norm is tanh(alpha x) w + b: no statistics. A run of layers [start, stop) is
walked `times` times with the same weights, pass t first adding row t of loop.step to x. The
mixer is a pair on the same input, a left + c right: left, softmax attention (biased q / k / v / o,
grouped key/value heads, rotation of the first dims entries in half-split pairs with frequencies
rescaled by how often a pair turns within a given number of positions, scores capped by a tanh,
an elementwise sigmoid output gate); right, a matrix memory with exponential input gates and a
running maximum that keeps them in range, read through a normaliser. Feed-forward: routed
two-matrix experts with the exact gelu (softmax scores over experts and identity outputs, a
correction added for the choice only, weights renormalised over the choice; a chosen identity
output is the input itself) plus a shared expert. Logits: head n(x), capped by a tanh.
"""

from __future__ import annotations

import math

import numpy as np

F = np.float64
_erf = np.vectorize(math.erf, otypes=[F])


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def gelu_erf(z):
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def tanh_norm(x, w, name):
    """tanh(alpha x) w + b, elementwise."""
    return np.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def rms_unit(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


# ------------------------------------------------------------------ attention
def rotation_frequencies(dims, base, scaling):
    """Angle per position of every pair. With a rescaling: a pair that turns more than `high` times
    within `original` positions keeps its frequency, one that turns fewer than `low` times turns
    `factor` times slower, between the two the frequencies are mixed linearly in the turns."""
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)], F)
    if not scaling:
        return f
    out = f.copy()
    for i, fi in enumerate(f):
        turns = scaling["original"] * fi / (2.0 * math.pi)
        if turns > scaling["high"]:
            continue
        if turns < scaling["low"]:
            out[i] = fi / scaling["factor"]
            continue
        s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
        out[i] = (1.0 - s) * fi / scaling["factor"] + s * fi
    return out


def rotate_halves(x, freq):
    """x [T, heads, D]: entries (i, i + n) turned by position * freq[i], n = len(freq); the rest pass."""
    n = len(freq)
    a = np.arange(len(x))[:, None, None] * freq[None, None, :]
    u, v = x[..., :n], x[..., n:2 * n]
    out = x.copy()
    out[..., :n] = u * np.cos(a) - v * np.sin(a)
    out[..., n:2 * n] = v * np.cos(a) + u * np.sin(a)
    return out


def softmax(s):
    e = np.exp(s - np.max(s, axis=-1, keepdims=True))
    return e / np.sum(e, axis=-1, keepdims=True)


def mixer_attention(cfg, w, pre, h, m, weights_out=None):
    H, G, D, V = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    T = len(h)

    def proj(n, heads):
        return (h @ w[pre + n].T + w[pre + n + ".b"]).reshape(T, heads, -1)

    q, k, v = proj("q", H), proj("k", G), proj("v", G)
    rot = m.get("rot")
    if rot and rot["dims"]:
        f = rotation_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
        q, k = rotate_halves(q, f), rotate_halves(k, f)
    mask = np.tril(np.ones((T, T), bool))
    out = np.zeros((T, H, V), F)
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * m["scale"]
        if m.get("softcap"):
            s = soft_cap(s, m["softcap"])
        p = softmax(np.where(mask, s, -np.inf))
        if weights_out is not None:
            weights_out.append(p)
        out[:, hd] = p @ v[:, g]
    gated = out.reshape(T, H * V) * sigmoid(h @ w[pre + "g"].T)
    return gated @ w[pre + "o"].T + w[pre + "o.b"]


# ------------------------------------------------------------------ matrix memory
def memory_gates(h, w, pre, cap):
    """Log input and log forget gates [T, H]."""
    i = soft_cap(h @ w[pre + "i"].T + w[pre + "i.b"], cap)
    f = log_sigmoid(soft_cap(h @ w[pre + "f"].T + w[pre + "f.b"], cap))
    return i, f


def normaliser(nq, m):
    return max(abs(nq), np.exp(-m)) + 1e-6


def memory_scan(q, k, v, i, f):
    """q, k [T, H, D], v [T, H, V], i, f [T, H]: the read-outs [T, H, V]."""
    T, H, D = q.shape
    o = np.zeros((T, H, v.shape[2]), F)
    for h in range(H):
        S, n, m = np.zeros((D, v.shape[2]), F), np.zeros(D, F), 0.0
        for t in range(T):
            new = max(f[t, h] + m, i[t, h])
            keep, put = np.exp(f[t, h] + m - new), np.exp(i[t, h] - new)
            m = new
            S = keep * S + put * np.outer(k[t, h], v[t, h])
            n = keep * n + put * k[t, h]
            o[t, h] = S.T @ q[t, h] / normaliser(n @ q[t, h], m)
    return o


def mixer_memory(cfg, w, pre, h, m):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    T = len(h)
    q = (h @ w[pre + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ w[pre + "k"].T).reshape(T, H, D)
    v = (h @ w[pre + "v"].T).reshape(T, H, V)
    i, f = memory_gates(h, w, pre, m["gate_cap"])
    o = rms_unit(memory_scan(q, k, v, i, f), cfg["norm"]["eps"]).reshape(T, H * V)
    return (o * w[pre + "norm"] * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def mixer_pair(cfg, w, pre, h, m, weights_out=None):
    return (m["left_scale"] * mixer_attention(cfg, w, pre + "left.", h, m["left"], weights_out)
            + m["right_scale"] * mixer_memory(cfg, w, pre + "right.", h, m["right"]))


# ------------------------------------------------------------------ feed-forward
def expert(w, pre, h):
    return gelu_erf(h @ w[pre + "up"].T) @ w[pre + "down"].T


def route(z, correction, top):
    """Router logits z [E] -> (the `top` chosen outputs, their weights). Scores: softmax over all;
    the choice ranks score + correction (ties: the lower index); weights: the chosen scores over
    their sum."""
    s = softmax(z)
    idx = np.argsort(-(s + correction), kind="stable")[:top]
    return idx, s[idx] / (s[idx].sum() + 1e-20)


def feed_forward(w, pre, h, mlp, choice_out=None):
    r = mlp["router"]
    out = np.zeros_like(h)
    zs = h @ w[pre + "router"].T
    for t in range(len(h)):
        idx, wt = route(zs[t], w[pre + "correction"], r["top"])
        if choice_out is not None:
            choice_out.append((idx, wt))
        for e, a in zip(idx, wt):
            out[t] += a * (expert(w, f"{pre}e{e}.", h[t:t + 1])[0] if e < r["experts"] else h[t])
    if mlp.get("shared"):
        out = out + expert(w, pre + "shared.", h)
    return out


# ------------------------------------------------------------------ the model
def run_order(cfg):
    """[(layer, pass number at the first layer of a pass, else None)] in running order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def layer(cfg, w, i, x, weights_out=None, choice_out=None):
    e, p = cfg["layers"][i], f"l{i}."
    y = mixer_pair(cfg, w, p + "mix.", tanh_norm(x, w, p + "norm1"), e["mixer"], weights_out)
    if e.get("mlp"):
        y = y + feed_forward(w, p + "mlp.", tanh_norm(x, w, p + "norm2"), e["mlp"], choice_out)
    return x + cfg["residual_mult"] * y


def forward(cfg, w, tokens, layers_out=None, weights_out=None, choice_out=None):
    """Logits [T, vocab] of a whole sequence from position 0."""
    x = w["embed"][np.asarray(tokens)]
    for i, step in run_order(cfg):
        if step is not None:
            x = x + w["loop.step"][step]
        x = layer(cfg, w, i, x, weights_out, choice_out)
        if layers_out is not None:
            layers_out.append(x.copy())
    z = tanh_norm(x, w, "final.norm") @ w["head"].T
    return soft_cap(z, cfg["logit_softcap"]) if cfg.get("logit_softcap") else z
