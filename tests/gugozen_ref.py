"""Plain, slow restatement of the Gugozen design (test infrastructure only).

One function per mechanism, float64 numpy, whole sequences at once (no cache, no state
object): the recurrence is walked token by token from a zero state, attention rows see every
earlier position. Nothing here is shared with the product path; the tests compare the HIP
engine against these functions on small random models.

A model is (cfg, w): cfg the parsed config.json dict, w a dict name -> float64 array under
the checkpoint's tensor names.

The design in short. x = E[token] + B[row], row a hash of the previous and the current token (the
table's last row for a sequence's first token). Every layer normalises AFTER its sums: x <-
n1(a x + mix(x)), x <- n2(a x + ff(x)) (the feed-forward may be absent), n a layer norm with weight
and bias, a one number for the model. Three mixers: gated linear attention (a decay per head
and key channel from a low-rank projection, read-outs rms-normed per head and gated by a silu);
latent attention (rms-normed cached latents, one rotated key part shared by all heads, an
elementwise sigmoid output gate; a layer may read the latents and the rotated key part another
layer cached); softmax attention (queries and keys rms-normed over the whole projection, half-
split rotary pairs, a learned sink in the denominator). Feed-forward: routed clamped experts
whose weight, sigmoid(logit), multiplies the expert's INPUT, plus a shared expert. Logits: the
embedding table on the final norm.
"""

from __future__ import annotations

import numpy as np

F = np.float64


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def layer_norm(x, w, name, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w[name] + w[name + ".b"]


def rms_norm(x, weight, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * weight


# ------------------------------------------------------------------ embedding
def bigram_rows(tokens, spec):
    """The table row of every token of a sequence that starts here."""
    rows = [spec["buckets"]]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((int(prev) * int(spec["mul_prev"]) + int(cur) * int(spec["mul_cur"])) % int(spec["buckets"]))
    return rows


def embedding(cfg, w, tokens):
    x = w["embed"][np.asarray(tokens)]
    spec = (cfg.get("embedding") or {}).get("bigram")
    return x + w["bigram"][bigram_rows(tokens, spec)] if spec else x


# ------------------------------------------------------------------ attention
def rotate_halves(x, rot):
    """x [T, heads, D]: entries (i, i + n) of the first 2 n = rot.dims turned by position * base^(-i / n)."""
    n = rot["dims"] // 2
    if n == 0:
        return x
    f = np.array([float(rot["base"]) ** (-2.0 * i / rot["dims"]) for i in range(n)], F)
    a = np.arange(len(x))[:, None, None] * f[None, None, :]
    u, v = x[..., :n], x[..., n:2 * n]
    out = x.copy()
    out[..., :n] = u * np.cos(a) - v * np.sin(a)
    out[..., n:2 * n] = v * np.cos(a) + u * np.sin(a)
    return out


def causal_softmax(s, sink=None):
    """Rows of scores s [T, T] -> weights; sink: the score of one more key that has no value."""
    T = len(s)
    s = np.where(np.tril(np.ones((T, T), bool)), s, -np.inf)
    if sink is not None:
        s = np.concatenate([s, np.full((T, 1), float(sink))], axis=1)
    e = np.exp(s - s.max(axis=1, keepdims=True))
    return (e / e.sum(axis=1, keepdims=True))[:, :T]


def mixer_attention(cfg, w, pre, h, m, weights_out=None):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    T, eps = len(h), cfg["norm"]["eps"]
    q = rms_norm(h @ w[pre + "q"].T, w[pre + "q.norm"], eps).reshape(T, H, D)
    k = rms_norm(h @ w[pre + "k"].T, w[pre + "k.norm"], eps).reshape(T, G, D)
    v = (h @ w[pre + "v"].T).reshape(T, G, V)
    if m.get("rot"):
        q, k = rotate_halves(q, m["rot"]), rotate_halves(k, m["rot"])
    out = np.zeros((T, H, V), F)
    for hd in range(H):
        g = hd // (H // G)
        p = causal_softmax((q[:, hd] @ k[:, g].T) * m["scale"], w[pre + "sink"][hd])
        if weights_out is not None:
            weights_out.append(p)
        out[:, hd] = p @ v[:, g]
    return out.reshape(T, H * V) @ w[pre + "o"].T


def latent_rows(cfg, w, pre, h, m):
    """What a latent attention layer caches: the normed latents [T, kv_rank] and the rotated key
    part [T, rot_dim]."""
    z = h @ w[pre + "dkv"].T
    c = rms_norm(z[:, :m["kv_rank"]], w[pre + "dkv.norm"], cfg["norm"]["eps"])
    return c, rotate_halves(z[:, None, m["kv_rank"]:], m["rot"])[:, 0]


def mixer_latent(cfg, w, pre, h, m, rows, weights_out=None):
    """rows: the cached (latents, rotated key part) this layer reads, its own or another layer's."""
    H, D, R, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    T = len(h)
    c, kr = rows
    q = (h @ w[pre + "q"].T).reshape(T, H, D + R)
    qr = rotate_halves(q[..., D:], m["rot"])
    k = (c @ w[pre + "uk"].T).reshape(T, H, D)
    v = (c @ w[pre + "uv"].T).reshape(T, H, V)
    out = np.zeros((T, H, V), F)
    for hd in range(H):
        p = causal_softmax((q[:, hd, :D] @ k[:, hd].T + qr[:, hd] @ kr.T) * m["scale"])
        if weights_out is not None:
            weights_out.append(p)
        out[:, hd] = p @ v[:, hd]
    return (out.reshape(T, H * V) * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


# ------------------------------------------------------------------ gated linear attention
def gla_decays(w, pre, h, m):
    """Decay of every head's key channels, [T, heads, dim]."""
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "a2.b"]
    return (sigmoid(z) ** (1.0 / m["tau"])).reshape(len(h), m["heads"], m["dim"])


def gla_scan(q, k, v, a):
    """q, k, a [T, H, D], v [T, H, V]: the read-outs [T, H, V]."""
    T, H, D = q.shape
    o = np.zeros((T, H, v.shape[2]), F)
    for h in range(H):
        S = np.zeros((D, v.shape[2]), F)
        for t in range(T):
            S = a[t, h][:, None] * S + np.outer(k[t, h], v[t, h])
            o[t, h] = S.T @ q[t, h]
    return o


def mixer_gla(cfg, w, pre, h, m):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    T = len(h)
    q = (h @ w[pre + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ w[pre + "k"].T).reshape(T, H, D)
    v = (h @ w[pre + "v"].T).reshape(T, H, V)
    o = gla_scan(q, k, v, gla_decays(w, pre, h, m))
    o = rms_norm(o, w[pre + "norm"], cfg["norm"]["eps"]).reshape(T, H * V)
    return (o * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


# ------------------------------------------------------------------ feed-forward
def expert(w, pre, h, limit):
    g = np.minimum(h @ w[pre + "gate"].T, limit)
    u = np.clip(h @ w[pre + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


def route(z, top):
    """Router logits z [E] -> (the `top` chosen experts, their weights)."""
    idx = np.argsort(-z, kind="stable")[:top]
    return idx, sigmoid(z[idx])


def feed_forward(w, pre, h, mlp, choice_out=None):
    zs = h @ w[pre + "router"].T
    out = np.zeros_like(h)
    for t in range(len(h)):
        idx, wt = route(zs[t], mlp["router"]["top"])
        if choice_out is not None:
            choice_out.append((idx, wt))
        for e, a in zip(idx, wt):
            out[t] += expert(w, f"{pre}e{e}.", a * h[t:t + 1], mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        out = out + expert(w, pre + "shared.", h, mlp["shared"]["limit"])
    return out


# ------------------------------------------------------------------ the model
def layer(cfg, w, i, x, rows_of, weights_out=None, choice_out=None):
    """rows_of: layer -> what that latent attention layer has cached (filled as layers run)."""
    e, p = cfg["layers"][i], f"l{i}."
    m, eps, alpha = e["mixer"], cfg["norm"]["eps"], cfg["postln_alpha"]
    if e["type"] == "gla":
        y = mixer_gla(cfg, w, p + "mix.", x, m)
    elif e["type"] == "attention":
        y = mixer_attention(cfg, w, p + "mix.", x, m, weights_out)
    else:
        src = m.get("kv_from")
        if src is None:
            src = i
            rows_of[i] = latent_rows(cfg, w, p + "mix.", x, m)
        y = mixer_latent(cfg, w, p + "mix.", x, m, rows_of[src], weights_out)
    x = layer_norm(alpha * x + y, w, p + "norm1", eps)
    if e.get("mlp"):
        x = layer_norm(alpha * x + feed_forward(w, p + "mlp.", x, e["mlp"], choice_out), w, p + "norm2", eps)
    return x


def forward(cfg, w, tokens, layers_out=None, weights_out=None, choice_out=None):
    """Logits [T, vocab] of a whole sequence from position 0."""
    x = embedding(cfg, w, tokens)
    rows_of = {}
    for i in range(len(cfg["layers"])):
        x = layer(cfg, w, i, x, rows_of, weights_out, choice_out)
        if layers_out is not None:
            layers_out.append(x.copy())
    return layer_norm(x, w, "final.norm", cfg["norm"]["eps"]) @ w["embed"].T
