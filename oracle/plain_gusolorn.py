"""Plain, slow restatement of the Gusolorn decoder (test infrastructure only; float64 on the CPU).

One function per mechanism, written from its equation, whole sequence at once, no cache:

    x        = E[t]
    x       <- x + ls1 * mixer(norm(x; 1 + w1));   x <- x + ls2 * ff(norm(x; 1 + w2))
    norm(z; w) = z / sqrt(mean z^2 + eps) * w
    logits   = head norm(x; 1 + w)

Mixers: a matrix memory with exponential gates (mlstm), and windowed attention over a low-rank latent, whose latent rows
another layer may lend.  Feed-forwards: dense with the erf gelu, or sigmoid-routed experts with clamped gates and a
gated shared expert.

A model is (cfg, tensors): cfg as in config.json, tensors name -> numpy array.
"""
import math

import numpy as np

_erf = np.vectorize(math.erf, otypes=[np.float64])


def rms_norm(x, eps, weight=None):
    y = x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)
    return y if weight is None else y * weight


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


# ------------------------------------------------------------------ matrix memory

def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def matrix_memory(q, k, v, log_i, log_f, state=None):
    """q, k [n, H, d], v [n, H, e], log gates [n, H] -> outputs [n, H, e] and the state (S, n, m) after the last token:

        m' = max(f + m, i);  S' = e^(f + m - m') S + e^(i - m') k v^T;  n' likewise with k
        o  = S'^T q / (max(|n' . q|, e^(-m')) + 1e-6)
    """
    n, H, d = q.shape
    S, N, m = (np.zeros((H, d, v.shape[2])), np.zeros((H, d)), np.zeros(H)) if state is None else state
    out = np.empty((n, H, v.shape[2]))
    for t in range(n):
        m_new = np.maximum(log_f[t] + m, log_i[t])
        keep, put = np.exp(log_f[t] + m - m_new), np.exp(log_i[t] - m_new)
        S = keep[:, None, None] * S + put[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        N = keep[:, None] * N + put[:, None] * k[t]
        m = m_new
        dot = np.abs(np.einsum("hd,hd->h", N, q[t]))
        out[t] = np.einsum("hde,hd->he", S, q[t]) / (np.maximum(dot, np.exp(-m)) + 1e-6)[:, None]
    return out, (S, N, m)


def mlstm(m, w, name, h, eps):
    n, H, d, e = len(h), m["heads"], m["dim"], m["vdim"]
    lin = lambda t: h @ w[name + "." + t].T
    q, k, v = (lin("q") * d ** -0.5).reshape(n, H, d), lin("k").reshape(n, H, d), lin("v").reshape(n, H, e)
    log_i = soft_cap(lin("i") + w[name + ".i.b"], m["gate_cap"])
    log_f = log_sigmoid(soft_cap(lin("f") + w[name + ".f.b"], m["gate_cap"]))
    o = rms_norm(matrix_memory(q, k, v, log_i, log_f)[0], eps).reshape(n, H * e)
    return (o * w[name + ".norm"] * sigmoid(lin("g"))) @ w[name + ".o"].T


# ------------------------------------------------------------------ latent attention

def rotate(x, base, positions=None):
    """Interleaved rotary positions over the last axis; x [n, ..., dims]: pair (2 i, 2 i + 1) turned by p base^(-2 i / dims)."""
    n, dims = x.shape[0], x.shape[-1]
    p = np.arange(n) if positions is None else np.asarray(positions)
    a = p[:, None] * base ** (-2.0 * np.arange(dims // 2) / dims)
    a = a.reshape((n,) + (1,) * (x.ndim - 2) + (dims // 2,))
    u, v = x[..., 0::2], x[..., 1::2]
    out = np.empty_like(x)
    out[..., 0::2] = u * np.cos(a) - v * np.sin(a)
    out[..., 1::2] = v * np.cos(a) + u * np.sin(a)
    return out


def window_mask(n, size):
    """[query, key] True where the key is seen: the query's own position and the size - 1 before it."""
    d = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (d >= 0) & (d < size)


def softmax_attention(q, k, v, scale, seen):
    """q, k [n, H, d], v [n, H, e], seen [n, n] -> [n, H, e]."""
    out = np.empty((q.shape[0], q.shape[1], v.shape[2]))
    for h in range(q.shape[1]):
        s = np.where(seen, scale * (q[:, h] @ k[:, h].T), -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, h]
    return out


def latent_rows(m, w, name, h, eps):
    """(latent [n, rank], rotated key part [n, rot_dim]) that a layer caches."""
    y = h @ w[name + ".dkv"].T
    r = m["kv_rank"]
    return rms_norm(y[:, :r], eps, w[name + ".dkv.norm"]), rotate(y[:, r:], m["rot"]["base"])


def latent_attention(m, w, name, h, rows):
    c, k_rot = rows
    n, H, d, r, e = len(h), m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = (h @ w[name + ".q"].T).reshape(n, H, d + r)
    q = np.concatenate([q[:, :, :d], rotate(q[:, :, d:], m["rot"]["base"])], axis=2)
    k = np.concatenate([(c @ w[name + ".uk"].T).reshape(n, H, d), np.repeat(k_rot[:, None], H, axis=1)], axis=2)
    v = (c @ w[name + ".uv"].T).reshape(n, H, e)
    seen = window_mask(n, m["mask"]["size"] if m.get("mask") else n)
    return softmax_attention(q, k, v, m["scale"], seen).reshape(n, H * e) @ w[name + ".o"].T


# ------------------------------------------------------------------ feed-forwards

def gelu_erf(z):
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def dense_ff(w, name, h):
    return gelu_erf(h @ w[name + ".up"].T) @ w[name + ".down"].T


def clamped_glu(g, u, limit):
    g, u = np.minimum(g, limit), np.clip(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def expert(w, name, h, limit):
    return clamped_glu(h @ w[name + ".gate"].T, h @ w[name + ".up"].T, limit) @ w[name + ".down"].T


def route(scores, top):
    """Indices [n, top] of the largest scores of every row (the lower index first among equals)."""
    return np.argsort(-scores, axis=1, kind="stable")[:, :top]


def experts_ff(mlp, w, name, h):
    scores = sigmoid(h @ w[name + ".router"].T)
    chosen = route(scores, mlp["router"]["top"])
    out = np.zeros_like(h)
    for t in range(len(h)):
        for j in chosen[t]:
            out[t] += expert(w, "%s.e%d" % (name, j), scores[t, j] * h[t], mlp["expert"]["limit"])
    if mlp.get("shared"):
        out += sigmoid(h @ w[name + ".shared.sg"].T) * expert(w, name + ".shared", h, mlp["shared"]["limit"])
    return out


# ------------------------------------------------------------------ model

def forward(cfg, tensors, tokens, want_layers=False):
    """Logits [n, vocab] of every position (and the residual stream after every layer)."""
    w = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    streams, lent = [], {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = "l%d" % i, layer["mixer"]
        h = rms_norm(x, eps, 1.0 + w[p + ".norm1"])
        if layer["type"] == "mlstm":
            y = mlstm(m, w, p + ".mix", h, eps)
        else:
            lent[i] = lent[m["kv_from"]] if m.get("kv_from") is not None else latent_rows(m, w, p + ".mix", h, eps)
            y = latent_attention(m, w, p + ".mix", h, lent[i])
        x = x + w[p + ".ls1"] * y
        mlp = layer.get("mlp")
        if mlp is not None:
            h = rms_norm(x, eps, 1.0 + w[p + ".norm2"])
            y = dense_ff(w, p + ".mlp", h) if mlp["kind"] == "dense" else experts_ff(mlp, w, p + ".mlp", h)
            x = x + w[p + ".ls2"] * y
        streams.append(x)
    logits = rms_norm(x, eps, 1.0 + w["final.norm"]) @ w["head"].T
    return (logits, np.stack(streams)) if want_layers else logits


def greedy(cfg, tensors, prompt, count):
    """count greedy tokens after the prompt, the whole sequence recomputed for every one."""
    seq = list(prompt)
    for _ in range(count):
        seq.append(int(np.argmax(forward(cfg, tensors, seq)[-1])))
    return seq[len(prompt):]
