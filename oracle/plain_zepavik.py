"""Plain, slow restatement of the Zepavik decoder (test infrastructure only; float64 on the CPU).

One function per mechanism, written from its equation, whole sequence at once, no cache:

    x_p      = E[t_p] + B[row(t_{p-1}, t_p)] + P[p]                       row of position 0: the table's last
    h        = norm(x; w, eps)                                            norm(z) = z / sqrt(mean z^2 + eps)
    x       <- x + mixer(h) + ff(h)                                       both sublayers read the same h
    s_hij    = c q_hi . k_gj - r1_h ln(1 + r2_h (i - j)),   0 <= i - j < window
    o_hi     = sigmoid(g_h . h_i) sum_j softmax_j(s_hij) v_gj             v_gj = norm(value of head g at j)
    ff(h)    = W_down relu(W_up h)^2
    logits   = a * head norm(x_L; w, eps)

A model is (cfg, tensors): cfg as in config.json, tensors name -> numpy array.
"""
import numpy as np


def rms_norm(x, eps, weight=None):
    y = x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)
    return y if weight is None else y * weight


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the bigram table for every token of a sequence that starts with tokens[0]."""
    rows = [buckets]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((int(prev) * mul_prev + int(cur) * mul_cur) % buckets)
    return np.array(rows, np.int64)


def embed(cfg, w, tokens):
    b = cfg["embedding"]["bigram"]
    rows = bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])
    return w["embed"][np.asarray(tokens)] + w["bigram"][rows] + w["pos"][np.arange(len(tokens))]


def log_distance_bias(r1, r2, distance):
    """[heads, ...] numbers taken off the scores at these distances."""
    shape = (-1,) + (1,) * np.ndim(distance)
    return r1.reshape(shape) * np.log(1.0 + r2.reshape(shape) * distance)


def window_mask(n, size):
    """[query, key] True where the key is seen: the query's own position and the size - 1 before it."""
    d = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (d >= 0) & (d < size)


def attention(q, k, v, scale, r1, r2, window):
    """q [n, H, d], k [n, G, d], v [n, G, e] -> [n, H, e]."""
    n, H, _ = q.shape
    per = H // k.shape[1]
    dist = np.arange(n)[:, None] - np.arange(n)[None, :]
    seen = window_mask(n, window)
    out = np.empty((n, H, v.shape[2]))
    for h in range(H):
        s = scale * (q[:, h] @ k[:, h // per].T)
        s = s - log_distance_bias(r1[h:h + 1], r2[h:h + 1], np.where(seen, dist, 0))[0]
        s = np.where(seen, s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, h // per]
    return out


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def mixer(m, w, name, h, eps):
    n, H, G, d, e = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    lin = lambda t: h @ w[name + "." + t].T + w[name + "." + t + ".b"]
    q, k = lin("q").reshape(n, H, d), lin("k").reshape(n, G, d)
    v = rms_norm(lin("v").reshape(n, G, e), eps)
    o = attention(q, k, v, m["scale"], w[name + ".r1"], w[name + ".r2"], m["mask"]["size"])
    o = o * sigmoid(h @ w[name + ".g"].T)[:, :, None]
    return o.reshape(n, H * e) @ w[name + ".o"].T


def feed_forward(w, name, h):
    return np.square(np.maximum(h @ w[name + ".up"].T, 0.0)) @ w[name + ".down"].T


def forward(cfg, tensors, tokens, want_layers=False):
    """Logits [n, vocab] of every position (and the residual stream after every layer)."""
    w = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = embed(cfg, w, tokens)
    streams = []
    for i, layer in enumerate(cfg["layers"]):
        h = rms_norm(x, eps, w["l%d.norm1" % i])
        y = mixer(layer["mixer"], w, "l%d.mix" % i, h, eps)
        if layer["mlp"] is not None:
            y = y + feed_forward(w, "l%d.mlp" % i, h)
        x = x + y
        streams.append(x)
    logits = cfg["logit_scale"] * (rms_norm(x, eps, w["final.norm"]) @ w["head"].T)
    return (logits, np.stack(streams)) if want_layers else logits


def greedy(cfg, tensors, prompt, count):
    """count greedy tokens after the prompt, the whole sequence recomputed for every one."""
    seq = list(prompt)
    for _ in range(count):
        seq.append(int(np.argmax(forward(cfg, tensors, seq)[-1])))
    return seq[len(prompt):]
