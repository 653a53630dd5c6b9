"""A plain, slow implementation of the Nidasun decoder.

Whole sequences, no cache, one function per mechanism, NumPy in float64 throughout.  It shares no
code with ``sonicboom_amd``: the configuration is the dict of config.json and the weights a dict of
arrays by the file's tensor names.

The design in this file's notation (positions t = 0 .. n-1, r(v) = v / sqrt(mean v^2 + eps)):

* S streams X_1 .. X_S [n, width], all the table's rows at the start.  A sublayer f with numbers a [S],
  b [S] and M [S, S] reads u = sum_s a_s X_s and leaves X_t <- sum_s M_st X_s + b_t f(r(u) w).  A layer is
  two of them, mixer and feed-forward; the model's end reads the sum of the streams.
* a run of layers (``loop``) is repeated with the same weights.
* mixer ``attention``: q, k, v with biases, rotate-half pairs of the first ``rot.dims`` numbers of a head turn by
  t base^(-2i/dims), scores scale * q.k over the earlier positions of t's own chunk of ``mask.size``, weights
  exp(s_j) / (exp(sink_a) + sum exp(s_j)), Wo with a bias.
* mixer ``lightning``: q, k, v = silu of their products, S_t = decay_a S_(t-1) + k_t v_t^T, o_t = S_t^T q_t a head;
  Wo (r(all heads side by side) w * sigmoid(Wg h)).
* mixer ``parallel``: left_scale left + right_scale right.  left: attention whose q and k are r(.) w over the whole
  projection before the heads turn (frequencies divided by ``rot.scaling.factor``), over the last ``mask.size``
  positions.  right: y = gelu(Wy h + b), u = conv(Wx h + b) + b' over time a channel, in equal blocks of channels
  rho = sigmoid(Ra u + ba), iota = sigmoid(Ri u + bi), log alpha = -8 rho softplus(lam),
  S_t = alpha S_(t-1) + sqrt(1 - alpha^2) iota u; Wo (S y).
* feed-forward ``dense``: Wdown max(Wup h, 0)^2; ``moe``: experts Wdown (silu(Wgate h) * Wup h), scores
  sigma = sigmoid(Wr h), chosen by sigma + correction within the groups whose two best choice scores have the
  largest sums, weights scale * sigma / (their sum + 1e-20).
"""
from __future__ import annotations

import numpy as np

F64 = np.float64


def f64(a):
    return np.asarray(a, dtype=F64)


def sigmoid(a):
    a = f64(a)
    e = np.exp(-np.abs(a))
    return np.where(a >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(a):
    return f64(a) * sigmoid(a)


def softplus(a):
    a = f64(a)
    return np.maximum(a, 0.0) + np.log1p(np.exp(-np.abs(a)))


def gelu_tanh(z):
    z = f64(z)
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def linear(x, weight, bias=None):
    y = f64(x) @ f64(weight).T
    return y if bias is None else y + f64(bias)


def rms_norm(v, weight, eps: float):
    v = f64(v)
    y = v / np.sqrt((v * v).mean(-1, keepdims=True) + eps)
    return y if weight is None else y * f64(weight)


def turn(v, positions, rot):
    """v [n, heads, m]: pairs (i, i + dims/2) of the first ``dims`` numbers turn, the rest pass."""
    v = np.array(v, dtype=F64)
    dims = int(rot["dims"])
    half = dims // 2
    if not half:
        return v
    f = float(rot["base"]) ** (-2.0 * np.arange(half, dtype=F64) / dims)
    if rot.get("scaling"):
        f = f / float(rot["scaling"]["factor"])
    ang = f64(positions)[:, None, None] * f
    c, s = np.cos(ang), np.sin(ang)
    a, b = v[..., :half].copy(), v[..., half:dims].copy()
    v[..., :half], v[..., half:dims] = a * c - b * s, b * c + a * s
    return v


# ---- attention ------------------------------------------------------------------------------------

def window_mask(n, size):
    """[n, n]: row i sees column j."""
    back = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (back >= 0) & (back < size)


def chunk_mask(n, size):
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & (i // size == j // size)


def attend(q, k, v, scale, mask, sink=None):
    """q [n, H, d], k [n, G, d], v [n, G, e] -> [n, H * e]; ``sink`` [H] or None."""
    n, H = q.shape[:2]
    out = np.empty((n, H, v.shape[2]), dtype=F64)
    for a in range(H):
        b = a // (H // k.shape[1])
        s = np.where(mask, (q[:, a] @ k[:, b].T) * F64(scale), -np.inf)
        top = s.max(-1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, F64(sink[a]))
        e = np.exp(s - top)
        den = e.sum(-1, keepdims=True)
        if sink is not None:
            den = den + np.exp(F64(sink[a]) - top)
        out[:, a] = (e / den) @ v[:, b]
    return out.reshape(n, -1)


def chunked_attention(mx, eps, w, p, h):
    n, pos = h.shape[0], np.arange(h.shape[0])
    H, G, d, e = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = turn(linear(h, w[p + "q"], w[p + "q.b"]).reshape(n, H, d), pos, mx["rot"])
    k = turn(linear(h, w[p + "k"], w[p + "k.b"]).reshape(n, G, d), pos, mx["rot"])
    v = linear(h, w[p + "v"], w[p + "v.b"]).reshape(n, G, e)
    o = attend(q, k, v, mx["scale"], chunk_mask(n, mx["mask"]["size"]), f64(w[p + "sink"]))
    return linear(o, w[p + "o"], w[p + "o.b"])


def windowed_attention(mx, eps, w, p, h):
    n, pos = h.shape[0], np.arange(h.shape[0])
    H, G, d, e = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = rms_norm(linear(h, w[p + "q"]), w[p + "q.norm"], eps).reshape(n, H, d)
    k = rms_norm(linear(h, w[p + "k"]), w[p + "k.norm"], eps).reshape(n, G, d)
    v = linear(h, w[p + "v"]).reshape(n, G, e)
    o = attend(turn(q, pos, mx["rot"]), turn(k, pos, mx["rot"]), v, mx["scale"], window_mask(n, mx["mask"]["size"]))
    return linear(o, w[p + "o"])


# ---- recurrences ----------------------------------------------------------------------------------

def lightning_reads(q, k, v, decay):
    """S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t for one head."""
    S = np.zeros((k.shape[1], v.shape[1]), dtype=F64)
    out = np.empty((k.shape[0], v.shape[1]), dtype=F64)
    for t in range(k.shape[0]):
        S = F64(decay) * S + np.outer(k[t], v[t])
        out[t] = q[t] @ S
    return out


def lightning(mx, eps, w, p, h):
    n, H, D, E = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q, k = silu(linear(h, w[p + "q"])).reshape(n, H, D), silu(linear(h, w[p + "k"])).reshape(n, H, D)
    v = silu(linear(h, w[p + "v"])).reshape(n, H, E)
    o = np.concatenate([lightning_reads(q[:, a], k[:, a], v[:, a], mx["decay"][a]) for a in range(H)], axis=1)
    return linear(rms_norm(o, w[p + "norm"], eps) * sigmoid(linear(h, w[p + "g"])), w[p + "o"])


def time_conv(x, taps, bias):
    """y[t, c] = sum_j taps[c, j] x[t - T + 1 + j, c] + bias[c], zeros before the start."""
    x, taps = f64(x), f64(taps)
    T = taps.shape[1]
    padded = np.concatenate([np.zeros((T - 1, x.shape[1])), x])
    y = np.zeros_like(x)
    for j in range(T):
        y += padded[j:j + x.shape[0]] * taps[:, j]
    return y + f64(bias)


def block_gates(u, mats, biases):
    """sigmoid of the blocks' products: u [n, width], mats [blocks, m, m], biases [blocks, m]."""
    n, (B, m, _) = u.shape[0], mats.shape
    parts = u.reshape(n, B, m)
    return np.concatenate([sigmoid(linear(parts[:, b], mats[b], biases[b])) for b in range(B)], axis=1)


def gated_recurrence(u, r, i, lam):
    log_a = -8.0 * r * softplus(lam)
    a, keep = np.exp(log_a), np.sqrt(-np.expm1(2.0 * log_a))
    S, out = np.zeros(u.shape[1], dtype=F64), np.empty_like(u)
    for t in range(u.shape[0]):
        S = a[t] * S + keep[t] * i[t] * u[t]
        out[t] = S
    return out


def recurrent_block(mx, w, p, h):
    y = gelu_tanh(linear(h, w[p + "y"], w[p + "y.b"]))
    u = time_conv(linear(h, w[p + "x"], w[p + "x.b"]), w[p + "conv"], w[p + "conv.b"])
    r, i = block_gates(u, f64(w[p + "ra"]), w[p + "ra.b"]), block_gates(u, f64(w[p + "ri"]), w[p + "ri.b"])
    return linear(gated_recurrence(u, r, i, w[p + "lam"]) * y, w[p + "o"])


def side_by_side(mx, eps, w, p, h):
    return F64(mx["left_scale"]) * windowed_attention(mx["left"], eps, w, p + "left.", h) \
        + F64(mx["right_scale"]) * recurrent_block(mx["right"], w, p + "right.", h)


MIXERS = {"attention": chunked_attention, "lightning": lightning, "parallel": side_by_side}


# ---- feed-forwards --------------------------------------------------------------------------------

def dense(w, p, h):
    return linear(np.maximum(linear(h, w[p + "up"]), 0.0) ** 2, w[p + "down"])


def choose(scores, correction, router):
    """(chosen experts, their weights) of one row."""
    E, top, groups = router["experts"], router["top"], router["groups"]
    choice = scores + f64(correction)
    m = E // groups["count"]
    sums = [np.sort(choice[g * m:(g + 1) * m])[::-1][:2].sum() for g in range(groups["count"])]
    kept = np.argsort(-np.array(sums), kind="stable")[:groups["keep"]]
    seen = np.where(np.isin(np.arange(E) // m, kept), choice, -np.inf)
    ids = np.argsort(-seen, kind="stable")[:top]
    return ids, scores[ids] / (scores[ids].sum() + 1e-20) * F64(router["scale"])


def routed(mlp, w, p, h):
    scores = sigmoid(linear(h, w[p + "router"]))
    out = np.zeros_like(f64(h))
    for t in range(h.shape[0]):
        for e, a in zip(*choose(scores[t], w[p + "correction"], mlp["router"])):
            q = f"{p}e{e}."
            out[t] += a * linear(silu(linear(h[t], w[q + "gate"])) * linear(h[t], w[q + "up"]), w[q + "down"])
    return out


def feed_forward(mlp, w, p, h):
    return routed(mlp, w, p, h) if mlp["kind"] == "moe" else dense(w, p, h)


# ---- streams, loop, model -------------------------------------------------------------------------

def sublayer(X, a, b, M, f):
    """X [S, n, width]."""
    y = f(np.tensordot(f64(a), X, axes=(0, 0)))
    return np.tensordot(f64(M).T, X, axes=(1, 0)) + f64(b)[:, None, None] * y


def layer(cfg, w, i, X):
    eps, lay, p = cfg["norm"]["eps"], cfg["layers"][i], f"l{i}."
    X = sublayer(X, w[p + "hc1.in"], w[p + "hc1.out"], w[p + "hc1.mix"],
                 lambda u: MIXERS[lay["type"]](lay["mixer"], eps, w, p + "mix.", rms_norm(u, w[p + "norm1"], eps)))
    if lay["mlp"] is not None:
        X = sublayer(X, w[p + "hc2.in"], w[p + "hc2.out"], w[p + "hc2.mix"],
                     lambda u: feed_forward(lay["mlp"], w, p + "mlp.", rms_norm(u, w[p + "norm2"], eps)))
    return X


def run_order(cfg):
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(cfg, w, tokens, layers_out=None):
    """Logits of every position [n, vocab]; ``layers_out``: a list that receives the streams [S, n, width] after
    every layer run."""
    x0 = f64(w["embed"])[np.asarray(tokens)]
    X = np.stack([x0] * cfg["streams"])
    for i in run_order(cfg):
        X = layer(cfg, w, i, X)
        if layers_out is not None:
            layers_out.append(X.copy())
    return linear(rms_norm(X.sum(0), w["final.norm"], cfg["norm"]["eps"]), w["head"])


def greedy(cfg, w, prompt, n: int):
    """``n`` tokens after ``prompt``, each the first largest logit of the whole sequence so far."""
    tokens, out = list(prompt), []
    for _ in range(n):
        t = int(np.argmax(forward(cfg, w, tokens)[-1]))
        out.append(t)
        tokens.append(t)
    return out
