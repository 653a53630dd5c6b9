"""A plain, slow implementation of the Dudatar decoder.

Whole sequences, no cache, one function per mechanism, NumPy in float64 throughout.  It shares no
code with ``sonicboom_amd``: the configuration is the dict of config.json and the weights a dict of
arrays by the file's tensor names.

The design in this file's notation (positions t = 0 .. n-1, stream x [n, width], x0 the table's rows,
c(v, w) = (v - mean v) / sqrt(mean (v - mean v)^2 + eps) * w, r(v) = v / sqrt(mean v^2 + eps)):

* a layer has one norm whose result h = c(x, norm1) both branches read: x <- x + (mixer(h) + ff(h)).
* a run of layers (``loop``) is repeated with the same weights; pass number s begins with
  x <- W [x; x0] + step[s].
* mixer ``parallel``: two mixers read the same h and meet as (r(left) w_l + r(right) w_r) / 2.
  left: grouped-query attention; pairs (i, i + dims/2) of a head's first ``rot.dims`` numbers turn by
  t base^(-2i/dims); every head of q and of k then becomes r(.); scores scale * q.k over j <= t, softmax;
  head a's result times sigmoid((Wg h)_a); Wo.
  right: S_t = decay_a S_(t-1) + k_t v_t^T, o_t = S_t^T q_t a head, q and k turned, k times dim^(-1/2);
  every head becomes r(o), all heads times silu(Wg h); Wo.
* mixer ``gla``: S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t a head, q times dim^(-1/2),
  alpha = sigmoid(Wa2 (Wa1 h) + b)^(1/tau) a number per head and key channel; r(o) times a weight that the
  heads share, times silu(Wg h); Wo.
* feed-forward: Wdown (gelu(Wgate h) * (Wup h)), gelu by the hyperbolic tangent.
* logits: cap * tanh((head c(x, final.norm)) / cap).
"""
from __future__ import annotations

import numpy as np

F64 = np.float64


def sigmoid(a):
    a = np.asarray(a, dtype=F64)
    e = np.exp(-np.abs(a))
    return np.where(a >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(a):
    return np.asarray(a, dtype=F64) * sigmoid(a)


def linear(x, weight):
    return np.asarray(x, dtype=F64) @ np.asarray(weight, dtype=F64).T


def unit_rms(v, eps: float):
    v = np.asarray(v, dtype=F64)
    return v / np.sqrt((v * v).mean(-1, keepdims=True) + eps)


def layer_norm(v, weight, eps: float):
    v = np.asarray(v, dtype=F64)
    d = v - v.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * np.asarray(weight, dtype=F64)


def gelu_tanh(z):
    z = np.asarray(z, dtype=F64)
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def turn(v, positions, rot):
    """v [n, heads, m]: pairs (i, i + dims/2) of the first ``dims`` numbers turn, the rest pass."""
    v = np.array(v, dtype=F64)
    dims, base = int(rot["dims"]), float(rot["base"])
    half = dims // 2
    if not half:
        return v
    f = base ** (-2.0 * np.arange(half, dtype=F64) / dims)
    ang = np.asarray(positions, dtype=F64)[:, None, None] * f
    c, s = np.cos(ang), np.sin(ang)
    a, b = v[..., :half].copy(), v[..., half:dims].copy()
    v[..., :half], v[..., half:dims] = a * c - b * s, b * c + a * s
    return v


def softmax(s):
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


# ---- mixers ---------------------------------------------------------------------------------------

def attention_keys(mx, eps, w, p, h, positions):
    """(keys as they are scored [n, kv_heads, dim], values [n, kv_heads, vdim])."""
    n, G = h.shape[0], mx["kv_heads"]
    k = linear(h, w[p + "k"]).reshape(n, G, mx["dim"])
    return unit_rms(turn(k, positions, mx["rot"]), eps), linear(h, w[p + "v"]).reshape(n, G, mx["vdim"])


def gated_attention(mx, eps, w, p, h):
    n = h.shape[0]
    H, G = mx["heads"], mx["kv_heads"]
    pos = np.arange(n)
    q = unit_rms(turn(linear(h, w[p + "q"]).reshape(n, H, mx["dim"]), pos, mx["rot"]), eps)
    k, v = attention_keys(mx, eps, w, p, h, pos)
    gate = sigmoid(linear(h, w[p + "g"]))
    hidden = pos[None, :] > pos[:, None]
    out = np.empty((n, H, mx["vdim"]), dtype=F64)
    for a in range(H):
        b = a // (H // G)
        s = np.where(hidden, -np.inf, (q[:, a] @ k[:, b].T) * F64(mx["scale"]))
        out[:, a] = (softmax(s) @ v[:, b]) * gate[:, a:a + 1]
    return linear(out.reshape(n, -1), w[p + "o"])


def decayed_reads(q, k, v, decay):
    """S_t = decay_t S_(t-1) + k_t v_t^T (the decay acts on S's rows), o_t = S_t^T q_t; q, k, decay [n, D], v [n, E]."""
    S = np.zeros((k.shape[1], v.shape[1]), dtype=F64)
    out = np.empty((k.shape[0], v.shape[1]), dtype=F64)
    for t in range(k.shape[0]):
        S = decay[t][:, None] * S + np.outer(k[t], v[t])
        out[t] = q[t] @ S
    return out


def retention(mx, eps, w, p, h):
    n = h.shape[0]
    H, D, E = mx["heads"], mx["dim"], mx["vdim"]
    pos = np.arange(n)
    q = turn(linear(h, w[p + "q"]).reshape(n, H, D), pos, mx["rot"])
    k = turn(linear(h, w[p + "k"]).reshape(n, H, D), pos, mx["rot"]) * D ** -0.5
    v = linear(h, w[p + "v"]).reshape(n, H, E)
    out = np.empty((n, H, E), dtype=F64)
    for a in range(H):
        out[:, a] = decayed_reads(q[:, a], k[:, a], v[:, a], np.full((n, D), mx["decay"][a], dtype=F64))
    return linear(unit_rms(out, eps).reshape(n, H * E) * silu(linear(h, w[p + "g"])), w[p + "o"])


def side_by_side(mx, eps, w, p, h):
    left = gated_attention(mx["left"], eps, w, p + "left.", h)
    right = retention(mx["right"], eps, w, p + "right.", h)
    return 0.5 * (unit_rms(left, eps) * np.asarray(w[p + "left.out"], dtype=F64)
                  + unit_rms(right, eps) * np.asarray(w[p + "right.out"], dtype=F64))


def channel_decays(mx, w, p, h):
    z = linear(linear(h, w[p + "a1"]), w[p + "a2"]) + np.asarray(w[p + "a2.b"], dtype=F64)
    return sigmoid(z) ** (1.0 / F64(mx["tau"]))


def gated_linear_attention(mx, eps, w, p, h):
    n = h.shape[0]
    H, D, E = mx["heads"], mx["dim"], mx["vdim"]
    q = linear(h, w[p + "q"]).reshape(n, H, D) * D ** -0.5
    k, v = linear(h, w[p + "k"]).reshape(n, H, D), linear(h, w[p + "v"]).reshape(n, H, E)
    alpha = channel_decays(mx, w, p, h).reshape(n, H, D)
    out = np.empty((n, H, E), dtype=F64)
    for a in range(H):
        out[:, a] = decayed_reads(q[:, a], k[:, a], v[:, a], alpha[:, a])
    out = unit_rms(out, eps) * np.asarray(w[p + "norm"], dtype=F64)
    return linear(out.reshape(n, H * E) * silu(linear(h, w[p + "g"])), w[p + "o"])


# ---- feed-forward, loop, model ------------------------------------------------------------------------

def feed_forward(w, p, h):
    return linear(gelu_tanh(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


def layer(cfg, w, i, x):
    eps, lay, p = cfg["norm"]["eps"], cfg["layers"][i], f"l{i}."
    h = layer_norm(x, w[p + "norm1"], eps)
    mix = side_by_side if lay["type"] == "parallel" else gated_linear_attention
    y = mix(lay["mixer"], eps, w, p + "mix.", h)
    if lay["mlp"] is not None:
        y = y + feed_forward(w, p + "mlp.", h)
    return x + y


def begin_pass(w, x, x0, s):
    return linear(np.concatenate([x, x0], axis=1), w["loop.in"]) + np.asarray(w["loop.step"], dtype=F64)[s]


def run_order(cfg):
    """[(layer, the number of the pass that begins with it or None)] in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    order = [(i, None) for i in range(a)]
    for s in range(loop["times"]):
        order += [(i, s if i == a else None) for i in range(a, b)]
    return order + [(i, None) for i in range(b, n)]


def forward(cfg, w, tokens, layers_out=None):
    """Logits of every position [n, vocab]; ``layers_out``: a list that receives the stream after every layer run."""
    x0 = np.asarray(w["embed"], dtype=F64)[np.asarray(tokens)]
    x = x0.copy()
    for i, s in run_order(cfg):
        if s is not None:
            x = begin_pass(w, x, x0, s)
        x = layer(cfg, w, i, x)
        if layers_out is not None:
            layers_out.append(x.copy())
    z = linear(layer_norm(x, w["final.norm"], cfg["norm"]["eps"]), w["head"])
    cap = float(cfg.get("logit_softcap") or 0.0)
    return cap * np.tanh(z / cap) if cap else z


def greedy(cfg, w, prompt, n: int):
    """``n`` tokens after ``prompt``, each the first largest logit of the whole sequence so far."""
    tokens, out = list(prompt), []
    for _ in range(n):
        t = int(np.argmax(forward(cfg, w, tokens)[-1]))
        out.append(t)
        tokens.append(t)
    return out
