"""A plain, slow implementation of the Lapunex decoder: float64, numpy, whole sequences, no cache, one function per
mechanism.  It imports nothing from the package; the tests compare the engine with it.

A model is ``(cfg, W)``: ``cfg`` the dictionary of config.json, ``W`` a dictionary from tensor names to arrays.

The design in this file's notation.  ``X`` is the residual of one sequence, ``[T, streams, width]``, positions ``0 .. T-1``.

  start:     every stream is scale * embed[token];  end: x = sum of the streams, logits = head N_final(x)
  sublayer:  u = sum_s in[s] X_s,  y = f(N(u)),  X_t <- sum_s mix[s, t] X_s + out[t] y   (f the mixer, then the feed-forward;
             each with vectors and a matrix of its own;  N(u) = u / rms(u) (1 + w))
  loop:      the layers start .. stop - 1 run ``times`` times with the same weights
  lightning: q, k, v = silu(W h) per head;  S <- decay S + k v^T,  o = S^T q;
             out = W_o (N(all heads' o) * sigmoid(W_g h)),  a plain weight in N
  parallel:  left_scale left(h) + right_scale right(h)
  left:      q and k divided by their rms over all heads, times a weight; the first ``rot.dims`` dims turned (half-split pairs,
             frequencies blended between f and f / factor, cos and sin times 0.1 ln(factor) + 1); causal softmax of scale q . k with
             exp(sink) more in every denominator; each head times sigmoid of a number of its own; W_o
  right:     i = cap tanh(z_i / cap), f = log sigmoid(cap tanh(z_f / cap)) per head, m <- max(f + m, i) from m = 0,
             S <- exp(f + m' - m) S + exp(i - m) k v^T, n likewise with k alone (m' the m before),
             o = S^T q / (max(|n . q|, exp(-m)) + 1e-6), q = dim^(-1/2) W_q h;  o / rms(o) per head, * norm * sigmoid(W_g h); W_o
  dense:     W_down (silu(W_gate h) * W_up h)
  experts:   s = softmax(W_router h); of the ``groups.keep`` groups with the largest best score the ``top`` experts with the largest s;
             sum of scale s_e expert_e(h);  expert: g = min(W_gate h, limit), u = W_up h held within +-limit,
             W_down (g sigmoid(1.702 g) (u + 1))
"""
import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def rms_div(x, eps):
    return x / np.sqrt((x ** 2).mean(-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms_div(x, eps) * w


# ---------------------------------------------------------------- streams


def read_streams(X, inn):
    """X [T, streams, width] -> what a sublayer reads, before its norm."""
    return np.einsum("tsd,s->td", X, inn)


def update_streams(X, mix, out, y):
    """``mix``'s first index is the stream that is read, its second the one that is written."""
    return np.einsum("tsd,su->tud", X, mix) + out[None, :, None] * y[:, None, :]


# ---------------------------------------------------------------- rotation


def yarn(dims, base, scaling):
    """(frequencies [dims / 2], factor on cos and sin)"""
    i = np.arange(dims // 2)
    f = base ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0

    def dim_of(turns):
        return dims * np.log(scaling["original"] / (2 * np.pi * turns)) / (2 * np.log(base))

    lo = max(np.floor(dim_of(scaling["fast"])), 0)
    hi = min(np.ceil(dim_of(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(scaling["factor"]) + 1.0


def rotate_half_split(x, positions, freq, factor=1.0):
    """x [T, heads, dim]: dim i is paired with dim i + len(freq)."""
    half = len(freq)
    ang = positions[:, None] * freq[None, :]
    c, s = factor * np.cos(ang)[:, None, :], factor * np.sin(ang)[:, None, :]
    out = x.copy()
    u, v = x[..., :half], x[..., half:2 * half]
    out[..., :half] = u * c - v * s
    out[..., half:2 * half] = v * c + u * s
    return out


# ---------------------------------------------------------------- mixers


def attend(q, k, v, scale, sink=None):
    """One head, causal: q, k [T, dim], v [T, vdim].  ``sink``: one more term exp(sink) in every denominator."""
    T = q.shape[0]
    s = np.where(np.arange(T)[None, :] <= np.arange(T)[:, None], (q @ k.T) * scale, -np.inf)
    top = s.max(-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink)
    p = np.exp(s - top)
    total = p.sum(-1, keepdims=True)
    if sink is not None:
        total = total + np.exp(sink - top)
    return (p / total) @ v


def attention(h, W, pre, m, eps):
    T = h.shape[0]
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ W[pre + "q"].T, W[pre + "q.norm"], eps).reshape(T, H, dim)
    k = rms_norm(h @ W[pre + "k"].T, W[pre + "k.norm"], eps).reshape(T, G, dim)
    v = (h @ W[pre + "v"].T).reshape(T, G, vdim)
    if m.get("rot"):
        freq, factor = yarn(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
        pos = np.arange(T, dtype=np.float64)
        q, k = rotate_half_split(q, pos, freq, factor), rotate_half_split(k, pos, freq, factor)
    o = np.stack([attend(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], W[pre + "sink"][i]) for i in range(H)], 1)
    o = o * sigmoid(h @ W[pre + "g"].T)[:, :, None]
    return o.reshape(T, H * vdim) @ W[pre + "o"].T


def mlstm_gates(zi, zf, cap):
    """Logarithms of the input and the forget gate from their projections (bias included)."""
    return cap * np.tanh(zi / cap), log_sigmoid(cap * np.tanh(zf / cap))


def mlstm_scan(q, k, v, i, f):
    """One head: q, k [T, dim], v [T, vdim], i, f [T] -> o [T, vdim]."""
    S, n, m = np.zeros((q.shape[1], v.shape[1])), np.zeros(q.shape[1]), 0.0
    o = np.zeros_like(v)
    for t in range(q.shape[0]):
        before, m = m, max(f[t] + m, i[t])
        keep, take = np.exp(f[t] + before - m), np.exp(i[t] - m)
        S = keep * S + take * np.outer(k[t], v[t])
        n = keep * n + take * k[t]
        o[t] = (q[t] @ S) / (max(abs(n @ q[t]), np.exp(-m)) + 1e-6)
    return o


def mlstm(h, W, pre, m, eps):
    T = h.shape[0]
    H, dim, vdim = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[pre + "q"].T).reshape(T, H, dim) * dim ** -0.5
    k = (h @ W[pre + "k"].T).reshape(T, H, dim)
    v = (h @ W[pre + "v"].T).reshape(T, H, vdim)
    i, f = mlstm_gates(h @ W[pre + "i"].T + W[pre + "i.b"], h @ W[pre + "f"].T + W[pre + "f.b"], m["gate_cap"])
    o = np.stack([mlstm_scan(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(H)], 1)
    o = rms_div(o, eps).reshape(T, H * vdim) * W[pre + "norm"] * sigmoid(h @ W[pre + "g"].T)
    return o @ W[pre + "o"].T


def parallel(h, W, pre, m, eps):
    return m["left_scale"] * attention(h, W, pre + "left.", m["left"], eps) + m["right_scale"] * mlstm(h, W, pre + "right.", m["right"], eps)


def decay_scan(q, k, v, decay):
    """One head: S <- decay S + k v^T, o = S^T q."""
    S, o = np.zeros((q.shape[1], v.shape[1])), np.zeros_like(v)
    for t in range(q.shape[0]):
        S = decay * S + np.outer(k[t], v[t])
        o[t] = q[t] @ S
    return o


def lightning(h, W, pre, m, eps):
    T = h.shape[0]
    H, dim, vdim = m["heads"], m["dim"], m["vdim"]
    q, k = (silu(h @ W[pre + x].T).reshape(T, H, dim) for x in "qk")
    v = silu(h @ W[pre + "v"].T).reshape(T, H, vdim)
    o = np.stack([decay_scan(q[:, a], k[:, a], v[:, a], m["decay"][a]) for a in range(H)], 1).reshape(T, H * vdim)
    return (rms_norm(o, W[pre + "norm"], eps) * sigmoid(h @ W[pre + "g"].T)) @ W[pre + "o"].T


# ---------------------------------------------------------------- feed-forwards


def dense(h, W, pre):
    return (silu(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) @ W[pre + "down"].T


def limited_expert(h, W, pre, limit):
    g = np.minimum(h @ W[pre + "gate"].T, limit)
    u = np.clip(h @ W[pre + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1)) @ W[pre + "down"].T


def route(z, top, groups=None):
    """One token: (chosen experts, their scores).  Ties go to the lower index."""
    s = np.exp(z - z.max())
    s = s / s.sum()
    may = np.ones(len(s), bool)
    if groups:
        each = s.reshape(groups["count"], -1)
        best = np.argsort(-each.max(-1), kind="stable")[:groups["keep"]]
        may = np.repeat(np.isin(np.arange(groups["count"]), best), each.shape[1])
    chosen = np.argsort(-np.where(may, s, -1.0), kind="stable")[:top]
    return chosen, s[chosen]


def experts(h, W, pre, f):
    r, out = f["router"], np.zeros_like(h)
    z = h @ W[pre + "router"].T
    for t in range(h.shape[0]):
        for e, s in zip(*route(z[t], r["top"], r.get("groups"))):
            out[t] += r["scale"] * s * limited_expert(h[t], W, f"{pre}e{e}.", f["expert"]["limit"])
    return out


def feed_forward(h, W, pre, f):
    return dense(h, W, pre) if f["kind"] == "dense" else experts(h, W, pre, f)


# ---------------------------------------------------------------- the whole model

MIXERS = {"parallel": parallel, "lightning": lightning}


def run_order(cfg):
    order = list(range(len(cfg["layers"])))
    loop = cfg.get("loop")
    if loop:
        a, b = loop["start"], loop["stop"]
        order = order[:a] + order[a:b] * loop["times"] + order[b:]
    return order


def layer(X, W, i, entry, eps):
    def sublayer(q, f):
        c = f"l{i}.hc{q}."
        u = read_streams(X, W[c + "in"])
        return update_streams(X, W[c + "mix"], W[c + "out"], f(rms_norm(u, 1 + W[f"l{i}.norm{q}"], eps)))

    X = sublayer(1, lambda h: MIXERS[entry["type"]](h, W, f"l{i}.mix.", entry["mixer"], eps))
    if entry.get("mlp"):
        X = sublayer(2, lambda h: feed_forward(h, W, f"l{i}.mlp.", entry["mlp"]))
    return X


def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab]; ``layers_out`` takes the sum of the streams after every layer run."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    X = np.repeat(x[:, None, :], cfg["streams"], 1)
    for i in run_order(cfg):
        X = layer(X, W, i, cfg["layers"][i], eps)
        if layers_out is not None:
            layers_out.append(X.sum(1))
    return rms_norm(X.sum(1), 1 + W["final.norm"], eps) @ W["head"].T
