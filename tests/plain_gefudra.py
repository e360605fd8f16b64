"""A plain, slow implementation of the Gefudra decoder: float64, numpy, whole sequences, no cache, one function per
mechanism.  It imports nothing from the package; the tests compare the engine with it.

A model is ``(cfg, W)``: ``cfg`` the dictionary of config.json, ``W`` a dictionary from tensor names to arrays.

The design in this file's notation.  ``x`` is the residual stream ``[T, width]`` of one sequence, positions ``0 .. T-1``,
``m`` the factor on every branch.

  layer:     x <- x + m mixer(N1(x)), then x <- x + m ff(N2(x));  N is an RMS norm with a weight; no ff, no second line
  loop:      the layers start .. stop - 1 run ``times`` times with the same weights; in front of every pass
             x <- W_in [x, x0], x0 the embedding's rows
  latent:    cq = N(W_dq h), q = W_uq cq;  c = N(W_dkv h), k_h = W_uk_h c, v_h = W_uv_h c;  softmax of scale q . k over the
             last ``size`` keys with exp(sink_h) more in the denominator;  out = W_o (heads * sigmoid(W_g h))
  attention: two maps per head, each with queries and keys of its own over the head's one set of values; a rotation of the
             first ``rot.dims`` dims of each map; scores scale q . k, then softcap tanh(. / softcap); causal softmax;
             o = a_1 - lambda a_2, o / rms(o) (1 - diff), lambda = e^(lq1 . lk1) - e^(lq2 . lk2) + diff;
             out = W_o (heads * sigmoid(W_g h))
  wkv:       every projection s of r, k, v, g, w reads h + (h' - h) mu_s, h' the token before's h;
             w = exp(-exp(W_2 tanh(W_1 .) + w0)) per key channel;
             o = (S + diag(u) k v^T)^T r;  S <- diag(w) S + k v^T;  out = W_o (o / rms(o) * norm * silu(W_g .))
  ff:        g = min(W_gate h, limit), u = W_up h held within +-limit;  W_down (g sigmoid(1.702 g) (u + 1))
  output:    logit_scale N_final(x) @ embed^T
"""
import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def rms_div(x, eps):
    return x / np.sqrt((x ** 2).mean(-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms_div(x, eps) * w


def rotate_half_split(x, positions, base, dims):
    """x [T, heads, dim]: dim i of the first ``dims`` is paired with dim i + dims/2."""
    half = dims // 2
    freq = base ** (-2.0 * np.arange(half) / dims)
    ang = positions[:, None] * freq[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = x.copy()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def visible(T, window=None):
    """[T, T] true where the query of row i sees the key of column j."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = j <= i
    if window:
        seen &= i - j < window
    return seen


def attend(q, k, v, scale, seen, softcap=None, sink=None):
    """One head: q, k [T, dim], v [T, vdim].  ``sink``: one more term exp(sink) in every denominator."""
    s = (q @ k.T) * scale
    if softcap:
        s = softcap * np.tanh(s / softcap)
    s = np.where(seen, s, -np.inf)
    top = s.max(-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink)
    p = np.exp(s - top)
    total = p.sum(-1, keepdims=True)
    if sink is not None:
        total = total + np.exp(sink - top)
    return (p / total) @ v


def latent_attention(h, W, pre, m, eps):
    T = h.shape[0]
    H, dim, vdim = m["heads"], m["dim"], m["vdim"]
    cq = rms_norm(h @ W[pre + "dq"].T, W[pre + "dq.norm"], eps)
    q = (cq @ W[pre + "uq"].T).reshape(T, H, dim)
    c = rms_norm(h @ W[pre + "dkv"].T, W[pre + "dkv.norm"], eps)
    k = (c @ W[pre + "uk"].T).reshape(T, H, dim)
    v = (c @ W[pre + "uv"].T).reshape(T, H, vdim)
    seen = visible(T, m["mask"]["size"] if m.get("mask") else None)
    o = np.stack([attend(q[:, i], k[:, i], v[:, i], m["scale"], seen, sink=W[pre + "sink"][i]) for i in range(H)], 1)
    return (o.reshape(T, H * vdim) * sigmoid(h @ W[pre + "g"].T)) @ W[pre + "o"].T


def difference_weight(W, pre, diff):
    """The factor of the second map: one number for the layer."""
    return np.exp((W[pre + "lq1"] * W[pre + "lk1"]).sum()) - np.exp((W[pre + "lq2"] * W[pre + "lk2"]).sum()) + diff


def differential_attention(h, W, pre, m, eps):
    T = h.shape[0]
    H, G, dim, vdim = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    q = (h @ W[pre + "q"].T).reshape(T, 2 * H, dim)
    k = (h @ W[pre + "k"].T).reshape(T, 2 * G, dim)
    v = (h @ W[pre + "v"].T).reshape(T, G, vdim)
    if m.get("rot"):
        pos = np.arange(T, dtype=np.float64)
        q = rotate_half_split(q, pos, m["rot"]["base"], m["rot"]["dims"])
        k = rotate_half_split(k, pos, m["rot"]["base"], m["rot"]["dims"])
    lam = difference_weight(W, pre, m["diff"])
    seen = visible(T)
    o = np.zeros((T, H, vdim))
    for i in range(H):
        g = i // (H // G)
        a1, a2 = (attend(q[:, 2 * i + n], k[:, 2 * g + n], v[:, g], m["scale"], seen, softcap=m.get("softcap")) for n in (0, 1))
        o[:, i] = rms_div(a1 - lam * a2, eps) * (1.0 - m["diff"])
    return (o.reshape(T, H * vdim) * sigmoid(h @ W[pre + "g"].T)) @ W[pre + "o"].T


def wkv(h, W, pre, m, eps):
    T = h.shape[0]
    H, dim = m["heads"], m["dim"]
    before = np.concatenate([np.zeros_like(h[:1]), h[:-1]], 0)
    mixed = {s: h + (before - h) * W[pre + "mu." + s] for s in "rkvgw"}
    r, k, v = ((mixed[s] @ W[pre + s].T).reshape(T, H, dim) for s in "rkv")
    z = mixed["g"] @ W[pre + "g"].T
    gate = z * sigmoid(z)
    w = np.exp(-np.exp(np.tanh(mixed["w"] @ W[pre + "w1"].T) @ W[pre + "w2"].T + W[pre + "w0"])).reshape(T, H, dim)
    u = W[pre + "u"].reshape(H, dim)
    o = np.zeros((T, H, dim))
    for i in range(H):
        S = np.zeros((dim, dim))
        for t in range(T):
            kv = np.outer(k[t, i], v[t, i])
            o[t, i] = (S + u[i][:, None] * kv).T @ r[t, i]
            S = w[t, i][:, None] * S + kv
    o = rms_div(o, eps).reshape(T, H * dim) * W[pre + "norm"] * gate
    return o @ W[pre + "o"].T


def feed_forward(h, W, pre, f):
    g = np.minimum(h @ W[pre + "gate"].T, f["limit"])
    u = np.clip(h @ W[pre + "up"].T, -f["limit"], f["limit"])
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ W[pre + "down"].T


def run_order(cfg):
    """[(layer, whether the stream is mixed with the embedding in front of it)]"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    out = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        out += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return out + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out``: a list that takes the residual stream after every layer run."""
    W = {k: np.asarray(v, dtype=np.float64) for k, v in W.items()}
    eps, mult = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    x0 = W["embed"][np.asarray(tokens)]
    x = x0
    for i, mixes in run_order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        if mixes:
            x = np.concatenate([x, x0], -1) @ W["loop.in"].T
        h = rms_norm(x, W[p + "norm1"], eps)
        mixer = {"latent_attention": latent_attention, "attention": differential_attention, "wkv": wkv}[layer["type"]]
        x = x + mult * mixer(h, W, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + mult * feed_forward(rms_norm(x, W[p + "norm2"], eps), W, p + "mlp.", layer["mlp"])
        if layers_out is not None:
            layers_out.append(x.copy())
    return cfg.get("logit_scale", 1.0) * (rms_norm(x, W["final.norm"], eps) @ W["embed"].T)
