"""A plain, slow implementation of the Dobelix design in float64: one function per mechanism, loops
over positions and heads, no cache, no batching, nothing shared with the package.

Notation: x_t the residual stream at position t (counted from 0 per sequence); W maps tensor names
to float tensors; cfg is the config.json dictionary; h the input of a sublayer.

  embedding      x = s E[token]
  layer          x += N1(mixer(x + conv(x)));  x += N2(ff(x)) (if any);  the sublayers read x unnormed
  N(y)           y / sqrt(mean(y^2) + eps) * w
  conv(x)_t      sum_j w[:, j] x_(t - taps + 1 + j), nothing before position 0
  lightning      q = silu(Wq h), k = silu(Wk h), v = silu(Wv h);  S <- decay_head S + k v^T;  o = S^T q
                 out = Wo [N(all heads' o side by side) * sigmoid(Wg h)]
  attention      q = Wq h, k = Wk h, v = k;  q <- N(q), k <- N(k) over the whole projections;  rotation of q and k
                 p_ij = sigmoid(scale temp_head q_i . k_j + pb_head) for j <= i in the same chunk (not normalised over j)
                 out = Wo [(sum_j p_ij v_j, heads side by side) * sigmoid(Wg h)]
  dense ff       Wdown (gelu_tanh(Wgate h) * Wup h)
  output         logit_scale * head N_final(x)
"""
import math

import torch

F64 = torch.float64


def rms_norm(y, w, eps):
    return y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(x, w):
    """x [T, C], w [C, taps]: y_t = sum_j w[:, taps - 1 - j] x_(t - j), nothing before position 0."""
    y = torch.zeros_like(x)
    taps = w.shape[1]
    for t in range(x.shape[0]):
        for j in range(min(taps, t + 1)):
            y[t] += w[:, taps - 1 - j] * x[t - j]
    return y


def rotate_halves(vec, p, dims, base):
    """vec [..., d]: of the first `dims` entries, i and i + dims / 2 turned by the angle p base^(-2i / dims)."""
    out = vec.clone()
    half = dims // 2
    for i in range(half):
        a = p * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, v = vec[..., i], vec[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


# ------------------------------------------------------------------------------------------ mixers
def lightning_scan(q, k, v, decay):
    """q, k [T, H, dk], v [T, H, dv], decay H numbers -> o [T, H, dv]."""
    T, H, dk = q.shape
    o = torch.zeros(T, H, v.shape[2], dtype=F64)
    for hd in range(H):
        S = torch.zeros(dk, v.shape[2], dtype=F64)
        for t in range(T):
            S = decay[hd] * S + torch.outer(k[t, hd], v[t, hd])
            o[t, hd] = S.T @ q[t, hd]
    return o


def lightning(W, p, m, h, eps):
    T, H = h.shape[0], m["heads"]
    q = silu(h @ W[p + "q"].T).view(T, H, m["dim"])
    k = silu(h @ W[p + "k"].T).view(T, H, m["dim"])
    v = silu(h @ W[p + "v"].T).view(T, H, m["vdim"])
    o = lightning_scan(q, k, v, m["decay"]).reshape(T, -1)
    return (rms_norm(o, W[p + "norm"], eps) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def sigmoid_attention(q, k, v, scale, temp, pb, chunk):
    """q [T, H, d], k / v [T, G, .]: unnormalised sigmoid weights within the query's chunk (0: all earlier keys)."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    o = torch.zeros(T, H, v.shape[2], dtype=F64)
    for i in range(T):
        lo = (i // chunk) * chunk if chunk else 0
        for hd in range(H):
            s = (k[lo:i + 1, hd // rep] @ q[i, hd]) * scale * temp[hd]
            o[i, hd] = sigmoid(s + pb[hd]) @ v[lo:i + 1, hd // rep]
    return o


def attention(W, p, m, h, eps):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = h @ W[p + "q"].T, h @ W[p + "k"].T
    v = k.view(T, G, d)
    q = rms_norm(q, W[p + "q.norm"], eps).view(T, H, d)
    k = rms_norm(k, W[p + "k.norm"], eps).view(T, G, d)
    r = m["rot"]
    q = torch.stack([rotate_halves(q[t], t, r["dims"], r["base"]) for t in range(T)])
    k = torch.stack([rotate_halves(k[t], t, r["dims"], r["base"]) for t in range(T)])
    o = sigmoid_attention(q, k, v, m["scale"], W[p + "temp"], W[p + "pb"], (m.get("mask") or {}).get("size") or 0)
    return (o.reshape(T, H * d) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


MIXERS = {"lightning": lightning, "attention": attention}


def dense_ff(W, p, h):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


# ------------------------------------------------------------------------------------------ model
def forward(cfg, W, tokens, streams=None):
    """logits [T, vocab] (float64); streams: a list that receives the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens).long()] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = x + causal_conv(x, W[p + "canon1"])
        x = x + rms_norm(MIXERS[L["type"]](W, p + "mix.", L["mixer"], h, eps), W[p + "norm1"], eps)
        if L.get("mlp"):
            x = x + rms_norm(dense_ff(W, p + "mlp.", x), W[p + "norm2"], eps)
        if streams is not None:
            streams.append(x.clone())
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T * cfg["logit_scale"]
