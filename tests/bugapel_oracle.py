"""A plain, slow implementation of the Bugapel design in float64: one function per mechanism, loops
over positions and heads, no cache, no batching, nothing shared with the package.

Notation: X_s (s = 1 .. n) the n streams at position t (counted from 0 per sequence), all equal to the
scaled embedding at first; W maps tensor names to float tensors; cfg is the config.json dictionary.

  sublayer       u = sum_s in_s X_s;  y = f(N(u));  X_t <- sum_s mix_(s,t) X_s + out_t y   (all at once)
  N(u)           (u - mean) / sqrt(mean((u - mean)^2) + eps) * w + b
  attention      q = Wq h, k = Wk h, v = Wv h;  q, k turned (pairs i, i + r/2), then each head over its rms
                 p_ij = exp(s_ij) / (1 + sum_j' exp(s_ij')),  s_ij = scale q_i . k_j,  j <= i
  attention_2    projections with biases, pairs (2i, 2i + 1), p = softmax over j <= i with i - j < w or j < keep
  gla            q = Wq h / sqrt(d), k = Wk h, v = Wv h;  alpha = sigmoid(Wa2 Wa1 h + b)^(1 / tau)
                 S <- diag(alpha) S + k v^T;  o = S^T q;  out = Wo [(o / rms(o) * w, heads side by side) * silu(Wg h)]
  experts        s = softmax(Wr h);  a group's score is its largest s; the `top` largest s within the `keep` best
                 groups, weighted by s / (their sum + 1e-20) * scale;  expert: Wdown relu(Wup h)^2
  output         c tanh(E N_final(sum_s X_s) / c)
"""
import math

import torch

F64 = torch.float64


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def log_sigmoid(z):
    return -torch.clamp(-z, min=0) - torch.log1p(torch.exp(-z.abs()))


# ------------------------------------------------------------------------------------------ streams
def streams_in(X, w):
    """X [T, n, D], w [n] -> the sublayer's input before its norm [T, D]."""
    return sum(w[s] * X[:, s] for s in range(X.shape[1]))


def streams_out(X, y, mix, out):
    """The new streams: from the old ones by mix[from, to], plus out[to] times the sublayer's result."""
    n = X.shape[1]
    return torch.stack([sum(mix[s, t] * X[:, s] for s in range(n)) + out[t] * y for t in range(n)], 1)


# ------------------------------------------------------------------------------------------ rotation
def frequencies(dims, base, scaling=None):
    """The rotation's angular frequencies; with scaling, long wavelengths are stretched by the factor,
    short ones kept, those between blended linearly in original / wavelength."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            wave = 2.0 * math.pi / f
            fac, lo, hi, orig = (float(scaling[n]) for n in ("factor", "low", "high", "original"))
            if wave > orig / lo:
                f = f / fac
            elif wave >= orig / hi:
                s = (orig / wave - lo) / (hi - lo)
                f = (1.0 - s) * f / fac + s * f
        out.append(f)
    return out


def rotate(vec, p, freqs, interleaved):
    """vec [..., d] at position p: pair i of the first 2 len(freqs) entries turned by p freqs[i]."""
    out = vec.clone()
    n = len(freqs)
    for i, f in enumerate(freqs):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + n)
        c, s = math.cos(p * f), math.sin(p * f)
        out[..., a] = vec[..., a] * c - vec[..., b] * s
        out[..., b] = vec[..., b] * c + vec[..., a] * s
    return out


# ------------------------------------------------------------------------------------------ mixers
def visible(i, window, keep):
    """The keys query i sees: all up to i, or the last `window` and the first `keep`."""
    return [j for j in range(i + 1) if not window or i - j < window or j < keep]


def attend(q, k, v, scale, one=False):
    """One query q [H, d] over keys k [n, G, d] and values v [n, G, dv]; one: a 1 is added to the denominator."""
    H = q.shape[0]
    rep = H // k.shape[1]
    o = torch.zeros(H, v.shape[2], dtype=F64)
    for hd in range(H):
        s = (k[:, hd // rep] @ q[hd]) * scale
        m = max(float(s.max()), 0.0)
        e = torch.exp(s - m)
        o[hd] = (e / (e.sum() + (math.exp(-m) if one else 0.0))) @ v[:, hd // rep]
    return o


def softmax_attention(q, k, v, scale, window=0, keep=0, one=False):
    """q [T, H, d], k [T, G, d], v [T, G, dv]; one: a 1 is added to the denominator."""
    seen = [visible(i, window, keep) for i in range(q.shape[0])]
    return torch.stack([attend(q[i], k[js], v[js], scale, one) for i, js in enumerate(seen)])


def attention(W, p, m, h, eps):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q, k = (h @ W[p + "q"].T).view(T, H, -1), (h @ W[p + "k"].T).view(T, G, -1)
    v = (h @ W[p + "v"].T).view(T, G, -1)
    fr = frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    q = unit_rms(torch.stack([rotate(q[t], t, fr, False) for t in range(T)]), eps)
    k = unit_rms(torch.stack([rotate(k[t], t, fr, False) for t in range(T)]), eps)
    return softmax_attention(q, k, v, m["scale"], one=True).reshape(T, -1) @ W[p + "o"].T


def attention_2(W, p, m, h, eps):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q, k, v = (h @ W[p + n].T + W[p + n + ".b"] for n in "qkv")
    q, k, v = q.view(T, H, -1), k.view(T, G, -1), v.view(T, G, -1)
    fr = frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    q = torch.stack([rotate(q[t], t, fr, True) for t in range(T)])
    k = torch.stack([rotate(k[t], t, fr, True) for t in range(T)])
    o = softmax_attention(q, k, v, m["scale"], m["mask"]["size"], m["mask"]["keep_first"])
    return o.reshape(T, -1) @ W[p + "o"].T + W[p + "o.b"]


def gla_scan(q, k, v, alpha):
    """q, k, alpha [T, H, dk], v [T, H, dv] -> o [T, H, dv]."""
    T, H, dk = q.shape
    o = torch.zeros(T, H, v.shape[2], dtype=F64)
    for hd in range(H):
        S = torch.zeros(dk, v.shape[2], dtype=F64)
        for t in range(T):
            S = alpha[t, hd].unsqueeze(1) * S + torch.outer(k[t, hd], v[t, hd])
            o[t, hd] = S.T @ q[t, hd]
    return o


def gla(W, p, m, h, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    q, k = (h @ W[p + "q"].T).view(T, H, d) * d ** -0.5, (h @ W[p + "k"].T).view(T, H, d)
    v = (h @ W[p + "v"].T).view(T, H, -1)
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    alpha = torch.exp(log_sigmoid(z) / m["tau"]).view(T, H, d)
    o = (unit_rms(gla_scan(q, k, v, alpha), eps) * W[p + "norm"]).reshape(T, -1)
    g = h @ W[p + "g"].T
    return (o * g * sigmoid(g)) @ W[p + "o"].T


MIXERS = {"attention": attention, "attention_2": attention_2, "gla": gla}


# ------------------------------------------------------------------------------------------ experts
def route(z, top, groups, keep, scale):
    """One token's router logits z [E] -> ([expert], [weight])."""
    s = torch.exp(z - z.max())
    s = s / s.sum()
    n = z.shape[0] // groups
    best = sorted(range(groups), key=lambda g: -float(s[g * n:(g + 1) * n].max()))[:keep]
    ids = sorted((e for g in best for e in range(g * n, (g + 1) * n)), key=lambda e: -float(s[e]))[:top]
    tot = sum(float(s[e]) for e in ids) + 1e-20
    return ids, [float(s[e]) / tot * scale for e in ids]


def margin(z, top, groups, keep):
    """How far one token's choice is from another one, in logits: between the last kept and the first dropped
    group, and the last chosen and the first passed-over expert."""
    n = z.shape[0] // groups
    gs = sorted(range(groups), key=lambda g: -float(z[g * n:(g + 1) * n].max()))
    es = sorted((float(z[e]) for g in gs[:keep] for e in range(g * n, (g + 1) * n)), reverse=True)
    gaps = [es[top - 1] - es[top]] if top < len(es) else []
    if keep < groups:
        a, b = (float(z[g * n:(g + 1) * n].max()) for g in gs[keep - 1:keep + 1])
        gaps.append(a - b)
    return min(gaps, default=math.inf)


def experts(W, p, f, h, margins=None):
    """margins: a list of one number per token that is lowered to the token's margin here."""
    r = f["router"]
    gr = r.get("groups") or {"count": 1, "keep": 1}
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        if margins is not None:
            margins[t] = min(margins[t], margin(W[p + "router"] @ h[t], r["top"], gr["count"], gr["keep"]))
        for e, w in zip(*route(W[p + "router"] @ h[t], r["top"], gr["count"], gr["keep"], r["scale"])):
            y[t] += w * (W[p + f"e{e}.down"] @ torch.relu(W[p + f"e{e}.up"] @ h[t]) ** 2)
    return y


# ------------------------------------------------------------------------------------------ model
def forward(cfg, W, tokens, streams=None, margins=None):
    """logits [T, vocab] (float64); streams: a list that receives the sum of the streams after every layer;
    margins: a list of one number per token that is lowered to the token's smallest router margin."""
    eps, n = cfg["norm"]["eps"], cfg["streams"]
    x = W["embed"][torch.as_tensor(tokens).long()] * cfg["embedding"]["scale"]
    X = x.unsqueeze(1).repeat(1, n, 1)
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        subs = [lambda h: MIXERS[L["type"]](W, p + "mix.", L["mixer"], h, eps)]
        if L.get("mlp"):
            subs.append(lambda h: experts(W, p + "mlp.", L["mlp"], h, margins))
        for q, f in enumerate(subs, 1):
            y = f(layer_norm(streams_in(X, W[p + f"hc{q}.in"]), W[p + f"norm{q}"], W[p + f"norm{q}.b"], eps))
            X = streams_out(X, y, W[p + f"hc{q}.mix"], W[p + f"hc{q}.out"])
        if streams is not None:
            streams.append(X.sum(1))
    z = layer_norm(X.sum(1), W["final.norm"], W["final.norm.b"], eps) @ W["embed"].T
    c = cfg.get("logit_softcap")
    return c * torch.tanh(z / c) if c else z
