"""Plain, slow restatement of the Sopanex decoder (TEST INFRASTRUCTURE ONLY; nothing in pegainfer_amd/ imports it).

One function per mechanism, one whole sequence at a time, float64 on the CPU, no cache, no state carried between calls:
the recurrence is a Python loop over the tokens from position 0, every attention sees whole score rows.

Notation (n tokens, width D, p = a token's position counted from 0):
  zrms(x, w)      : x / sqrt(mean(x^2) + eps) * (1 + w)                          a gain kept as its offset from one
  start           : x_t = embed[t] * embedding.scale + bigram[row(t-1, t)],  row = (prev * mul_prev + cur * mul_cur) mod buckets;
                    the first token of a sequence reads the table's extra last row
  sublayer f      : x <- x + zrms(f(zrms(x, norm<q>)), norm<q>b)                 q = 1 mixer, 2 feed-forward (a layer may have no second)
  parallel mixer  : left_scale * left(h) + right_scale * right(h), both from the same h
  left            : q = W_q h, k = W_k h, v = k; q and k turned; softmax over the causal keys of (q . k) scale with exp(sink) in the
                    denominator; each head times sigmoid(W_g h)_head; W_o
  turn            : value i with value i + dims / 2 by p f_i, cos and sin times an amplitude.  Without scaling f_i = base^(-2i / dims)
                    and the amplitude is 1.  With it: f_i (1 - r_i) + f_i / factor r_i, r a ramp over i between the two dimensions
                    whose waves turn `fast` and `slow` times over `original` positions; amplitude 0.1 ln(factor) + 1
  right           : q = W_q h dim^-1/2, k = W_k h, v = W_v h; a = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau) per head and key channel;
                    S <- diag(a) S + k v^T, o = S^T q; o / rms(o) * norm per head; times silu(W_g h); W_o
  feed-forward    : s = softmax(W_router h) over experts and identities; the `top` largest s + correction are chosen; weights = their s /
                    (sum + 1e-20) * scale; expert e gives W_down gelu(W_up h) (erf form), an identity gives h; plus the shared expert
                    times sigmoid(W_sg h)
  end             : logits = W_head zrms(x, final.norm)
"""
import json
import math
import os

import torch

F = torch.float64


def read_config(path):
    with open(path if path.endswith(".json") else os.path.join(path, "config.json")) as f:
        return json.load(f)


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def zrms(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def silu(x):
    return x * torch.sigmoid(x)


def gelu_erf(x):
    return 0.5 * x * (1.0 + torch.erf(x / math.sqrt(2.0)))


def bigram_rows(tokens, bg):
    rows = [bg["buckets"]]
    for a, b in zip(tokens[:-1], tokens[1:]):
        rows.append((int(a) * bg["mul_prev"] + int(b) * bg["mul_cur"]) % bg["buckets"])
    return rows


def start(w, cfg, tokens):
    e = cfg["embedding"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * e["scale"]
    if e.get("bigram"):
        x = x + w["bigram"][torch.as_tensor(bigram_rows(tokens, e["bigram"]))]
    return x


def turn_frequencies(rot):
    """(frequencies [dims / 2], amplitude)"""
    dims, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0

    def where(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(where(sc["fast"])), 0), min(math.ceil(where(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def turn_halves(x, rot):
    """x [n, heads, d]"""
    f, amp = turn_frequencies(rot)
    half = rot["dims"] // 2
    out = x.clone()
    for p in range(x.shape[0]):
        for i in range(half):
            c, s = amp * math.cos(p * f[i]), amp * math.sin(p * f[i])
            u, v = x[p, :, i], x[p, :, i + half]
            out[p, :, i] = u * c - v * s
            out[p, :, i + half] = v * c + u * s
    return out


def softmax_with_sink(s, sink):
    """s [n, n] scores of one head; row i sees columns 0 .. i; exp(sink) joins the denominator"""
    n = s.shape[0]
    s = s.masked_fill(torch.ones(n, n, dtype=torch.bool).triu(1), float("-inf"))
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def shared_kv_attention(h, w, p, m):
    n, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w[p + ".q"].T).view(n, H, d)
    k = (h @ w[p + ".k"].T).view(n, G, d)
    v = k
    if m.get("rot"):
        q, k = turn_halves(q, m["rot"]), turn_halves(k, m["rot"])
    gate = torch.sigmoid(h @ w[p + ".g"].T)
    heads = []
    for hd in range(H):
        g = hd // (H // G)
        a = softmax_with_sink(q[:, hd] @ k[:, g].T * m["scale"], w[p + ".sink"][hd])
        heads.append(a @ v[:, g] * gate[:, hd:hd + 1])
    return torch.cat(heads, -1) @ w[p + ".o"].T


def channel_decays(h, w, p, m):
    z = (h @ w[p + ".a1"].T) @ w[p + ".a2"].T + w[p + ".a2.b"]
    return (torch.sigmoid(z) ** (1.0 / m["tau"])).view(h.shape[0], m["heads"], m["dim"])


def linear_memory(q, k, v, a):
    """q, k, a [n, heads, dim], v [n, heads, vdim] -> o [n, heads, vdim], token by token from an empty memory"""
    n, H, d = q.shape
    o = torch.zeros(n, H, v.shape[2], dtype=F)
    for hd in range(H):
        S = torch.zeros(d, v.shape[2], dtype=F)
        for t in range(n):
            S = a[t, hd][:, None] * S + torch.outer(k[t, hd], v[t, hd])
            o[t, hd] = S.T @ q[t, hd]
    return o


def gated_linear_attention(h, w, p, m, eps):
    n, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + ".q"].T).view(n, H, d) * d ** -0.5
    k = (h @ w[p + ".k"].T).view(n, H, d)
    v = (h @ w[p + ".v"].T).view(n, H, dv)
    o = rms(linear_memory(q, k, v, channel_decays(h, w, p, m)), eps) * w[p + ".norm"]
    return (o.reshape(n, H * dv) * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def parallel_mixer(h, w, p, m, eps):
    return (m["left_scale"] * shared_kv_attention(h, w, p + ".left", m["left"]) +
            m["right_scale"] * gated_linear_attention(h, w, p + ".right", m["right"], eps))


def router(h, w, p, r):
    """(choices [n, top], weights [n, top])"""
    s = torch.softmax(h @ w[p + ".router"].T, -1)
    idx = torch.topk(s + w[p + ".correction"], r["top"], dim=-1).indices
    val = torch.gather(s, 1, idx)
    return idx, val / (val.sum(-1, keepdim=True) + 1e-20) * r["scale"]


def expert(h, w, p):
    return gelu_erf(h @ w[p + ".up"].T) @ w[p + ".down"].T


def routed_ff(h, w, p, mlp):
    E = mlp["router"]["experts"]
    idx, val = router(h, w, p, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for c in range(idx.shape[1]):
            e = int(idx[t, c])
            out[t] += val[t, c] * (expert(h[t:t + 1], w, "%s.e%d" % (p, e))[0] if e < E else h[t])
    if mlp.get("shared"):
        out = out + expert(h, w, p + ".shared") * torch.sigmoid(h @ w[p + ".shared.sg"].T)
    return out


def forward(cfg, w, tokens, return_hidden=False):
    """w: {name: tensor}; -> logits [n, vocab] (and the stream after every layer [layers, n, D])"""
    w = {k: v.to(F) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = start(w, cfg, tokens)
    hidden = []
    for i, l in enumerate(cfg["layers"]):
        p = "l%d" % i
        if l["type"] != "parallel":
            raise ValueError(l["type"])
        y = parallel_mixer(zrms(x, w[p + ".norm1"], eps), w, p + ".mix", l["mixer"], eps)
        x = x + zrms(y, w[p + ".norm1b"], eps)
        if l.get("mlp"):
            y = routed_ff(zrms(x, w[p + ".norm2"], eps), w, p + ".mlp", l["mlp"])
            x = x + zrms(y, w[p + ".norm2b"], eps)
        hidden.append(x)
    lg = zrms(x, w["final.norm"], eps) @ w["head"].T
    return (lg, torch.stack(hidden)) if return_hidden else lg
