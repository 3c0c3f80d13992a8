"""Plain, slow restatement of the Zofadra decoder (TEST INFRASTRUCTURE ONLY; nothing in pegainfer_amd/ imports it).

One function per mechanism, one whole sequence at a time, float64 on the CPU, no cache, no state carried between calls:
the recurrence is a Python loop over the tokens from position 0, every attention sees whole score rows.

Notation (n tokens, width D, S = `streams` residual streams, m = `residual_mult`, p = a token's position counted from 0):
  rms(x), ln(x)    : x / sqrt(mean(x^2) + eps);  (x - mean) / sqrt(mean((x - mean)^2) + eps)      over the last axis
  start            : X_s = embed[token] * embedding.scale for every stream s
  sublayer f       : u = sum_s a[s] X_s;  y = f(ln(u) * norm);  X_t <- sum_s M[s, t] X_s + m b[t] y      (all t at once)
                     a, b, M = hc<q>.in, .out, .mix of the layer; q = 1 mixer, 2 feed-forward (a layer may have no second)
  end              : x = sum_s X_s;  logits = W_head (ln(x) * final.norm)
  latent_attention : q = W_uq (rms(W_dq h) w_q), heads [dim | rot_dim];  c | r = W_dkv h, c <- rms(c) w_c, r rotated, shared by
                     the heads; k = W_uk c, v = W_uv c per head; s = (q . k + turn(q_rot) . turn(r)) scale; causal softmax; W_o.
                     kv_from = j: c and turn(r) are those layer j made from ITS input
  turn             : neighbours (2i, 2i + 1) by p base^(-2i / dims)
  attention        : q, k normed as WHOLE rows (all heads at once) with a weight; s = q . k scale - 2^(-8 (h + 1) / H) (i - j);
                     key j visible to i if 0 <= i - j < mask.size; softmax; W_o
  lightning        : q, k, v = silu(W h); per head S <- g_h S + k v^T, y = S^T q; all heads' y normed together by rms, times a
                     weight and sigmoid(W_g h); W_o
  feed-forward     : W_down (gelu(W_gate h) * (W_up h)), the tanh form of gelu
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


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x * x * x)))


def turn_pairs(x, rot):
    """x [n, heads, d]: neighbours (2i, 2i + 1) of the first rot.dims values turn by p * base^(-2i/dims); the rest stays"""
    dims = rot["dims"]
    out = x.clone()
    for p in range(x.shape[0]):
        for i in range(dims // 2):
            a = p * rot["base"] ** (-2.0 * i / dims)
            c, s = math.cos(a), math.sin(a)
            u, v = x[p, :, 2 * i], x[p, :, 2 * i + 1]
            out[p, :, 2 * i] = u * c - v * s
            out[p, :, 2 * i + 1] = v * c + u * s
    return out


def softmax_over_visible(s, visible):
    """s [n, n] scores of one head, visible [n, n] bool; rows are queries"""
    s = s.masked_fill(~visible, float("-inf"))
    s = s - s.max(-1, keepdim=True).values
    e = torch.exp(s)
    return e / e.sum(-1, keepdim=True)


def distances(n):
    i = torch.arange(n)
    return i[:, None] - i[None, :]


def visible_in_window(n, size):
    """size None: every key up to the query; else the query itself and the size - 1 tokens before it"""
    d = distances(n)
    return (d >= 0) if not size else (d >= 0) & (d < size)


def slopes(heads):
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def make_latents(h, w, p, m, eps):
    """what a layer with a W_dkv of its own makes of its input: (c [n, kv_rank], rotated shared key part [n, rot_dim])"""
    a = h @ w[p + ".dkv"].T
    c = rms(a[:, :m["kv_rank"]], eps) * w[p + ".dkv.norm"]
    r = turn_pairs(a[:, None, m["kv_rank"]:], m["rot"])[:, 0]
    return c, r


def latent_attention(h, w, p, m, eps, latents):
    n, H = h.shape[0], m["heads"]
    d, dr, vd = m["dim"], m["rot_dim"], m["vdim"]
    c, r = latents
    cq = rms(h @ w[p + ".dq"].T, eps) * w[p + ".dq.norm"]
    q = (cq @ w[p + ".uq"].T).view(n, H, d + dr)
    qr = turn_pairs(q[:, :, d:], m["rot"])
    k = (c @ w[p + ".uk"].T).view(n, H, d)
    v = (c @ w[p + ".uv"].T).view(n, H, vd)
    vis = visible_in_window(n, None)
    heads = []
    for hd in range(H):
        s = (q[:, hd, :d] @ k[:, hd].T + qr[:, hd] @ r.T) * m["scale"]
        heads.append(softmax_over_visible(s, vis) @ v[:, hd])
    return torch.cat(heads, -1) @ w[p + ".o"].T


def windowed_attention(h, w, p, m, eps):
    n, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (rms(h @ w[p + ".q"].T, eps) * w[p + ".q.norm"]).view(n, H, m["dim"])
    k = (rms(h @ w[p + ".k"].T, eps) * w[p + ".k.norm"]).view(n, G, m["dim"])
    v = (h @ w[p + ".v"].T).view(n, G, m["vdim"])
    vis = visible_in_window(n, (m.get("mask") or {}).get("size"))
    d, sl = distances(n).to(F), slopes(H)
    heads = []
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * m["scale"] - sl[hd] * d
        heads.append(softmax_over_visible(s, vis) @ v[:, g])
    return torch.cat(heads, -1) @ w[p + ".o"].T


def lightning(h, w, p, m, eps):
    n, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[p + ".q"].T).view(n, H, dk)
    k = silu(h @ w[p + ".k"].T).view(n, H, dk)
    v = silu(h @ w[p + ".v"].T).view(n, H, dv)
    y = torch.zeros(n, H, dv, dtype=F)
    for hd in range(H):
        S = torch.zeros(dk, dv, dtype=F)
        for t in range(n):
            S = m["decay"][hd] * S + torch.outer(k[t, hd], v[t, hd])
            y[t, hd] = S.T @ q[t, hd]
    y = rms(y.reshape(n, H * dv), eps) * w[p + ".norm"] * torch.sigmoid(h @ w[p + ".g"].T)
    return y @ w[p + ".o"].T


def gelu_glu(h, w, p):
    return (gelu_tanh(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def read_streams(X, a):
    """X [S, n, D], a [S] -> u [n, D]"""
    return (a[:, None, None] * X).sum(0)


def write_streams(X, M, b, y, mult):
    """every stream at once from the old ones; M is indexed [from, to]"""
    out = torch.zeros_like(X)
    for t in range(X.shape[0]):
        for s in range(X.shape[0]):
            out[t] += M[s, t] * X[s]
        out[t] += mult * b[t] * y
    return out


def forward(cfg, w, tokens, return_hidden=False):
    """w: {name: tensor}; -> logits [n, vocab] (and the summed streams after every layer [layers, n, D])"""
    w = {k: v.to(F) for k, v in w.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x0 = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    X = torch.stack([x0] * cfg["streams"])
    latents, hidden = {}, []
    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d" % i, l["mixer"]
        h = layer_norm(read_streams(X, w[p + ".hc1.in"]), w[p + ".norm1"], eps)
        if l["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                latents[i] = make_latents(h, w, p + ".mix", m, eps)
            y = latent_attention(h, w, p + ".mix", m, eps, latents[i if src is None else src])
        elif l["type"] == "attention":
            y = windowed_attention(h, w, p + ".mix", m, eps)
        elif l["type"] == "lightning":
            y = lightning(h, w, p + ".mix", m, eps)
        else:
            raise ValueError(l["type"])
        X = write_streams(X, w[p + ".hc1.mix"], w[p + ".hc1.out"], y, mult)
        if l.get("mlp"):
            h = layer_norm(read_streams(X, w[p + ".hc2.in"]), w[p + ".norm2"], eps)
            X = write_streams(X, w[p + ".hc2.mix"], w[p + ".hc2.out"], gelu_glu(h, w, p + ".mlp"), mult)
        hidden.append(X.sum(0))
    lg = layer_norm(X.sum(0), w["final.norm"], eps) @ w["head"].T
    return (lg, torch.stack(hidden)) if return_hidden else lg
