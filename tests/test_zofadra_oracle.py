"""The plain restatement of the Zofadra decoder (oracle/zofadra_ref.py) against independent forms of its mechanisms, on the CPU: the
layer norm and the gelu against torch's, the rotation's invariants, the window and the distance bias by explicit loops, latent
attention in its folded form (everything in the latent space), the decayed recurrence against its quadratic form, the streams
against plain residual sums, borrowed latents, causality of the whole model."""
import math

import pytest
import torch
import torch.nn.functional as Fn

import zofadra_common as C
from oracle import zofadra_ref as R

F = torch.float64


def w64(w):
    return {k: v.double() for k, v in w.items()}


def rows(n, d, seed):
    return torch.randn(n, d, generator=torch.Generator().manual_seed(seed), dtype=F)


def test_layer_norm_and_gelu_match_torch():
    x, w = rows(5, 33, 0) * 3 + 2, rows(1, 33, 1)[0]
    assert torch.allclose(R.layer_norm(x, w, 1e-3), Fn.layer_norm(x, (33,), w, None, 1e-3), atol=1e-12)
    assert torch.allclose(R.gelu_tanh(x), Fn.gelu(x, approximate="tanh"), atol=1e-12)
    assert abs(float(R.layer_norm(x + 100.0, w, 1e-3)[0, 0] - R.layer_norm(x, w, 1e-3)[0, 0])) < 1e-9     # the mean comes off


def test_rotation_turns_neighbours_and_depends_on_distance_only():
    rot = {"dims": 6, "base": 40.0}
    q, k = rows(1, 10, 2)[:, None], rows(1, 10, 3)[:, None]
    qs, ks = R.turn_pairs(q.repeat(30, 1, 1), rot), R.turn_pairs(k.repeat(30, 1, 1), rot)
    assert torch.allclose(qs[0], q[0]) and torch.allclose(qs[:, :, 6:], q.repeat(30, 1, 1)[:, :, 6:])
    d5 = [(qs[p + 5, 0] * ks[p, 0]).sum() for p in range(25)]
    assert max(abs(float(v - d5[0])) for v in d5) < 1e-12
    e = torch.zeros(2, 1, 10, dtype=F)
    e[:, 0, 2] = 1.0                                            # value 2 turns with value 3, at the second frequency
    out = R.turn_pairs(e, rot)
    a = 40.0 ** (-2.0 / 6)
    assert abs(float(out[1, 0, 2]) - math.cos(a)) < 1e-12 and abs(float(out[1, 0, 3]) - math.sin(a)) < 1e-12


def test_window_and_distance_bias_by_explicit_loops():
    m = {"heads": 3, "kv_heads": 1, "dim": 4, "vdim": 5, "scale": 0.7, "mask": {"size": 4}}
    g = torch.Generator().manual_seed(4)
    w = {"p." + k: torch.randn(*s, generator=g, dtype=F) for k, s in (("q", (12, 6)), ("k", (4, 6)), ("v", (5, 6)), ("o", (6, 15)),
                                                                       ("q.norm", (12,)), ("k.norm", (4,)))}
    h = rows(9, 6, 5)
    got = R.windowed_attention(h, w, "p", m, 1e-5)
    q, k, v = h @ w["p.q"].T, h @ w["p.k"].T, h @ w["p.v"].T
    out = torch.zeros(9, 15, dtype=F)
    for i in range(9):
        qi = q[i] / math.sqrt(float((q[i] ** 2).mean()) + 1e-5) * w["p.q.norm"]       # one norm over all three heads
        for hd in range(3):
            js = [j for j in range(9) if 0 <= i - j < 4]
            sc = []
            for j in js:
                kj = k[j] / math.sqrt(float((k[j] ** 2).mean()) + 1e-5) * w["p.k.norm"]
                sc.append(float(qi[4 * hd:4 * hd + 4] @ kj) * 0.7 - 2.0 ** (-8.0 * (hd + 1) / 3) * (i - j))
            e = [math.exp(s) for s in sc]
            for j, x in zip(js, e):
                out[i, 5 * hd:5 * hd + 5] += x / sum(e) * v[j]
    assert torch.allclose(got, out @ w["p.o"].T, atol=1e-10)
    one = dict(m, mask={"size": 1})                             # a window of one token: every token reads its own value
    assert torch.allclose(R.windowed_attention(h, w, "p", one, 1e-5), torch.cat([v] * 3, 1) @ w["p.o"].T, atol=1e-10)


def test_latent_attention_equals_its_folded_form():
    cfg = C.config_a()
    w, m, p = w64(C.random_weights(cfg, 6)), cfg["layers"][1]["mixer"], "l1.mix"
    h = rows(17, cfg["width"], 7)
    c, r = R.make_latents(h, w, p, m, 1e-5)
    got = R.latent_attention(h, w, p, m, 1e-5, (c, r))
    H, d, dr, vd, k = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (R.rms(h @ w[p + ".dq"].T, 1e-5) * w[p + ".dq.norm"]) @ w[p + ".uq"].T
    q = q.view(17, H, d + dr)
    uk, uv = w[p + ".uk"].view(H, d, k), w[p + ".uv"].view(H, vd, k)
    qr = R.turn_pairs(q[:, :, d:], m["rot"])
    out = []
    for hd in range(H):
        qc = torch.cat([q[:, hd, :d] @ uk[hd], qr[:, hd]], 1)   # the key up-projection folded into the query
        s = (qc @ torch.cat([c, r], 1).T * m["scale"]).masked_fill(~R.visible_in_window(17, None), float("-inf"))
        out.append(torch.softmax(s, -1) @ c @ uv[hd].T)
    assert torch.allclose(got, torch.cat(out, 1) @ w[p + ".o"].T, atol=1e-9)


def test_decayed_recurrence_equals_its_quadratic_form():
    cfg = C.config_a()
    w, m, p = w64(C.random_weights(cfg, 8)), cfg["layers"][2]["mixer"], "l2.mix"
    h = rows(19, cfg["width"], 9)
    got = R.lightning(h, w, p, m, 1e-5)
    H = m["heads"]
    q, k, v = (Fn.silu(h @ w[p + "." + n].T).view(19, H, -1) for n in "qkv")
    i = torch.arange(19)
    y = []
    for hd in range(H):
        D = torch.where(i[:, None] >= i[None], torch.tensor(m["decay"][hd], dtype=F) ** (i[:, None] - i[None]), torch.zeros((), dtype=F))
        y.append((q[:, hd] @ k[:, hd].T * D) @ v[:, hd])
    y = torch.cat(y, 1)
    y = y / torch.sqrt((y ** 2).mean(-1, keepdim=True) + 1e-5) * w[p + ".norm"] * torch.sigmoid(h @ w[p + ".g"].T)
    assert torch.allclose(got, y @ w[p + ".o"].T, atol=1e-9)


def test_streams():
    X, y = rows(3 * 4, 5, 10).view(3, 4, 5), rows(4, 5, 11)
    M, b = rows(3, 3, 12), rows(1, 3, 13)[0]
    new = R.write_streams(X, M, b, y, 0.3)
    for t in range(3):
        assert torch.allclose(new[t], M[0, t] * X[0] + M[1, t] * X[1] + M[2, t] * X[2] + 0.3 * b[t] * y, atol=1e-12)
    # one stream with weights of one = plain residual sums
    cfg = C.config_b()
    w = C.random_weights(cfg, 14)
    for k in w:
        if ".hc" in k:
            w[k] = torch.ones_like(w[k])
    toks = C.tokens_for(cfg, 9, 1)
    _, hid = R.forward(cfg, w, toks, return_hidden=True)
    ww = w64(w)
    x = ww["embed"][torch.tensor(toks)] * cfg["embedding"]["scale"]
    x = x + cfg["residual_mult"] * R.lightning(R.layer_norm(x, ww["l0.norm1"], 1e-3), ww, "l0.mix", cfg["layers"][0]["mixer"], 1e-3)
    x = x + cfg["residual_mult"] * R.gelu_glu(R.layer_norm(x, ww["l0.norm2"], 1e-3), ww, "l0.mlp")
    assert torch.allclose(hid[0], x, atol=1e-9)


def test_a_borrower_reads_the_latents_of_its_source():
    cfg = C.config_borrow()
    w = C.random_weights(cfg, 15)
    toks = C.tokens_for(cfg, 12, 2)
    _, a = R.forward(cfg, w, toks, return_hidden=True)
    w2 = dict(w)
    w2["l1.mix.dkv"] = w["l1.mix.dkv"] * -1.0                   # layer 1's own latents change: its borrower (3) must notice
    w2["l1.mix.o"] = w["l1.mix.o"] * 0.0
    w3 = dict(w)
    w3["l1.mix.o"] = w["l1.mix.o"] * 0.0                        # the same stream after layer 1, the old latents
    _, b2 = R.forward(cfg, w2, toks, return_hidden=True)
    _, b3 = R.forward(cfg, w3, toks, return_hidden=True)
    assert torch.allclose(b2[:3], b3[:3]) and not torch.allclose(b2[3], b3[3], atol=1e-3) and torch.allclose(a[0], b2[0])
    assert not any(k.startswith("l3.mix.dkv") for k in w)


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_causality(name):
    cfg = C.CONFIGS[name]()
    w = C.random_weights(cfg, 16)
    toks = C.tokens_for(cfg, 14, 3)
    a = C.oracle_logits(cfg, w, toks)
    other = toks[:9] + [(t + 1) % cfg["vocab"] for t in toks[9:]]
    b = C.oracle_logits(cfg, w, other)
    assert abs(a[:9] - b[:9]).max() < 1e-9 and abs(a[9:] - b[9:]).max() > 1e-3
    assert abs(C.oracle_logits(cfg, w, toks[:5]) - a[:5]).max() < 1e-9
