"""The plain restatement of the Sopanex decoder (oracle/sopanex_ref.py) against independent forms of its mechanisms, on the CPU: norms and
gelu against torch's, the rotation's invariants and its frequency ramp at both ends, values that are keys by explicit loops, the sink's
share, the memory against its quadratic form, the router by hand, the token-pair rows, causality of the whole model; and planted mistakes
that the comparison of the other tests must notice."""
import math

import pytest
import torch
import torch.nn.functional as Fn

import sopanex_common as C
from oracle import sopanex_ref as R

F = torch.float64


def w64(w):
    return {k: v.double() for k, v in w.items()}


def rows(n, d, seed):
    return torch.randn(n, d, generator=torch.Generator().manual_seed(seed), dtype=F)


def test_norm_and_gelu_match_torch():
    x, w = rows(5, 33, 0) * 3 + 2, rows(1, 33, 1)[0]
    assert torch.allclose(R.zrms(x, w, 1e-3), Fn.rms_norm(x, (33,), 1.0 + w, 1e-3), atol=1e-12)
    assert torch.allclose(R.gelu_erf(x), Fn.gelu(x), atol=1e-12)


def test_rotation_pairs_halves_and_depends_on_distance_only():
    for ro in (C.rot(6, 40.0), C.rot(6, 40.0, (4.0, 20, 3.0, 0.5))):
        f, amp = R.turn_frequencies(ro)
        q, k = rows(1, 10, 2)[:, None], rows(1, 10, 3)[:, None]
        qs, ks = R.turn_halves(q.repeat(30, 1, 1), ro), R.turn_halves(k.repeat(30, 1, 1), ro)
        assert torch.allclose(qs[0, 0, :6], q[0, 0, :6] * amp) and torch.allclose(qs[:, :, 6:], q.repeat(30, 1, 1)[:, :, 6:])
        d5 = [(qs[p + 5, 0] * ks[p, 0]).sum() for p in range(25)]
        assert max(abs(float(v - d5[0])) for v in d5) < 1e-12
        e = torch.zeros(2, 1, 10, dtype=F)
        e[:, 0, 1] = 1.0                                        # value 1 turns with value 1 + 3, at the second frequency
        out = R.turn_halves(e, ro)
        assert abs(float(out[1, 0, 1]) - amp * math.cos(f[1])) < 1e-12 and abs(float(out[1, 0, 4]) - amp * math.sin(f[1])) < 1e-12


def test_frequency_ramp_keeps_short_waves_and_stretches_long_ones():
    ro = C.rot(64, 1e4, (4.0, 1000, 32.0, 1.0))
    f, amp = R.turn_frequencies(ro)
    plain, one = R.turn_frequencies(C.rot(64, 1e4))
    assert one == 1.0 and abs(amp - (0.1 * math.log(4.0) + 1.0)) < 1e-15
    for fi, pi in zip(f, plain):
        turns = 1000 * pi / (2 * math.pi)                       # how often this wave turns over the original positions
        assert pi / 4.0 - 1e-15 <= fi <= pi + 1e-15
        if turns > 33.0 * 1.4:
            assert fi == pi
        if turns < 0.7:
            assert abs(fi - pi / 4.0) < 1e-15
    assert f[0] == plain[0] and abs(f[-1] - plain[-1] / 4.0) < 1e-15 and sum(p / 4.0 + 1e-12 < x < p - 1e-12 for x, p in zip(f, plain)) > 5
    assert R.turn_frequencies(C.rot(8, 10.0, (2.0, 1, 5.0, 4.0)))[0] == pytest.approx([x / 2 if i else x for i, x in enumerate(R.turn_frequencies(C.rot(8, 10.0))[0])])


def test_values_are_the_unrotated_keys_with_sink_and_gate_by_explicit_loops():
    m = {"heads": 4, "kv_heads": 2, "dim": 6, "scale": 0.7, "rot": C.rot(4, 9.0, (2.0, 12, 2.0, 0.5))}
    g = torch.Generator().manual_seed(4)
    w = {"p." + k: torch.randn(*s, generator=g, dtype=F) for k, s in (("q", (24, 5)), ("k", (12, 5)), ("o", (5, 24)), ("g", (4, 5)), ("sink", (4,)))}
    h = rows(9, 5, 5)
    f, amp = R.turn_frequencies(m["rot"])

    def turned(x, p):
        y = x.clone()
        for i in range(2):
            c, s = math.cos(p * f[i]) * amp, math.sin(p * f[i]) * amp
            y[i], y[i + 2] = x[i] * c - x[i + 2] * s, x[i + 2] * c + x[i] * s
        return y
    q, k = h @ w["p.q"].T, h @ w["p.k"].T
    out = torch.zeros(9, 24, dtype=F)
    for i in range(9):
        for hd in range(4):
            e, acc = math.exp(float(w["p.sink"][hd])), torch.zeros(6, dtype=F)
            for j in range(i + 1):
                kj = k[j, 6 * (hd // 2):6 * (hd // 2) + 6]
                x = math.exp(0.7 * float(turned(q[i, 6 * hd:6 * hd + 6], i) @ turned(kj, j)))
                e += x
                acc += x * kj
            out[i, 6 * hd:6 * hd + 6] = acc / e * torch.sigmoid(h[i] @ w["p.g"][hd])
    assert torch.allclose(R.shared_kv_attention(h, w, "p", m), out @ w["p.o"].T, atol=1e-10)


def test_memory_equals_its_quadratic_form():
    cfg = C.config_a()
    w, m, p = w64(C.random_weights(cfg, 8)), cfg["layers"][0]["mixer"]["right"], "l0.mix.right"
    h = rows(19, cfg["width"], 9)
    a = R.channel_decays(h, w, p, m)
    assert (a > 0).all() and (a < 1).all()
    q, k, v = (rows(19, 3 * s, 10 + s).view(19, 3, s) for s in (12, 12, 20))
    o = R.linear_memory(q, k, v, a)
    cum = torch.log(a).cumsum(0)                                # logs of the products from the start
    for hd in range(3):
        for i in (0, 1, 7, 18):
            ref = sum(float((q[i, hd] * torch.exp(cum[i, hd] - cum[j, hd])) @ k[j, hd]) * v[j, hd] for j in range(i + 1))
            assert torch.allclose(o[i, hd], ref, atol=1e-10)
    z = (h @ w[p + ".a1"].T) @ w[p + ".a2"].T + w[p + ".a2.b"]
    assert torch.allclose(a.reshape(19, -1), torch.exp(Fn.logsigmoid(z) / m["tau"]), atol=1e-12)


def test_router_by_hand_and_identity_experts():
    r = {"experts": 3, "identity": 2, "top": 2, "scale": 1.5}
    w = {"p.router": torch.eye(5, dtype=F), "p.correction": torch.tensor([0.0, 0.0, 0.0, 0.0, 0.5], dtype=F)}
    h = torch.tensor([[1.0, 3.0, 0.0, 2.0, -2.0], [0.0, 0.0, 4.0, 4.0, 0.0]], dtype=F)
    idx, val = R.router(h, w, "p", r)
    s = torch.softmax(h, -1)
    assert sorted(idx[0].tolist()) == [1, 4] and sorted(idx[1].tolist()) in ([2, 4], [3, 4])     # the correction chooses ...
    got = dict(zip(idx[0].tolist(), val[0].tolist()))
    tot = float(s[0, 1] + s[0, 4])
    assert abs(got[1] - 1.5 * float(s[0, 1]) / tot) < 1e-12 and abs(got[4] - 1.5 * float(s[0, 4]) / tot) < 1e-12   # ... and does not weigh
    w.update({"p.e%d.%s" % (e, n): torch.zeros(*sh, dtype=F) for e in range(3) for n, sh in (("up", (4, 5)), ("down", (5, 4)))})
    out = R.routed_ff(h, w, "p", {"router": r})                 # experts that give nothing: what is left is the identity's share
    assert torch.allclose(out[0], h[0] * got[4], atol=1e-12)


def test_rows_of_token_pairs():
    bg = {"buckets": 7, "mul_prev": 3, "mul_cur": 5}
    assert R.bigram_rows([4, 1, 1, 6], bg) == [7, (12 + 5) % 7, (3 + 5) % 7, (3 + 30) % 7]
    cfg = C.config_tiny()
    w = w64(C.random_weights(cfg, 3))
    x = R.start(w, cfg, [5, 9])
    assert torch.allclose(x[0], w["embed"][5] + w["bigram"][29]) and torch.allclose(x[1], w["embed"][9] + w["bigram"][(5 * 3 + 9 * 17) % 29])


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


PLANTED = {
    "values are the rotated keys": lambda: ("shared_kv_attention", lambda h, w, p, m: _rotated_values(h, w, p, m)),
    "no sink": lambda: ("softmax_with_sink", lambda s, sink: _orig["softmax_with_sink"](s, sink - 1e9)),
    "amplitude left out": lambda: ("turn_frequencies", lambda rot: (_orig["turn_frequencies"](rot)[0], 1.0)),
    "gain without its offset": lambda: ("zrms", lambda x, w, eps: R.rms(x, eps) * w),
    "decay of a whole head": lambda: ("channel_decays", lambda h, w, p, m: _orig["channel_decays"](h, w, p, m).mean(-1, keepdim=True).expand(-1, -1, m["dim"])),
    "first token reads row 0": lambda: ("bigram_rows", lambda t, bg: [0] + _orig["bigram_rows"](t, bg)[1:]),
    "correction weighs too": lambda: ("router", lambda h, w, p, r: _weighing(h, w, p, r)),
}
_orig = {n: getattr(R, n) for n in ("softmax_with_sink", "turn_frequencies", "channel_decays", "bigram_rows", "shared_kv_attention")}


def _rotated_values(h, w, p, m):
    n, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = (R.turn_halves((h @ w[p + x].T).view(n, c, d), m["rot"]) for x, c in ((".q", H), (".k", G)))
    gate = torch.sigmoid(h @ w[p + ".g"].T)
    return torch.cat([R.softmax_with_sink(q[:, i] @ k[:, i // (H // G)].T * m["scale"], w[p + ".sink"][i]) @ k[:, i // (H // G)] * gate[:, i:i + 1]
                      for i in range(H)], -1) @ w[p + ".o"].T


def _weighing(h, w, p, r):
    s = torch.softmax(h @ w[p + ".router"].T, -1) + w[p + ".correction"]
    val, idx = torch.topk(s, r["top"], dim=-1)
    return idx, val / val.sum(-1, keepdim=True) * r["scale"]


@pytest.mark.parametrize("what", sorted(PLANTED))
def test_a_planted_mistake_shows(what, monkeypatch):
    """each mistake moves the logits by far more than the tolerances of the engine's tests"""
    cfg = C.config_a()
    w = C.random_weights(cfg, 11)
    toks = C.tokens_for(cfg, 40, 1)
    ref = C.oracle_logits(cfg, w, toks)
    name, fn = PLANTED[what]()
    monkeypatch.setattr(R, name, fn)
    e = C.row_err(C.oracle_logits(cfg, w, toks), ref)
    assert e.max() > 0.1, (what, float(e.max()))
