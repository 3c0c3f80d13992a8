"""Small Sopanex configurations with random weights for the tests.  Sizes are chosen so that values a real model tends to make equal
differ here (head counts of the two mixers, key / value sizes of the memory, rotated and unrotated part, ranks, expert and shared
sizes, the mixers' factors), and so that the special cases are met: no token-pair table, no rotation, a rotation of the whole head,
frequencies with and without long-context scaling, one key/value head and several, more query heads per key/value head than one
attention workgroup holds, decays of several speeds, memories too wide for the chunk form, layers without feed-forward, no identity
experts and more of them than real ones, one choice and nearly all, no shared expert, sizes that are no multiple of eight."""
import numpy as np
import torch

from oracle import sopanex_ref as R


def rot(dims, base, scaling=None):
    r = {"base": base, "dims": dims}
    if scaling:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def layer(left, right, scales=(1.0, 1.0), mlp=None):
    """left: heads, kv_heads, dim, scale, rot or None; right: heads, dim, vdim, tau, rank (a tensor's shape, no part of the configuration)"""
    h, g, d, sc, ro = left
    lf = {"heads": h, "kv_heads": g, "dim": d, "vdim": d, "scale": sc}
    if ro:
        lf["rot"] = ro
    rt = dict(zip(("heads", "dim", "vdim", "tau"), right))
    return {"type": "parallel", "mlp": mlp, "_rank": right[4],
            "mixer": {"left": lf, "right": rt, "left_scale": scales[0], "right_scale": scales[1]}}


def moe(ff, experts, identity, top, scale, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top, "scale": scale}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def base(width, vocab, layers, scale=1.0, bigram=None, eps=1e-5):
    e = {"scale": scale}
    if bigram:
        e["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    return {"architecture": "Sopanex", "width": width, "vocab": vocab, "embedding": e, "norm": {"eps": eps}, "layers": layers}


def config_a():
    """everything; keys far back matter, the ramp of the frequency scaling lies inside the rotated dimensions"""
    return base(88, 131, [
        layer((6, 2, 24, 0.25, rot(12, 300.0, (3.0, 60, 6.0, 0.5))), (3, 12, 20, 4.0, 6), (1.3, 0.6), moe(40, 7, 3, 3, 1.7, 56)),
        layer((4, 4, 16, 0.3, rot(16, 50.0)), (2, 20, 12, 1.0, 11), (0.7, 0.9)),
        layer((5, 1, 32, 0.2, rot(8, 1000.0, (8.0, 30, 4.0, 1.0))), (4, 16, 24, 16.0, 8), (0.8, 1.4), moe(24, 5, 1, 2, 0.8, 32)),
    ], scale=0.7, bigram=(37, 11, 5))


def config_b():
    """single heads, one choice, no identity experts, no shared expert, no pair table; eps of another size"""
    return base(64, 77, [
        layer((1, 1, 24, 0.2, rot(24, 10000.0)), (1, 24, 16, 2.0, 4), (1.0, 1.0), moe(48, 3, 0, 1, 1.0)),
        layer((2, 1, 40, 0.15, rot(20, 500.0)), (2, 8, 8, 8.0, 16), (1.0, 1.0), moe(16, 4, 0, 4, 1.0, 24)),
    ], eps=1e-3)


def config_odd():
    """nothing is a multiple of 8; no rotation in the second layer; a table of one bucket"""
    return base(50, 61, [
        layer((3, 3, 10, 0.3, rot(6, 30.0, (2.0, 20, 3.0, 0.7))), (5, 7, 9, 3.0, 5), (0.9, 1.1), moe(13, 5, 2, 3, 1.2, 11)),
        layer((6, 2, 7, 0.4, None), (1, 11, 5, 1.5, 3), (1.2, 0.4), moe(9, 3, 1, 1, 2.0)),
    ], scale=1.3, bigram=(1, 3, 2))


def config_wide():
    """20 query heads per key/value head, heads wider than a wave, a memory over more than one block of columns and one too wide for the
    chunk form; more identity experts than real ones"""
    return base(128, 90, [
        layer((20, 1, 72, 0.12, rot(32, 2000.0, (4.0, 100, 16.0, 1.0))), (2, 72, 136, 8.0, 24), (1.1, 0.7), moe(32, 2, 6, 5, 1.5, 40)),
        layer((4, 2, 136, 0.08, rot(64, 1e5)), (1, 160, 40, 16.0, 16), (0.6, 1.2), moe(24, 9, 2, 4, 1.1)),
    ], bigram=(301, 65537, 2147483647))


def config_plain():
    """no feed-forward anywhere, no rotation, one state of the largest size the chunk form takes"""
    return base(48, 40, [layer((2, 2, 8, 0.35, None), (1, 128, 256, 16.0, 8), (1.0, 0.5)), layer((3, 1, 12, 0.3, None), (2, 32, 64, 4.0, 8))],
                bigram=(13, 7, 1))


def config_tiny():
    return base(48, 50, [layer((3, 1, 16, 0.3, rot(8, 100.0, (4.0, 50, 8.0, 1.0))), (2, 8, 16, 16.0, 4), (1.2, 0.6), moe(16, 4, 2, 2, 1.3, 24)),
                         layer((4, 2, 8, 0.35, rot(4, 100.0)), (1, 16, 8, 4.0, 4), (0.8, 0.9), moe(16, 3, 1, 2, 1.0))], bigram=(29, 3, 17))


CONFIGS = {"a": config_a, "b": config_b, "odd": config_odd, "wide": config_wide, "plain": config_plain, "tiny": config_tiny}


def shipped(cfg):
    """the configuration as a model folder holds it"""
    c = dict(cfg)
    c["layers"] = [{k: v for k, v in l.items() if not k.startswith("_")} for l in cfg["layers"]]
    return c


def bf16_round(a):
    return torch.as_tensor(np.asarray(a, dtype=np.float32)).bfloat16().float()


def random_weights(cfg, seed=0, soft=False):
    """{name: float32 tensor holding bf16 values}.  soft (for bf16 runs): a rounding that flips one near-tied expert choice moves a row by
    far more than rounding does, and through the caches every later row - so the experts of a layer are nearly alike and the corrections
    settle which identity experts are chosen; fp32 runs take unrelated experts and mild corrections."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]
    w = {}

    def lin(name, o, i, gain=1.5):
        w[name] = bf16_round(torch.randn(o, i, generator=g) * gain / i ** 0.5)

    def vec(name, n, mean=0.0, std=0.3):
        w[name] = bf16_round(mean + std * torch.randn(n, generator=g))

    w["embed"] = bf16_round(torch.randn(V, D, generator=g))
    bg = cfg["embedding"].get("bigram")
    if bg:
        w["bigram"] = bf16_round(0.8 * torch.randn(bg["buckets"] + 1, D, generator=g))
    for i, l in enumerate(cfg["layers"]):
        p, f = "l%d" % i, l.get("mlp")
        a, m, rank = l["mixer"]["left"], l["mixer"]["right"], l["_rank"]
        for n in (".norm1", ".norm1b") + ((".norm2", ".norm2b") if f else ()):
            vec(p + n, D)
        q = p + ".mix.left"
        lin(q + ".q", a["heads"] * a["dim"], D)
        lin(q + ".k", a["kv_heads"] * a["dim"], D)
        vec(q + ".sink", a["heads"], 0.5, 1.0)
        lin(q + ".g", a["heads"], D, 2.0)
        lin(q + ".o", D, a["heads"] * a["dim"])
        q = p + ".mix.right"
        for n, s in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
            lin("%s.%s" % (q, n), m["heads"] * s, D)
        lin(q + ".o", D, m["heads"] * m["vdim"])
        vec(q + ".norm", m["vdim"], 1.0, 0.3)
        lin(q + ".a1", rank, D)
        lin(q + ".a2", m["heads"] * m["dim"], rank, 2.0)
        vec(q + ".a2.b", m["heads"] * m["dim"], 1.0, 1.5)
        if not f:
            continue
        E, I = f["router"]["experts"], f["router"]["identity"]
        for e in range(E):
            for n, o, k in ((".up", f["expert"]["ff"], D), (".down", D, f["expert"]["ff"])):
                own, first = "%s.mlp.e%d%s" % (p, e, n), "%s.mlp.e0%s" % (p, n)
                lin(own, o, k)
                if soft and e:
                    w[own] = bf16_round(w[first] + w[own] / 8.0)
        lin(p + ".mlp.router", E + I, D, 1.0 if soft else 3.0)
        vec(p + ".mlp.correction", E + I, 0.0, 0.05)
        if soft:
            for k in range(I):
                w[p + ".mlp.correction"][E + k] = 10.0 if k < min(I, f["router"]["top"] - 1) else -10.0
        if f.get("shared"):
            lin(p + ".mlp.shared.up", f["shared"]["ff"], D)
            lin(p + ".mlp.shared.down", D, f["shared"]["ff"])
            lin(p + ".mlp.shared.sg", 1, D, 2.0)
    vec("final.norm", D)
    lin("head", V, D)
    return w


def weights_for(cfg, seed, dtype):
    return random_weights(cfg, seed, soft=dtype != "float32")


def engine_for(cfg, w, dtype, max_tokens=512, max_requests=4):
    from pegainfer_amd.sopanex import SopanexEngine
    eng = SopanexEngine(shipped(cfg), max_tokens=max_tokens, max_requests=max_requests, dtype=dtype)
    return eng.load_tensors({k: v.numpy() for k, v in w.items()})


def oracle_logits(cfg, w, tokens, hidden=False):
    out = R.forward(cfg, w, tokens, return_hidden=hidden)
    return (out[0].numpy(), out[1].numpy()) if hidden else out.numpy()


def row_err(got, ref):
    """per row: rms of the difference with its mean taken off, relative to the rms of the reference rows"""
    d = np.asarray(got, dtype=np.float64) - ref
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt(((ref - ref.mean(-1, keepdims=True)) ** 2).mean())


TOL = {"float32": 1e-5, "bfloat16": 4e-2}


def tokens_for(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()
