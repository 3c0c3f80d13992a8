"""Small Zofadra configurations with random weights for the tests.  Sizes are chosen so that values a real model tends to make
equal differ here (query / value sizes, the rotated and the unrotated part, latent ranks, head counts of every mixer, window
sizes that are no multiple of a page or a key tile), and so that the special cases are met: one to five streams, a layer that
borrows the latents of an earlier one (also with other head counts and sizes), of a late one, several borrowers of one layer, layers
without feed-forward, a window of one token and one wider than any sequence, no window, one key/value head and several, more query
heads per key/value head than one attention workgroup holds, head counts that are no power of two, decays of one and close to
nothing, a model of one kind of layer only, latents too wide or too odd for the matrix-core kernel."""
import numpy as np
import torch

from oracle import zofadra_ref as R


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=500.0, kv_from=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": mlp} if mlp else None}


def attn(heads, kv, dim, vdim, scale, window=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": mlp} if mlp else None}


def lightning(heads, dim, vdim, decay, mlp=None):
    assert len(decay) == heads
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay},
            "mlp": {"kind": "dense", "ff": mlp} if mlp else None}


def base(width, vocab, layers, streams=2, scale=3.0, mult=0.4, eps=1e-5):
    return {"architecture": "Zofadra", "width": width, "vocab": vocab, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "residual_mult": mult, "streams": streams, "layers": layers}


def config_a():
    """every kind of layer; three streams; a window of 21; latents borrowed across an attention and a lightning layer"""
    return base(88, 131, [
        attn(6, 2, 20, 12, 0.22, window=21, mlp=40),
        latent(5, 12, 8, 16, 24, 48, 0.2, mlp=56),
        lightning(3, 12, 20, [0.5, 0.97, 0.999]),
        latent(3, 20, 8, 12, 40, 48, 0.25, base=500.0, kv_from=1, mlp=24),
        attn(4, 1, 28, 8, 0.17, window=40),
        lightning(2, 16, 24, [0.9, 0.3], mlp=32),
    ], streams=3)


def config_b():
    """one stream; a window wider than any test sequence and no window at all; single heads; a decay of one; eps of another size"""
    return base(64, 77, [
        lightning(1, 24, 16, [1.0], mlp=48),
        attn(1, 1, 24, 40, 0.2, window=4096),
        latent(1, 16, 4, 24, 16, 32, 0.2, base=10000.0),
        attn(2, 2, 8, 8, 0.3, mlp=16),
    ], streams=1, scale=1.0, mult=1.0, eps=1e-3)


def config_odd():
    """nothing is a multiple of 8; windows of one and three tokens; the latent runs on the plain kernel; five streams"""
    return base(50, 61, [
        latent(3, 10, 6, 7, 13, 27, 0.3, base=30.0, mlp=14),
        attn(3, 3, 10, 6, 0.3, window=3),
        lightning(5, 7, 9, [0.99, 0.2, 0.75, 0.999, 1e-4], mlp=10),
        latent(2, 6, 6, 11, 9, 27, 0.35, base=30.0, kv_from=0),
        attn(5, 1, 6, 10, 0.4, window=1, mlp=22),
    ], streams=5, mult=0.7)


def config_wide_heads():
    """more query heads per key/value head than an attention workgroup's 16 rows; more latent heads than fit a 64-row tile with
    whole tokens; states and values over more than one 64-column block; values wider than a wave"""
    return base(128, 90, [
        attn(20, 1, 8, 72, 0.3, window=70, mlp=32),
        latent(24, 8, 16, 8, 48, 64, 0.2, mlp=24),
        lightning(2, 72, 136, [0.98, 0.6]),
        latent(9, 24, 16, 24, 32, 64, 0.15, kv_from=1),
        lightning(4, 40, 144, [0.9, 0.95, 0.99, 0.5], mlp=24),
    ], streams=4, mult=0.25)


def config_borrow():
    """two latents of different sizes, each borrowed more than once and in turn"""
    return base(72, 53, [
        latent(2, 8, 4, 12, 20, 16, 0.3, base=100.0),
        latent(4, 12, 8, 8, 16, 32, 0.25, base=1000.0, mlp=24),
        latent(3, 16, 4, 8, 24, 16, 0.3, base=100.0, kv_from=0, mlp=16),
        latent(6, 4, 8, 4, 12, 32, 0.3, base=1000.0, kv_from=1),
        latent(1, 20, 4, 20, 8, 16, 0.2, base=100.0, kv_from=0, mlp=16),
    ], streams=2)


def config_only(kind):
    make = {"latent": lambda i: latent(2 + i, 8, 4, 12, 16, 24 + 8 * i, 0.3, base=100.0, mlp=16 if i != 1 else None),
            "attention": lambda i: attn(2 * (i + 1), 1 + i, 8, 12, 0.35, window=10 + 7 * i, mlp=16 if i % 2 else None),
            "lightning": lambda i: lightning(2, 8 + 4 * i, 12, [0.9, 0.99 - 0.1 * i], mlp=16 if i != 2 else None)}[kind]
    return base(40, 33, [make(i) for i in range(3)], streams=2)


def config_tiny():
    return base(48, 50, [latent(2, 8, 4, 8, 16, 32, 0.3, base=100.0, mlp=16), attn(3, 1, 8, 8, 0.3, window=70, mlp=16),
                         lightning(2, 8, 16, [0.999, 0.9]), latent(2, 8, 4, 8, 16, 32, 0.3, base=100.0, kv_from=0)])


CONFIGS = {"a": config_a, "b": config_b, "odd": config_odd, "wide": config_wide_heads, "borrow": config_borrow, "tiny": config_tiny,
           "only_latent": lambda: config_only("latent"), "only_attention": lambda: config_only("attention"),
           "only_lightning": lambda: config_only("lightning")}


def bf16_round(a):
    return torch.as_tensor(np.asarray(a, dtype=np.float32)).bfloat16().float()


def random_weights(cfg, seed=0):
    """{name: float32 tensor holding bf16 values}"""
    g = torch.Generator().manual_seed(seed)
    D, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    w = {}

    def lin(name, o, i, gain=1.5):
        w[name] = bf16_round(torch.randn(o, i, generator=g) * gain / i ** 0.5)

    def vec(name, n, mean=1.0, std=0.3):
        w[name] = bf16_round(mean + std * torch.randn(n, generator=g))

    w["embed"] = bf16_round(torch.randn(V, D, generator=g))
    for i, l in enumerate(cfg["layers"]):
        p, q, m = "l%d" % i, "l%d.mix" % i, l["mixer"]
        for k in (1, 2) if l.get("mlp") else (1,):
            vec("%s.norm%d" % (p, k), D)
            vec("%s.hc%d.in" % (p, k), S, 1.0 / S, 0.4)
            vec("%s.hc%d.out" % (p, k), S, 1.0, 0.4)
            w["%s.hc%d.mix" % (p, k)] = bf16_round(0.7 * torch.eye(S) + 0.25 * torch.randn(S, S, generator=g))     # not symmetric
        H = m["heads"]
        if l["type"] == "latent_attention":
            lin(q + ".dq", m["q_rank"], D)
            vec(q + ".dq.norm", m["q_rank"])
            lin(q + ".uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"])
            if "kv_from" not in m:
                lin(q + ".dkv", m["kv_rank"] + m["rot_dim"], D)
                vec(q + ".dkv.norm", m["kv_rank"])
            lin(q + ".uk", H * m["dim"], m["kv_rank"])
            lin(q + ".uv", H * m["vdim"], m["kv_rank"])
        elif l["type"] == "attention":
            G = m["kv_heads"]
            lin(q + ".q", H * m["dim"], D)
            lin(q + ".k", G * m["dim"], D)
            lin(q + ".v", G * m["vdim"], D)
            vec(q + ".q.norm", H * m["dim"])
            vec(q + ".k.norm", G * m["dim"])
        else:
            for n, s in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
                lin("%s.%s" % (q, n), H * s, D)
            vec(q + ".norm", H * m["vdim"])
        lin(q + ".o", D, H * m["vdim"])
        if l.get("mlp"):
            ff = l["mlp"]["ff"]
            lin(p + ".mlp.gate", ff, D)
            lin(p + ".mlp.up", ff, D)
            lin(p + ".mlp.down", D, ff)
    vec("final.norm", D)
    lin("head", V, D)
    return w


def engine_for(cfg, w, dtype, max_tokens=512, max_requests=4):
    from pegainfer_amd.zofadra import ZofadraEngine
    eng = ZofadraEngine(cfg, max_tokens=max_tokens, max_requests=max_requests, dtype=dtype)
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
