"""Prefill and decode throughput of Zofadra at layer sizes of a real model, beside the two closest existing models at equal width, head
counts, head sizes, feed-forward size and layer count: Kukulorn (windowed attention with a distance bias, a recurrence with one
decay per head, the same one-step runtime with captured decode steps) and Duguzen (latent attention over the same cache).  Random
weights, bf16, one GPU.
`python bench.py --model zofadra [--zf-size mid]` prints one JSON line; the default bench workload is untouched."""
import json

from .bench_kukulorn import WINDOW, _timed, kukulorn_config
from .bench_kukulorn import SIZES as KK_SIZES

SIZES = {
    # width; attention heads / kv heads x 128; latent heads x (128 + 64) over kv_rank + 64, queries through q_rank; lightning heads
    # x 128 x 128; dense ff; vocab
    "small": dict(width=1024, heads=8, kv=2, q_rank=512, kv_rank=256, ff=3072, vocab=32768),
    "mid": dict(width=2048, heads=16, kv=4, q_rank=768, kv_rank=512, ff=6144, vocab=65536),
    "large": dict(width=4096, heads=32, kv=8, q_rank=1536, kv_rank=512, ff=12288, vocab=65536),
}
LAYERS = 8      # latent, attention, attention, lightning, twice; the second latent layer borrows the first one's latents
STREAMS = 4


def zofadra_config(s):
    ff = {"kind": "dense", "ff": s["ff"]}
    H = s["heads"]
    lat = {"heads": H, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": s["q_rank"], "kv_rank": s["kv_rank"], "scale": 192 ** -0.5,
           "rot": {"base": 5e5, "dims": 64}}
    att = {"heads": H, "kv_heads": s["kv"], "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": WINDOW}}
    lin = {"heads": H, "dim": 128, "vdim": 128, "decay": [1.0 - 2.0 ** (-2.0 - 6.0 * h / H) for h in range(H)]}
    four = [("attention", att), ("attention", att), ("lightning", lin)]
    layers = [("latent_attention", lat)] + four + [("latent_attention", dict(lat, kv_from=0))] + four
    return {"architecture": "Zofadra", "width": s["width"], "vocab": s["vocab"], "embedding": {"scale": 4.0}, "norm": {"eps": 1e-5},
            "residual_mult": 0.5, "streams": STREAMS, "layers": [{"type": t, "mixer": m, "mlp": ff} for t, m in layers]}


def duguzen_config(s):
    """eight layers of latent attention (queries straight from the stream, a sigmoid gate per head) with the same dense feed-forward size"""
    mx = {"heads": s["heads"], "dim": 128, "rot_dim": 64, "kv_rank": s["kv_rank"], "vdim": 128, "rot": {"base": 5e5, "dims": 64},
          "scale": 192 ** -0.5}
    return {"architecture": "Duguzen", "width": s["width"], "vocab": s["vocab"], "norm": {"eps": 1e-5},
            "layers": [{"type": "latent_attention", "mixer": mx, "mlp": {"kind": "dense", "ff": s["ff"]}}] * LAYERS}


def measure(engine_cls, cfg, s, prompt_len, ctx, batches, iters, phase="all"):
    eng = engine_cls(cfg, max_tokens=max(batches) * (ctx + 64) + prompt_len + 64, max_requests=max(batches),
                     dtype="bfloat16").fill_synthetic(seed=1, std=0.02)
    prompt = [(100 + i) % s["vocab"] for i in range(prompt_len)]
    out = {"weight_bytes": eng.weight_bytes()}

    def prefill():
        r = eng.new_request()
        eng.step([(r, prompt)], logits=False, tokens=True)
        eng.drop_request(r)
    if phase in ("all", "prefill"):
        out["prefill_tok_s"] = round(prompt_len / _timed(prefill, iters), 1)
        out["prefill_device_ms"] = round(eng.last_step_ms(), 3)
    for bs in batches if phase in ("all", "decode") else ():
        rids = [eng.new_request() for _ in range(bs)]
        eng.step([(r, prompt[:ctx]) for r in rids], logits=False, tokens=True)
        dt = _timed(lambda: eng.step([(r, [7]) for r in rids], logits=False, tokens=True), max(iters, 20))
        out["decode_bs%d_tok_s" % bs] = round(bs / dt, 1)
        out["decode_bs%d_device_ms" % bs] = round(eng.last_step_ms(), 3)
        for r in rids:
            eng.drop_request(r)
    eng.close()
    return out


def run(args):
    from .duguzen import DuguzenEngine
    from .kukulorn import KukulornEngine
    from .zofadra import ZofadraEngine
    sizes = [args.zf_size] if args.zf_size != "all" else list(SIZES)
    phase = args.zf_phase                       # one phase alone gives a kernel trace of that phase only
    batches = (1, 4) if phase == "all" else (1,)
    res = {}
    for name in sizes:
        s = SIZES[name]
        sides = {"zofadra": (ZofadraEngine, zofadra_config(s)), "kukulorn": (KukulornEngine, kukulorn_config(KK_SIZES[name])),
                 "duguzen": (DuguzenEngine, duguzen_config(s))}
        res[name] = {"layers": LAYERS, "sizes": s}
        for side, (cls, cfg) in sides.items():
            if args.zf_only in ("all", side):
                res[name][side if side == "zofadra" else side + "_equal_size"] = measure(cls, cfg, s, args.ctx, args.ctx, batches,
                                                                                       max(2, args.warmup), phase)
    print(json.dumps({"metric": "zofadra_layer_throughput_beside_kukulorn_and_duguzen", "unit": "tokens/s", "dtype": "bf16",
                      "data": "synthetic", "n_gpus": 1, "prompt_len": args.ctx, "decode_ctx": args.ctx, "results": res}))
    return 0
