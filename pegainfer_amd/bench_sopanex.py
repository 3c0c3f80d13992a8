"""Prefill and decode throughput of Sopanex at layer sizes of a real model, beside the two closest existing models at equal width, head
counts, head sizes, expert sizes and layer count: Feruzen (two mixers side by side in every layer - softmax attention and a matrix
memory - and softmax-routed experts with a shared one) and Ramalix (attention with a sink, a recurrence with a decay per key channel, the
same router with a gated shared expert).  Random weights, bf16, one GPU.
`python bench.py --model sopanex [--sx-size mid]` prints one JSON line; the default bench workload is untouched."""
import json
import sys

from .bench_ramalix import SIZES, measure, ramalix_config

LAYERS = 8


def sopanex_config(s):
    left = {"heads": s["heads"], "kv_heads": s["kv"], "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
            "rot": {"base": 1e6, "dims": 64, "scaling": {"factor": 8.0, "original": 8192, "fast": 32.0, "slow": 1.0}}}
    right = {"heads": s["lin_k"], "dim": 128, "vdim": 128, "tau": 16.0, "rank": s["rank"]}
    moe = {"kind": "moe", "expert": {"ff": s["eff"]}, "router": {"experts": s["experts"], "identity": s["experts"] // 4, "top": s["top"], "scale": 2.0},
           "shared": {"ff": s["sff"]}}
    return {"architecture": "Sopanex", "width": s["width"], "vocab": s["vocab"], "norm": {"eps": 1e-5},
            "embedding": {"scale": 1.0, "bigram": {"buckets": s["vocab"] // 2 - 1, "mul_prev": 9973, "mul_cur": 31}},
            "layers": [{"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": 1.0, "right_scale": 0.7}, "mlp": moe}] * LAYERS}


def feruzen_config(s):
    """the same heads side by side: attention of equal sizes beside a matrix memory of equal sizes, the same expert sizes (gated: three matrices)"""
    moe = {"kind": "moe", "expert": {"ff": s["eff"], "limit": 7.0}, "router": {"experts": s["experts"], "top": s["top"]},
           "shared": {"ff": s["sff"], "limit": 7.0}}
    par = {"left": {"heads": s["heads"], "kv_heads": s["kv"], "dim": 128, "vdim": 128, "rot": {"base": 1e6, "dims": 64}, "scale": 128 ** -0.5},
           "right": {"heads": s["lin_k"], "dim": 128, "vdim": 128, "gate_cap": 15.0}, "left_scale": 1.0, "right_scale": 1.0}
    return {"architecture": "Feruzen", "width": s["width"], "vocab": s["vocab"], "norm": {"eps": 1e-5, "groups": 1}, "canon": {"taps": 4},
            "layers": [{"type": "parallel", "mixer": par, "mlp": moe}] * LAYERS}


def run(args):
    from .feruzen import FeruzenEngine
    from .ramalix import RamalixEngine
    from .sopanex import SopanexEngine
    sizes = [args.sx_size] if args.sx_size != "all" else list(SIZES)
    phase = args.sx_phase                       # one phase alone gives a kernel trace of that phase only
    batches = (1, 4) if phase == "all" else (1,)
    res = {}
    for name in sizes:
        s = SIZES[name]
        sides = {"sopanex": (SopanexEngine, sopanex_config(s)), "feruzen": (FeruzenEngine, feruzen_config(s)),
                 "ramalix": (RamalixEngine, ramalix_config(s))}
        res[name] = {"layers": LAYERS, "sizes": s}
        for side, (cls, cfg) in sides.items():
            if args.sx_only in ("all", side):
                res[name][side if side == "sopanex" else side + "_equal_size"] = measure(cls, cfg, s, args.ctx, args.ctx, batches,
                                                                                       max(2, args.warmup), phase)
                print("%s, %s: done" % (name, side), file=sys.stderr, flush=True)
    print(json.dumps({"metric": "sopanex_layer_throughput_beside_feruzen_and_ramalix", "unit": "tokens/s", "dtype": "bf16",
                      "data": "synthetic", "n_gpus": 1, "prompt_len": args.ctx, "decode_ctx": args.ctx, "results": res}))
    return 0
