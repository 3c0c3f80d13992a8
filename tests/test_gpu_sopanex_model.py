"""The Sopanex engine (host runtime, paged cache + state arena, batched step, scheduler) on the GPU against the plain
restatement (oracle/sopanex_ref.py) on small random models: whole prompts with the stream after every layer, prefill against
token-by-token decoding, portions down to two tokens (a token pair across the cut), unequal requests in one batch against each alone,
pages, slots, state regions and last tokens that are freed and used again, long decoding across pages and key tiles, a checkpoint
folder through the registry, the trace replay program, greedy generation through the scheduler and the command line."""
import json
import os

import numpy as np
import pytest

import sopanex_common as C

pytestmark = pytest.mark.gpu


def check(got, ref, dtype, what=""):
    """fp32: the typical row agrees to 1e-5 and every row to 1e-4 (a wrong mechanism moves rows by 0.1 and more).  bf16 (milder weights:
    C.random_weights): the typical row inside the rounding tolerance, nine in ten inside twice that, every row inside five times that."""
    e = C.row_err(got, ref)
    if dtype == "float32":
        assert np.median(e) < C.TOL[dtype] and e.max() < 1e-4, (what, float(np.median(e)), float(e.max()), int(e.argmax()))
    else:
        assert np.median(e) < C.TOL[dtype] and (len(e) < 10 or np.quantile(e, 0.9) < 2 * C.TOL[dtype]) and e.max() < 5 * C.TOL[dtype], \
            (what, float(np.median(e)), float(e.max()), int(e.argmax()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_whole_prompt_every_position_and_every_layer_run(name, dtype):
    cfg = C.CONFIGS[name]()
    w = C.weights_for(cfg, 11, dtype)
    toks = C.tokens_for(cfg, 110, 1)
    ref, hid = C.oracle_logits(cfg, w, toks, hidden=True)
    eng = C.engine_for(cfg, w, dtype)
    assert eng.layer_runs == len(hid)
    eng.debug_hidden_enable(True)
    r = eng.new_request()
    got = eng.step([(r, toks)], want=list(range(len(toks))))
    H = eng.debug_hidden(len(toks))
    for i in range(len(hid)):
        per_row = np.abs(H[i] - hid[i]).max(-1) / np.abs(hid[i]).max()
        if dtype == "float32":
            assert np.median(per_row) < C.TOL[dtype] and per_row.max() < 3e-4, (i, float(per_row.max()))
        else:
            assert np.median(per_row) < 5e-2 and np.quantile(per_row, 0.9) < 0.15, (i, float(np.quantile(per_row, 0.9)))
    check(got, ref, dtype)
    if dtype == "bfloat16":          # the tuned GEMM routes and the plain tile kernel agree to rounding
        eng.drop_request(r)
        eng.debug_hidden_enable(False)
        eng.set_plain_kernels(True)
        r = eng.new_request()
        check(eng.step([(r, toks)], want=list(range(len(toks)))), ref, dtype)
    eng.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["a", "odd", "wide", "plain", "b"])
def test_prefill_then_token_by_token(name, dtype):
    cfg = C.CONFIGS[name]()
    w = C.weights_for(cfg, 12, dtype)
    toks = C.tokens_for(cfg, 100, 2)
    ref = C.oracle_logits(cfg, w, toks)
    eng = C.engine_for(cfg, w, dtype)
    r = eng.new_request()
    rows = [eng.step([(r, toks[:15])], want=list(range(15)))]          # 15: the prompt ends one short of a page
    for t in range(15, 100):                                           # decoding passes page borders and the key tile at 64
        rows.append(eng.step([(r, [toks[t]])]))
    check(np.concatenate(rows), ref, dtype)
    r2 = eng.new_request()      # the very first tokens decoded one by one: one key, then two, ...; states from zero
    first = np.concatenate([eng.step([(r2, [toks[t]])]) for t in range(7)])
    check(first, ref[:7], dtype)
    eng.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [[2, 3, 1, 17, 16, 2, 29, 30], [31, 2, 2, 33, 2, 26], [16, 16, 16, 16, 6, 26], [1, 1, 2, 64, 2, 2, 24]])
def test_portions(dtype, sizes):
    cfg = C.config_a()
    w = C.weights_for(cfg, 13, dtype)
    toks = C.tokens_for(cfg, sum(sizes), 3)
    ref = C.oracle_logits(cfg, w, toks)
    eng = C.engine_for(cfg, w, dtype)
    r, at, rows = eng.new_request(), 0, []
    for n in sizes:             # token-by-token and chunked recurrences follow each other; cuts inside pages, key tiles and sub-blocks
        rows.append(eng.step([(r, toks[at:at + n])], want=list(range(n))))
        at += n
    got = np.concatenate(rows)
    check(got, ref, dtype)
    if dtype == "float32":      # cutting the prompt changes next to nothing in the fp32 engine
        r2 = eng.new_request()
        whole = eng.step([(r2, toks)], want=list(range(len(toks))))
        assert np.abs(whole - got).max() <= 1e-4 * np.abs(whole).max()
    eng.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_requests_in_one_batch_against_each_alone(dtype):
    cfg = C.config_a()
    w = C.weights_for(cfg, 14, dtype)
    P = [C.tokens_for(cfg, n, 10 + n) for n in (37, 5, 50, 1)]
    refs = [C.oracle_logits(cfg, w, p) for p in P]
    eng = C.engine_for(cfg, w, dtype, max_tokens=256)
    ids = [eng.new_request() for _ in P]
    # schedule: (request, tokens taken) per step - portions of some beside single tokens of others; a request sits a step out
    plan = [[(0, 20), (1, 2), (3, 1)], [(0, 2), (1, 1), (2, 33)], [(0, 1), (2, 1)], [(0, 14), (1, 2), (2, 16)]]
    at, got = [0] * 4, [[] for _ in P]
    for stp in plan:
        entries, want, off = [], [], 0
        for q, n in stp:
            entries.append((ids[q], P[q][at[q]:at[q] + n]))
            want += list(range(off, off + n))
            off += n
        lg = eng.step(entries, want=want)
        off = 0
        for q, n in stp:
            got[q].append(lg[off:off + n])
            at[q] += n
            off += n
    alone = C.engine_for(cfg, w, dtype, max_tokens=256)
    for q in range(4):
        g = np.concatenate(got[q])
        check(g, refs[q][:at[q]], dtype, q)
        r = alone.new_request()
        solo = alone.step([(r, P[q][:at[q]])], want=list(range(at[q])))
        alone.drop_request(r)
        if dtype == "float32":       # what else is in the batch does not reach a row's arithmetic
            assert np.abs(solo - g).max() <= 1e-4 * np.abs(solo).max(), q
    eng.close()
    alone.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_pages_slots_and_state_regions_are_used_again(dtype):
    cfg = C.config_a()
    w = C.weights_for(cfg, 15, dtype)
    eng = C.engine_for(cfg, w, dtype, max_tokens=96, max_requests=2)      # 6 pages of 16 tokens, 2 slots
    assert eng.capacity_pages() == 6 and eng.state_floats() > 0
    A, B_, Cq, Dq = (C.tokens_for(cfg, n, 20 + n) for n in (40, 50, 30, 33))
    a = eng.new_request()
    check(eng.step([(a, A)], want=list(range(40))), C.oracle_logits(cfg, w, A), dtype)        # 3 pages
    b = eng.new_request()
    with pytest.raises(RuntimeError):
        eng.new_request()                                                                       # both slots are taken
    with pytest.raises(RuntimeError):
        eng.step([(b, B_)])                                                                     # 4 pages wanted, 3 free
    assert eng.seq_len(b) == 0 and eng.available_pages() == 3 and eng.seq_len(a) == 40         # a rejected step changes nothing
    eng.drop_request(a)
    assert eng.available_pages() == 6
    check(eng.step([(b, B_)], want=list(range(50))), C.oracle_logits(cfg, w, B_), dtype)       # reuses a's pages
    c = eng.new_request()        # reuses a's slot: memories start from zero, the first token has none before it
    lg = eng.step([(c, Cq[:20]), (b, [B_[0]])], want=list(range(20)))                          # b decodes on while c starts
    check(lg, C.oracle_logits(cfg, w, Cq)[:20], dtype)
    eng.drop_request(b)
    d = eng.new_request()
    lg = eng.step([(d, Dq), (c, Cq[20:])], want=list(range(33 + 10)))
    check(lg[:33], C.oracle_logits(cfg, w, Dq), dtype)
    check(lg[33:], C.oracle_logits(cfg, w, Cq)[20:], dtype)
    eng.close()


def test_long_decoding_across_pages_and_key_tiles():
    cfg = C.config_tiny()
    w = C.weights_for(cfg, 16, "float32")
    toks = C.tokens_for(cfg, 300, 4)
    ref = C.oracle_logits(cfg, w, toks)
    eng = C.engine_for(cfg, w, "float32", max_tokens=640)
    a, b = eng.new_request(), eng.new_request()
    got = [eng.step([(a, toks[:100])], want=[0, 1, 63, 64, 69, 70, 99])]
    eng.step([(b, toks[:3])], want=[])
    gb = []
    for t in range(100, 300):       # key tiles end at 127 / 191 / 255; b runs 97 tokens behind
        lg = eng.step([(a, [toks[t]]), (b, [toks[t - 97]])])
        got.append(lg[:1])
        gb.append(lg[1])
    check(np.concatenate(got), ref[[0, 1, 63, 64, 69, 70, 99] + list(range(100, 300))], "float32")
    check(np.stack(gb), ref[3:203], "float32")
    eng.close()


def test_a_long_prompt_matches_its_portions_and_the_restatement():
    """2100 tokens in one step (33 key tiles, 33 chunks) against the same prompt in portions
    and the restatement at some positions"""
    cfg = C.config_tiny()
    w = C.weights_for(cfg, 23, "bfloat16")
    toks = C.tokens_for(cfg, 2100, 9)
    want = [0, 15, 16, 63, 64, 69, 70, 71, 72, 73, 500, 1023, 1024, 2047, 2048, 2099]
    ref = C.oracle_logits(cfg, w, toks)[want]
    for dtype in ("bfloat16", "float32"):
        eng = C.engine_for(cfg, w, dtype, max_tokens=4400, max_requests=2)
        a, b = eng.new_request(), eng.new_request()
        whole = eng.step([(a, toks)], want=want)
        check(whole, ref, dtype)
        parts, at = [], 0
        while at < len(toks):
            n = min(150, len(toks) - at)
            wn = [p - at for p in want if at <= p < at + n]
            lg = eng.step([(b, toks[at:at + n])], want=wn)
            if wn:
                parts.append(lg)
            at += n
        got = np.concatenate(parts)
        check(got, ref, dtype)
        assert np.abs(whole - got).max() <= (1e-4 if dtype == "float32" else 0.1) * np.abs(whole).max()
        eng.close()


def test_prompts_long_enough_for_wide_attention_tiles():
    """1500 tokens and eight key/value heads: 64-row tiles, beside short portions of other requests in the same step, against the restatement"""
    cfg = C.base(64, 70, [C.layer((16, 8, 16, 0.25, C.rot(8, 1000.0, (4.0, 300, 16.0, 1.0))), (2, 16, 16, 16.0, 4), (1.1, 0.8), C.moe(16, 4, 2, 2, 1.3, 24)),
                          C.layer((8, 8, 24, 0.2, C.rot(24, 500.0)), (1, 16, 24, 4.0, 4))], bigram=(29, 3, 17))
    w = C.weights_for(cfg, 27, "bfloat16")
    toks, other = C.tokens_for(cfg, 1500, 12), C.tokens_for(cfg, 40, 13)
    want = [0, 1, 15, 16, 62, 63, 64, 65, 127, 128, 700, 1023, 1024, 1490, 1499]
    ref, ref_o = C.oracle_logits(cfg, w, toks)[want], C.oracle_logits(cfg, w, other)
    for dtype in ("bfloat16", "float32"):
        eng = C.engine_for(cfg, w, dtype, max_tokens=3200, max_requests=3)
        a, b = eng.new_request(), eng.new_request()
        check(eng.step([(a, toks)], want=want), ref, dtype)
        eng.step([(b, other[:7])], want=[])
        c = eng.new_request()
        lg = eng.step([(b, other[7:40]), (c, toks)], want=[32] + [33 + p for p in want])
        check(lg[:1], ref_o[39:], dtype)
        check(lg[1:], ref, dtype)
        eng.close()


def test_graph_replays_of_decode_steps_match_eager_steps():
    """single-token steps are replayed from a captured graph: several replays, with prompt steps and synchronisations of other
    requests between them, against the same steps run eagerly (the per-layer tap switches the capture off)"""
    cfg = C.config_a()
    w = C.weights_for(cfg, 21, "bfloat16")
    toks = C.tokens_for(cfg, 60, 7)
    eng = C.engine_for(cfg, w, "bfloat16")
    g, e = eng.new_request(), None
    eng.step([(g, toks[:20])], want=[])
    replayed = []
    for t in range(20, 40):
        replayed.append(eng.step([(g, [toks[t]])])[0])
        if t % 5 == 0:              # eager work of the program between replays
            x = eng.new_request()
            eng.step([(x, toks[:9])])
            eng.drop_request(x)
    eng.debug_hidden_enable(True)
    e = eng.new_request()
    eng.step([(e, toks[:20])], want=[])
    eager = [eng.step([(e, [toks[t]])])[0] for t in range(20, 40)]
    assert np.array_equal(np.stack(replayed), np.stack(eager))
    eng.close()


def test_checkpoint_folder_through_the_registry_and_trace_replay(tmp_path):
    from safetensors.torch import save_file
    from pegainfer_amd import registry
    cfg = C.config_odd()
    w = C.weights_for(cfg, 17, "bfloat16")
    json.dump(C.shipped(cfg), open(tmp_path / "config.json", "w"))
    save_file({k: v.bfloat16().contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    assert registry.family_of(cfg) == "sopanex"
    toks = C.tokens_for(cfg, 25, 5)
    ref = C.oracle_logits(cfg, w, toks)
    for dtype in ("bfloat16", "float32"):
        eng = registry.load_engine(str(tmp_path), dtype=dtype, max_tokens=64, max_requests=2)
        r = eng.new_request()
        check(eng.step([(r, toks)], want=list(range(25))), ref, dtype)
        eng.close()
    with pytest.raises(ValueError):
        registry.load_engine(str(tmp_path), dtype="float16")
    # the trace replay program: two requests, portions, a request that ends and frees its slot, a step that wants nothing
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:7], "want": [6]}, {"id": "y", "tokens": toks[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[7:25], "want": [0, 17]}], "end": ["x"]},
             {"step": 2, "entries": [{"id": "z", "tokens": toks[:3], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "y", "tokens": toks[2:3], "want": [0]}, {"id": "z", "tokens": toks[3:5], "want": [1]}], "end": ["y", "z"]}]
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    V = cfg["vocab"]
    check(np.fromfile(out / "0.f32", dtype="<f4").reshape(-1, V), ref[[6]], "float32")
    check(np.fromfile(out / "1.f32", dtype="<f4").reshape(-1, V), ref[[7, 24]], "float32")
    assert not (out / "2.f32").exists()
    check(np.fromfile(out / "3.f32", dtype="<f4").reshape(-1, V), ref[[2, 4]], "float32")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_scheduler(dtype):
    from pegainfer_amd import registry
    from pegainfer_amd import scheduler as S
    cfg = C.config_a()
    w = C.weights_for(cfg, 18, dtype)
    prompts = [C.tokens_for(cfg, n, 30 + n) for n in (9, 21, 4)]
    eng = C.engine_for(cfg, w, dtype, max_tokens=256, max_requests=4)
    sch = registry.scheduler_for(eng)
    rids = [sch.submit(p, 6, params=(0.0, -1, 1.0, True)) for p in prompts]
    out = {r: [] for r in rids}
    for _ in range(40):
        if sch.step() == 0 and sch.num_active() == 0 and sch.num_deferred() == 0:
            break
        for ev in sch.poll():
            if ev[1] == S.TOKEN:
                out[ev[0]].append(int(ev[2]))
    assert all(len(v) == 6 for v in out.values()), out
    for rid, p in zip(rids, prompts):
        seq = list(p)
        for tok in out[rid]:
            lg = C.oracle_logits(cfg, w, seq)[-1]
            best = int(lg.argmax())
            margin = float(lg[best] - np.partition(lg, -2)[-2])
            thr = 1e-3 if dtype == "float32" else 0.3 * float(lg.std())
            if tok != best:       # only a near tie (bf16: within the rounding noise of the logits) may differ
                assert margin < thr and lg[tok] >= lg[best] - thr
            seq.append(tok)
    assert eng.available_pages() == eng.capacity_pages()          # finished requests gave their pages back
    sch.close()
    eng.close()


def test_command_line_generates_like_the_plain_restatement(tmp_path):
    import subprocess
    import sys
    from safetensors.torch import save_file
    cfg = C.config_tiny()
    w = C.weights_for(cfg, 19, "float32")
    json.dump(C.shipped(cfg), open(tmp_path / "config.json", "w"))
    save_file({k: v.bfloat16().contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    prompt = C.tokens_for(cfg, 11, 6)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run([sys.executable, "-m", "pegainfer_amd", "generate", "--model", str(tmp_path), "--dtype", "float32",
                        "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "5"], cwd=root, capture_output=True,
                       text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    got = json.loads([l for l in p.stdout.split("\n") if l.startswith("{")][-1])["tokens"]
    seq = list(prompt)
    for tok in got:
        lg = C.oracle_logits(cfg, w, seq)[-1]
        assert tok == int(lg.argmax()) or lg[tok] >= lg.max() - 1e-3
        seq.append(tok)
    assert len(got) == 5


def test_synthetic_weights_run_and_stay_finite():
    cfg = C.config_a()
    from pegainfer_amd.sopanex import SopanexEngine
    eng = SopanexEngine(C.shipped(cfg), max_tokens=128, max_requests=2, dtype="bfloat16").fill_synthetic(seed=3, std=0.05)
    r = eng.new_request()
    lg = eng.step([(r, C.tokens_for(cfg, 40, 8))])
    for _ in range(5):
        lg = eng.step([(r, [int(lg[0].argmax())])])
    assert np.isfinite(lg).all() and np.abs(lg).max() > 0
    eng.close()


def test_the_first_tokens_of_requests_side_by_side():
    """one-token prompts, decoded on: every request's first token takes the pair table's extra row, the second the pair's row - also in a
    slot whose last user ended with another token"""
    cfg = C.config_tiny()
    w = C.weights_for(cfg, 25, "float32")
    eng = C.engine_for(cfg, w, "float32", max_tokens=128, max_requests=3)
    P = [C.tokens_for(cfg, 6, 40 + i) for i in range(5)]
    refs = [C.oracle_logits(cfg, w, p) for p in P]
    ids, at, live, todo = {}, {}, [], list(range(5))
    while live or todo:
        while todo and len(live) < 3:
            i = todo.pop(0)
            ids[i], at[i] = eng.new_request(), 0
            live.append(i)
        take = {i: 1 if (at[i] + i) % 3 else min(2, 6 - at[i]) for i in live}
        lg = eng.step([(ids[i], P[i][at[i]:at[i] + take[i]]) for i in live])
        for k, i in enumerate(list(live)):
            at[i] += take[i]
            check(lg[k:k + 1], refs[i][at[i] - 1:at[i]], "float32", (i, at[i]))
            if at[i] == 6:
                eng.drop_request(ids[i])
                live.remove(i)
    eng.close()


def test_configurations_that_cannot_run_are_refused():
    from pegainfer_amd.sopanex import SopanexEngine

    def broken(change):
        cfg = C.shipped(C.config_a())
        change(cfg["layers"])
        with pytest.raises(RuntimeError):
            SopanexEngine(cfg, max_tokens=64, max_requests=1)
    broken(lambda ls: ls[0]["mixer"]["left"].update(vdim=8))                # values are the keys
    broken(lambda ls: ls[0]["mixer"]["left"].update(kv_heads=4))            # heads are no multiple of it
    broken(lambda ls: ls[0]["mixer"]["left"]["rot"].update(dims=26))        # wider than a head
    broken(lambda ls: ls[0]["mixer"]["right"].update(tau=0))
    broken(lambda ls: ls[0]["mixer"].pop("right"))
    broken(lambda ls: ls[0]["mlp"]["router"].update(top=11))                # more choices than experts
    broken(lambda ls: ls[0]["mlp"].update(kind="other"))
    broken(lambda ls: ls[1].update(type="other"))
    cfg = C.config_a()
    w = C.weights_for(cfg, 26, "float32")
    w["l0.mlp.e0.up"] = w["l0.mlp.e0.up"][:-1]                              # a tensor of another size than config.json gives
    with pytest.raises(RuntimeError):
        C.engine_for(cfg, w, "float32")
