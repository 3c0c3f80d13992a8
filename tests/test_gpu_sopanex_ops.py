"""Every Sopanex mechanism alone on the GPU (torch wrappers of pegainfer_amd/ops_blocks.py over the HIP blocks) against its function in
the plain restatement (oracle/sopanex_ref.py), in both storage types; and crafted inputs where random weights would hide a fault: one
far key whose score stands out among hundreds, a sink that takes nearly all of the weight, a write that one key channel keeps and
another forgets, channels that forget at once inside a chunk, identity experts next to real ones, cache pages full of other things,
state regions used by another request before."""
import math

import pytest
import torch

import sopanex_common as C
from oracle import sopanex_ref as R

pytestmark = pytest.mark.gpu

DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
BOTH = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])


def dev(t, dtype):
    return t.to(DT[dtype]).cuda().contiguous()


def close(got, ref, dtype, tol32=2e-5, tol16=3e-2):
    got, ref = got.detach().double().cpu(), ref.double()
    err = float((got - ref).abs().max() / ref.abs().max().clamp_min(1e-9))
    assert err < (tol32 if dtype == "float32" else tol16), err


def B():
    from pegainfer_amd import ops_blocks
    return ops_blocks


def w64(w):
    return {k: v.double() for k, v in w.items()}


def draw(*shape, seed=0, scale=1.0):
    return C.bf16_round(torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale)


# ------------------------------------------------------------------ norms, stream, activations
@BOTH
@pytest.mark.parametrize("d", [50, 88, 1024, 1030, 4100, 9000])
def test_normed_output_joins_the_stream_and_the_next_norm_reads_it(dtype, d):
    x = torch.randn(7, d, generator=torch.Generator().manual_seed(d)) * 2
    y, post, gain = draw(7, d, seed=1, scale=3.0), draw(d, seed=2, scale=0.3), draw(d, seed=3, scale=0.3)
    ref = x.double() + R.zrms(y.double(), post.double(), 1e-3)
    r, n = B().terms_rms(DT[dtype], d, x=x.cuda(), terms=[(dev(y, dtype), None, dev(post, dtype), 1.0)], gain=dev(gain, dtype), eps=1e-3, gain_offset=1.0)
    close(r, ref, "float32", tol32=3e-6)
    close(n, R.zrms(ref, gain.double(), 1e-3), dtype, tol16=1e-2)
    idx = torch.tensor([6, 0, 6, 3], dtype=torch.int32, device="cuda")                 # the end: some rows only
    _, n = B().terms_rms(DT[dtype], d, x=r, row_index=idx, gain=dev(gain, dtype), eps=1e-3, gain_offset=1.0)
    close(n, R.zrms(ref, gain.double(), 1e-3)[[6, 0, 6, 3]], dtype, tol16=1e-2)


@BOTH
@pytest.mark.parametrize("rows", [1, 6, 200])
@pytest.mark.parametrize("d", [50, 1024, 1030, 2048, 4096, 4100, 8192, 9000])
def test_one_launch_joins_norms_and_sums_routed_experts(dtype, rows, d):
    if rows == 200 and d > 2048:
        rows = 130
    g = torch.Generator().manual_seed(d + rows)
    x, y = torch.randn(rows, d, generator=g) * 2, draw(rows, d, seed=1, scale=3.0)
    post, gain = draw(d, seed=2, scale=0.3), draw(d, seed=3, scale=0.3)
    xs = x.cuda()
    n = B().join_rms(xs, dev(post, dtype), dev(gain, dtype), eps=1e-3, gain_offset=1.0, y=dev(y, dtype))
    ref = x.double() + R.zrms(y.double(), post.double(), 1e-3)
    close(xs, ref, "float32", tol32=3e-6)
    close(n, R.zrms(ref, gain.double(), 1e-3), dtype, tol16=1e-2)
    E, I, top = 3, 2, 3
    e = torch.stack([torch.randperm(E + I, generator=g)[:top] for _ in range(rows)]).int()
    wt, yp = torch.rand(rows, top, generator=g), torch.randn(rows * top, d, generator=g)
    yp[(e.view(-1) >= E)] = float("nan")                         # rows no expert has written
    h, add, gate = draw(rows, d, seed=11), draw(rows, d, seed=12), torch.randn(rows, 4, generator=g)
    own = (e >= E)[:, :, None]
    routed = (wt.double()[:, :, None] * torch.where(own, h.double()[:, None], yp.double().view(rows, top, d))).sum(1)
    for extra in (False, True):
        xs = x.cuda()
        kw = dict(add=dev(add, dtype), add_gate_f32=gate.cuda()[:, 2]) if extra else {}
        n = B().join_rms(xs, dev(post, dtype), None if extra else dev(gain, dtype), eps=1e-5, gain_offset=1.0, y_pairs=yp.cuda(), weight=wt.cuda(),
                         expert=e.cuda(), same_from=E, same=dev(h, dtype), **kw)
        t = routed + add.double() * torch.sigmoid(gate[:, 2:3].double()) if extra else routed
        ref = x.double() + R.zrms(t, post.double(), 1e-5)
        close(xs, ref, "float32", tol32=3e-6)
        if extra:
            assert n is None
        else:
            close(n, R.zrms(ref, gain.double(), 1e-5), dtype, tol16=1e-2)


@BOTH
@pytest.mark.parametrize("buckets,muls", [(1, (3, 2)), (29, (3, 17)), (301, (65537, 2147483647))])
def test_stream_starts_from_embedding_and_token_pair_rows(dtype, buckets, muls):
    d, toks = 72, [39, 0, 7, 7, 38]
    E, P, gain = draw(40, d, seed=4), draw(buckets + 1, d, seed=5), draw(d, seed=6, scale=0.3)
    cfg = {"embedding": {"scale": 2.5, "bigram": {"buckets": buckets, "mul_prev": muls[0], "mul_cur": muls[1]}}}
    ref = R.start({"embed": E.double(), "bigram": P.double()}, cfg, toks)
    ids = torch.tensor(toks, dtype=torch.int32, device="cuda")
    kw = dict(embed=dev(E, dtype), token_ids=ids, embed_scale=2.5, gain=dev(gain, dtype), gain_offset=1.0)
    prev = torch.tensor([-1] + toks[:-1], dtype=torch.int32, device="cuda")
    r, n = B().terms_rms(DT[dtype], d, pair_table=dev(P, dtype), prev_ids=prev, muls=muls, **kw)
    close(r, ref, "float32", tol32=1e-6)
    close(n, R.zrms(ref, gain.double(), 1e-5), dtype, tol16=1e-2)
    r, _ = B().terms_rms(DT[dtype], d, **kw)                                            # no table
    close(r, E.double()[toks] * 2.5, "float32", tol32=1e-6)


@BOTH
def test_exact_gelu_alone_and_behind_products(dtype):
    x = draw(9, 77, seed=7, scale=2.0)
    wide = dev(x, dtype)
    close(B().act_rows(wide[:, 3:60], "gelu_erf"), R.gelu_erf(x[:, 3:60].double()), dtype, tol32=1e-6, tol16=1e-2)
    far = torch.tensor([[-30.0, -6.0, -3.0, -0.0, 3.0, 6.0, 30.0, 1.0]])
    close(B().act_rows(far.cuda(), "gelu_erf"), R.gelu_erf(far.double()), "float32", tol32=1e-6)
    for rows, k, m in ((1, 72, 40), (6, 64, 33), (70, 72, 136), (5, 13, 9), (33, 50, 20)):       # few rows, matrix cores, plain
        a, w = draw(rows, k, seed=8), draw(m, k, seed=9, scale=k ** -0.5)
        got = B().linear(dev(a, dtype), dev(w, dtype), epilogue=B().EPI_GELU_ERF)
        close(got, R.gelu_erf(a.double() @ w.double().T), dtype, tol16=1e-2)


# ------------------------------------------------------------------ router, identity experts
@BOTH
@pytest.mark.parametrize("rows", [1, 5, 16, 17, 90])
@pytest.mark.parametrize("E,I,top,scale", [(7, 3, 3, 1.7), (3, 0, 1, 1.0), (2, 6, 5, 1.5), (4, 0, 4, 1.0), (100, 28, 8, 2.5)])
def test_router_chooses_by_corrected_and_weighs_by_plain_scores(dtype, rows, E, I, top, scale):
    z = torch.randn(rows, E + I + 1, generator=torch.Generator().manual_seed(rows + E)) * 2          # one more column beside the logits
    corr = draw(E + I, seed=10, scale=0.2)
    w = {"r.router": torch.eye(E + I, dtype=torch.float64), "r.correction": corr.double()}
    idx, val = R.router(z[:, :E + I].double(), w, "r", {"top": top, "scale": scale})
    for per_tile in (64, 128):
        e, wt, s = B().route_plan(z.cuda(), E + I, top, E, correction=dev(corr, dtype), factor=scale, rows_per_tile=per_tile, dtype=DT[dtype])
        e, wt = e.cpu().long(), wt.cpu().double()
        assert torch.equal(e, idx) and float((wt - val).abs().max()) < 1e-5
        assert not torch.equal(idx.sort(-1).values, torch.topk(z[:, :E + I], top).indices.sort(-1).values) or rows < 90 or top == E + I
        # positions: every pair of a real expert once, grouped by expert, tiles that cover them; identity experts nowhere
        n_real = int((e < E).sum())
        nt = int(s["n_tiles"])
        pp, pr = s["pos_pair"].cpu()[:n_real], s["pos_row"].cpu()[:n_real]
        assert sorted(pp.tolist()) == [i for i in range(rows * top) if int(e.view(-1)[i]) < E] and torch.equal(pr, pp // top)
        assert (s["pos_pair"].cpu()[n_real:] == -7).all() and nt <= s["max_tiles"]
        covered = []
        for t in range(nt):
            g, r0, n = (int(s[k][t]) for k in ("tile_group", "tile_row0", "tile_rows"))
            assert 0 < n <= per_tile and all(int(e.view(-1)[int(pp[i])]) == g for i in range(r0, r0 + n))
            covered += list(range(r0, r0 + n))
        assert sorted(covered) == list(range(n_real))


@BOTH
@pytest.mark.parametrize("rows,d", [(3, 50), (20, 300), (260, 72)])
def test_identity_experts_give_their_input(dtype, rows, d):
    E, I, top = 3, 2, 3
    g = torch.Generator().manual_seed(rows)
    e = torch.stack([torch.randperm(E + I, generator=g)[:top] for _ in range(rows)]).int()
    wt = torch.rand(rows, top, generator=g)
    y = torch.randn(rows * top, d, generator=g)
    y[(e.view(-1) >= E)] = float("nan")                          # rows no expert has written
    h, add, gate = draw(rows, d, seed=11), draw(rows, d, seed=12), torch.randn(rows, 4, generator=g)
    ref = torch.zeros(rows, d, dtype=torch.float64)
    for r in range(rows):
        for c in range(top):
            ref[r] += wt[r, c].double() * (h[r] if e[r, c] >= E else y[r * top + c]).double()
    got = B().route_combine_same(y.cuda(), wt.cuda(), e.cuda(), E, dev(h, dtype))
    close(got, ref, dtype, tol16=1e-2)
    got = B().route_combine_same(y.cuda(), wt.cuda(), e.cuda(), E, dev(h, dtype), add=dev(add, dtype), add_gate_f32=gate.cuda()[:, 2])
    close(got, ref + add.double() * torch.sigmoid(gate[:, 2:3].double()), dtype, tol16=1e-2)


# ------------------------------------------------------------------ attention whose values are its unrotated keys
class Paged:
    """one request's part of scattered pages that hold other things too, filled with NaN"""

    def __init__(self, page_ids, per_token, dtype, page_size=16, lead=80):
        self.offs, at = [], lead
        for n in per_token:
            self.offs.append(at)
            at += page_size * n
        self.page_stride = at + 8
        self.cache = torch.full(((max(page_ids) + 2) * self.page_stride,), float("nan"), dtype=DT[dtype], device="cuda")
        self.indptr = torch.tensor([0, len(page_ids)], dtype=torch.int32, device="cuda")
        self.pids = torch.tensor(page_ids, dtype=torch.int32, device="cuda")


PAGES = [7, 2, 11, 0, 5, 9, 3, 12, 1, 10, 4, 6, 8, 13, 14, 15, 16, 17, 18, 19, 27, 22, 24, 20, 21, 26, 23, 25]
# portions that end just before, at and just after page (16) and key tile (64) borders, then token by token
PORTIONS = [15, 1, 1, 6, 2, 23, 15, 1, 1, 15] + [1] * 70


def attend(qkg, H, G, d, dtype, plan, scale, rot=None, sink=None, gate=True, n_split=1, plain=False, factor=1.0, tail=None,
           tile_rows=16):
    """rows [q | k | gate logits] -> the heads' outputs of every row; tail: key values read from the values (None: all the rotation leaves)"""
    Bk = B()
    dims = rot["dims"] if rot else 0
    tail = d - dims if tail is None else tail
    f, amp = R.turn_frequencies(rot) if rot else ([], 1.0)
    inv = torch.tensor(f, dtype=torch.float32).cuda() if f else None
    pc = Paged(PAGES, [G * (d - tail), G * d], dtype)
    outs, at = [], 0
    for n in plan:
        rg = Bk.Ragged([n], starts=[at])
        x = dev(qkg[at:at + n], dtype)
        q = Bk.qk_prep(x, [0, H * d, H * d], H, G, d, d, rg, pc.indptr, pc.pids, pc.cache, pc.page_stride, pc.offs[0], pc.offs[1], 16, inv_freq=inv,
                       rot_dims=dims, rot_amp=amp, shared_tail=tail)
        outs.append(Bk.paged_attention_opt(q, pc.cache, pc.page_stride, pc.offs[0], pc.offs[1], 16, rg, pc.indptr, pc.pids, G, d, scale,
                                           sink=None if sink is None else dev(sink, dtype), gate=x[:, (H + G) * d:] if gate else None,
                                           n_split=n_split, plain=plain, factor=factor, shared_tail=tail, tile_rows=tile_rows))
        at += n
    return torch.cat(outs)


def attend_ref(qkg, m, sink):
    """the restatement on projections that are given"""
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    n = H * d + G * d + H
    eye = torch.eye(n, dtype=torch.float64)
    w = {"p.q": eye[:H * d], "p.k": eye[H * d:(H + G) * d], "p.g": eye[(H + G) * d:], "p.sink": sink.double(), "p.o": torch.eye(H * d, dtype=torch.float64)}
    return R.shared_kv_attention(qkg.double(), w, "p", m)


@BOTH
@pytest.mark.parametrize("layer", [("a", 0), ("a", 1), ("a", 2), ("b", 1), ("odd", 0), ("odd", 1), ("wide", 0), ("wide", 1), ("plain", 0)])
def test_attention_whole_in_portions_and_split(dtype, layer):
    m = C.CONFIGS[layer[0]]()["layers"][layer[1]]["mixer"]["left"]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    n = 150
    x = draw(n, (H + G) * d + H, seed=13)
    sink = draw(H, seed=14, scale=1.5)
    ref = attend_ref(x, m, sink)
    kw = dict(rot=m.get("rot"), sink=sink)
    tol = dict(tol32=1e-4, tol16=6e-2)
    close(attend(x, H, G, d, dtype, [n], m["scale"], **kw), ref, dtype, **tol)
    close(attend(x, H, G, d, dtype, PORTIONS, m["scale"], **kw), ref, dtype, **tol)
    close(attend(x, H, G, d, dtype, [100] + [1] * 50, m["scale"], n_split=5, **kw), ref, dtype, **tol)
    close(attend(x, H, G, d, dtype, [2, 62, 2, 84], m["scale"], n_split=3, factor=0.5, **kw), ref * 0.5, dtype, **tol)
    close(attend(x, H, G, d, dtype, [n], m["scale"], tail=0, **kw), ref, dtype, **tol)         # keys stored whole
    if dtype == "bfloat16":
        close(attend(x, H, G, d, dtype, [n], m["scale"], plain=True, **kw), ref, dtype, **tol)


@pytest.mark.parametrize("tile_rows", [32, 64])
@pytest.mark.parametrize("heads", [(6, 2, 24, 16, 0.25), (4, 4, 16, 16, 0.3), (5, 1, 32, 8, 0.2), (20, 1, 72, 32, 0.12), (70, 1, 8, 8, 0.4), (4, 2, 136, 64, 0.08),
                                   (2, 1, 256, 128, 0.06), (3, 1, 64, 0, 0.1), (4, 1, 128, 64, 0.1)], ids=lambda h: "x".join(map(str, h[:3])))
def test_prompts_on_wide_tiles(heads, tile_rows):
    """the kernel for prompts (bf16): lengths around its 64-key tiles, portions behind a cached prefix, the 16-row kernel's cache"""
    H, G, d, dims, scale = heads
    ro = C.rot(dims, 300.0, (3.0, 60, 6.0, 0.5)) if dims else None
    sink = draw(H, seed=14, scale=1.5)
    m = {"heads": H, "kv_heads": G, "dim": d, "scale": scale, "rot": ro}
    for n, plan in ((1, [1]), (31, [31]), (64, [64]), (65, [65]), (129, [129]), (200, [200]), (200, [63, 2, 66, 69]), (330, [330]), (330, [1, 128, 201])):
        x = draw(n, (H + G) * d + H, seed=n)
        ref = attend_ref(x, m, sink)
        close(attend(x, H, G, d, "bfloat16", plan, scale, rot=ro, sink=sink, tile_rows=tile_rows), ref, "bfloat16", tol16=6e-2)
    close(attend(x, H, G, d, "bfloat16", plan, scale, rot=ro, sink=sink, tile_rows=tile_rows, tail=0, factor=0.5), ref * 0.5, "bfloat16", tol16=6e-2)


@pytest.mark.parametrize("tile_rows", [32, 64])
@pytest.mark.parametrize("window", [0, 1, 2, 31, 32, 33, 64, 65, 100, 200])
@pytest.mark.parametrize("hot", [0, 31, 32, 63, 64, 130])
def test_a_marked_key_on_wide_tiles_up_to_the_windows_edge(tile_rows, window, hot):
    """every later row reads the one key that stands out while its window (0: none) reaches it; two heads read different values of it"""
    Bk = B()
    n, d = 300, 16
    q, k = torch.zeros(n, 2 * d), torch.zeros(n, d)
    q[:, 8], q[:, d + 8] = 8.0, 8.0
    k[hot, 8], k[hot, 3] = 5.0, 1.0
    x = dev(torch.cat([q, k], 1), "bfloat16")
    pc = Paged(PAGES, [d, d], "bfloat16")
    for plan in ([n], [hot + 1, n - hot - 1]):
        outs, at = [], 0
        for c in plan:
            rg = Bk.Ragged([c], starts=[at])
            qq = Bk.qk_prep(x[at:at + c], [0, 2 * d, 2 * d], 2, 1, d, d, rg, pc.indptr, pc.pids, pc.cache, pc.page_stride, pc.offs[0], pc.offs[1], 16)
            outs.append(Bk.paged_attention_opt(qq, pc.cache, pc.page_stride, pc.offs[0], pc.offs[1], 16, rg, pc.indptr, pc.pids, 1, d, 1.0,
                                               window=window, tile_rows=tile_rows))
            at += c
        got = torch.cat(outs).double().cpu()
        i = torch.arange(n)
        seen = (i >= hot) & ((i - hot < window) if window else (i >= 0))
        for h in range(2):
            assert (got[seen][:, h * d + 3] > 0.99).all() and (got[~seen][:, h * d + 3] == 0).all(), (window, hot, h)


@BOTH
@pytest.mark.parametrize("hot", [0, 1, 15, 16, 63, 64, 101, 300])
def test_one_far_key_stands_out_among_hundreds(dtype, hot):
    """value 3 of every query asks for the one key that has it: later rows read that key as their value, and its unrotated form at that"""
    n, d = 420, 16
    ro = C.rot(8, 50.0, (4.0, 100, 8.0, 1.0))
    x = torch.zeros(n, 2 * d)
    x[:, 10] = 8.0                                   # asked for in the part the rotation leaves
    x[hot, d + 10] = 5.0
    x[hot, d + 1] = 2.0                              # a value inside the rotated part must come out as projected
    for plan, split, rows in (([n], 1, 16), ([hot + 1, n - hot - 1], 1, 16), ([400] + [1] * 20, 7, 16), ([n], 1, 64), ([hot + 1, n - hot - 1], 1, 32)):
        if rows > 16 and dtype == "float32":
            continue
        got = attend(x, 1, 1, d, dtype, plan, 1.0, rot=ro, gate=False, n_split=split, tile_rows=rows).double().cpu()
        assert (got[hot:, 10] > 4.9).all() and ((got[hot:, 1] - 2.0).abs() < 0.05).all(), hot
        assert (got[:hot].abs() < 1e-6).all()


@BOTH
def test_rotated_values_of_a_key_decide_by_distance(dtype):
    """keys and queries alike in the rotated values: the score is amp^2 times a sum of cosines of the distance - against weights computed directly"""
    n, d, ro = 200, 8, C.rot(8, 200.0, (2.0, 64, 6.0, 0.5))
    f, amp = R.turn_frequencies(ro)
    x = torch.zeros(n, 2 * d)
    x[:, :4], x[:, d:d + 4] = 3.0, 1.0
    x[:, d + 4] = draw(n, seed=15)                   # what is read out
    i = torch.arange(n, dtype=torch.float64)
    v = x[:, d + 4].double()
    dist = i[:, None] - i[None]
    s = sum(torch.cos(dist * fk) for fk in f) * 3.0 * amp * amp
    s = s + 3.0 * amp * amp * torch.sin(dist * f[0]) * v[None]       # value 4 turns with value 0
    s = s.masked_fill(dist < 0, -math.inf)
    ref = torch.softmax(s, -1) @ v
    for plan in ([n], [64, 1, 135], [190] + [1] * 10):
        got = attend(x, 1, 1, d, dtype, plan, 1.0, rot=ro, gate=False)[:, 4].double().cpu()
        assert float((got - ref).abs().max()) < (2e-5 if dtype == "float32" else 0.05)


@BOTH
def test_sink_takes_its_share_of_the_weight(dtype):
    """zero queries: with a sink logit s over j visible keys every key weighs 1 / (j + e^s)"""
    n, d = 130, 8
    x = torch.zeros(n, 2 * 2 * d)
    x[:, 2 * d:3 * d] = 1.0
    x[:, 3 * d:] = 1.0
    for s in (-40.0, 0.0, 3.0, 12.0):
        sink = torch.tensor([s, s + 1.0])
        got = attend(x, 2, 2, d, dtype, [70] + [1] * 60, 1.0, sink=sink, gate=False, n_split=2).double().cpu()
        j = torch.arange(1, n + 1, dtype=torch.float64)
        for h in range(2):
            ref = j / (j + math.exp(float(C.bf16_round(sink[h])) if dtype == "bfloat16" else s + h))
            assert float((got[:, h * d] - ref).abs().max()) < (1e-5 if dtype == "float32" else 2e-2), (s, h)


# ------------------------------------------------------------------ gated linear attention
def run_memory(m, qkv, z, bias, dtype, plans, slots, scan_max, dirty=5.0):
    """several requests; plans[i]: rows per step of request i; a step takes the next portion of every request that has one"""
    Bk = B()
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    state = torch.full((max(slots) + 2, H * dk * dv), dirty, device="cuda")
    for s in slots:
        state[s] = 0.0
    at, outs = [0] * len(plans), [[] for _ in plans]
    for k in range(max(len(p) for p in plans)):
        live = [i for i in range(len(plans)) if k < len(plans[i])]
        rg = Bk.Ragged([plans[i][k] for i in live], slots=[slots[i] for i in live], starts=[at[i] for i in live])
        part = lambda src: torch.cat([src[i][at[i]:at[i] + plans[i][k]] for i in live])  # noqa: E731
        o = Bk.gated_linear(dev(part(qkv), dtype), [0, H * dk, 2 * H * dk], part(z).float().cuda().contiguous(), None if bias is None else dev(bias, dtype),
                            m["tau"], dk ** -0.5, state, H, dk, dv, rg, scan_max=scan_max)
        row = 0
        for i in live:
            n = plans[i][k]
            outs[i].append(o[row:row + n])
            row += n
            at[i] += n
    assert float((state[max(slots) + 1] - dirty).abs().max()) == 0.0          # a slot outside the step stays as it was
    return [torch.cat(o) for o in outs], state


def memory_ref(m, qkv, z, bias):
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    n = qkv.shape[0]
    x = qkv.double()
    q, k, v = x[:, :H * dk].view(n, H, dk) * dk ** -0.5, x[:, H * dk:2 * H * dk].view(n, H, dk), x[:, 2 * H * dk:].view(n, H, dv)
    a = torch.exp(torch.nn.functional.logsigmoid(z.double() + (0 if bias is None else bias.double())) / m["tau"]).view(n, H, dk)
    S, end = [torch.zeros(dk, dv, dtype=torch.float64) for _ in range(H)], []
    for h in range(H):
        for t in range(n):
            S[h] = a[t, h][:, None] * S[h] + torch.outer(k[t, h], v[t, h])
        end.append(S[h].reshape(-1))
    return R.linear_memory(q, k, v, a).reshape(n, H * dv), torch.cat(end)


SIZES = [dict(heads=3, dim=12, vdim=20, tau=4.0), dict(heads=1, dim=24, vdim=16, tau=1.0), dict(heads=5, dim=7, vdim=9, tau=3.0),
         dict(heads=2, dim=72, vdim=136, tau=8.0), dict(heads=2, dim=128, vdim=64, tau=16.0), dict(heads=1, dim=128, vdim=256, tau=16.0),
         dict(heads=2, dim=160, vdim=40, tau=2.0), dict(heads=1, dim=33, vdim=70, tau=16.0)]


@BOTH
@pytest.mark.parametrize("m", SIZES, ids=lambda m: "%dx%dx%d" % (m["heads"], m["dim"], m["vdim"]))
def test_gated_linear_attention_token_by_token_and_in_chunks(dtype, m):
    from pegainfer_amd import ffi
    w = m["heads"] * (2 * m["dim"] + m["vdim"])
    lens = (200, 77, 9)
    qkv = [draw(n, w, seed=20 + n) for n in lens]
    z = [draw(n, m["heads"] * m["dim"], seed=30 + n, scale=2.0) for n in lens]
    bias = draw(m["heads"] * m["dim"], seed=23, scale=2.0)
    refs = [memory_ref(m, x, y, bias) for x, y in zip(qkv, z)]
    chunks = ffi.lib().pegainfer_gated_linear_chunked_ok(m["dim"], m["vdim"])
    assert bool(chunks) == (m["dim"] <= 128)
    for plans, scan_max in (([[200], [77], [9]], 0), ([[200], [77], [9]], 32), ([[64, 63, 65, 8], [1, 76], [2, 2, 5]], 32),
                            ([[128, 1, 1, 70], [33, 44], [3, 1, 1, 4]], 32), ([[2, 100, 98], [40, 1, 36], [9]], 1), ([[17, 49, 134], [48, 29], [2, 7]], 1)):
        outs, state = run_memory(m, qkv, z, bias, dtype, plans, [2, 0, 3], scan_max if chunks else 0)
        for i in range(3):
            close(outs[i], refs[i][0], "float32", tol32=1e-5)              # bf16: the stored inputs are exact, everything else is fp32
            close(state[[2, 0, 3][i]], refs[i][1], "float32", tol32=1e-5)


@BOTH
@pytest.mark.parametrize("scan_max", [0, 32])
def test_an_old_write_is_kept_by_one_channel_and_forgotten_by_another(dtype, scan_max):
    """one token writes value 3 through key channels 0 (slow) and 1 (fast); later queries ask for either channel in turn"""
    m = dict(heads=2, dim=8, vdim=8, tau=1.0)
    n, hot = 500, 40
    x, z = torch.zeros(n, 2 * 24), torch.zeros(n, 16)
    for h in range(2):
        x[0::2, h * 8] = 1.0                                      # even tokens ask for channel 0, odd ones for channel 1
        x[1::2, h * 8 + 1] = 1.0
        x[hot, 16 + h * 8:16 + h * 8 + 2] = 2.0
        x[hot, 32 + h * 8 + 3] = 4.0
    z[:, :8] = torch.tensor([8.0, 0.0] + [1.0] * 6)               # head 0: sigmoid(8) and 1/2
    z[:, 8:] = torch.tensor([-60.0, 12.0] + [-5.0] * 6)           # head 1: 1e-26 and nearly one
    ref, _ = memory_ref(m, x, z, None)
    for plan in ([n], [41, 459], [40, 1, 130, 1, 1, 327]):
        out = run_memory(m, [x], [z], None, dtype, [plan], [0], scan_max)[0][0].double().cpu().view(n, 2, 8)
        close(out, ref.view(n, 2, 8), "float32", tol32=1e-5)
        peak = float(out[hot, 0, 3])
        assert peak > 1.0 and (out[:hot] == 0).all()
        keep = 1.0 / (1.0 + math.exp(-8.0))
        assert abs(float(out[n - 2, 0, 3]) / peak - keep ** (n - 2 - hot)) < 1e-4 and float(out[n - 1, 0, 3]) < 1e-30
        assert float(out[hot + 2, 1, 3]) < 1e-24 and abs(float(out[n - 1, 1, 3]) / peak - 1.0) < 1e-2


@BOTH
def test_channels_that_forget_at_once_and_remember_again(dtype):
    """decay inputs between -300 and 300 that change from token to token: products of decays pass through 1e-130, zero and one inside one
    sub-block, and nothing overflows or turns into NaN"""
    m = dict(heads=2, dim=16, vdim=16, tau=1.0)
    n = 150
    x = draw(n, 2 * 48, seed=40)
    g = torch.Generator().manual_seed(41)
    z = torch.randint(0, 5, (n, 32), generator=g).float()
    z = torch.tensor([-300.0, -20.0, 2.0, 9.0, 300.0])[z.long()]
    ref, end = memory_ref(m, x, z, None)
    for plan, sm in (([n], 0), ([n], 32), ([70, 2, 78], 32), ([n], 1)):
        outs, state = run_memory(m, [x], [z], None, dtype, [plan], [0], sm)
        assert torch.isfinite(outs[0]).all()
        close(outs[0], ref, "float32", tol32=1e-5)
        close(state[0], end, "float32", tol32=1e-5)


@BOTH
@pytest.mark.parametrize("m,rank", [(SIZES[0], 6), (SIZES[2], 5), (SIZES[3], 24), (SIZES[4], 96), (SIZES[6], 250)], ids=lambda v: str(v) if isinstance(v, int) else "")
def test_scan_makes_the_decay_inputs_itself(dtype, m, rank):
    """one to four tokens of two requests, the low-rank values inside the rows: the same outputs and states as with the inputs given"""
    Bk = B()
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    rp, wq = (rank + 7) // 8 * 8, H * (2 * dk + dv)
    up = torch.zeros(H * dk, rp)
    up[:, :rank] = draw(H * dk, rank, seed=50, scale=2 * rank ** -0.5)
    bias = draw(H * dk, seed=51)
    for lens in ([1, 1], [3, 1], [4, 4]):
        x = draw(sum(lens), wq + 3 + rp, seed=52)                 # values past the rank are not read as inputs
        z = x[:, wq + 3:wq + 3 + rank].double() @ up[:, :rank].double().T
        start = torch.randn(2, H * dk * dv, generator=torch.Generator().manual_seed(53)).cuda()
        rg, offs = Bk.Ragged(lens), [0, H * dk, 2 * H * dk]
        sa, sb = start.clone(), start.clone()
        a = Bk.gated_linear(dev(x, dtype), offs, z.float().cuda(), dev(bias, dtype), m["tau"], 0.5, sa, H, dk, dv, rg)
        b = Bk.gated_linear(dev(x, dtype), offs, None, dev(bias, dtype), m["tau"], 0.5, sb, H, dk, dv, rg, w_up=dev(up, dtype), low_off=wq + 3, rank=rank)
        close(b, a.cpu(), "float32", tol32=1e-5)
        close(sb, sa.cpu(), "float32", tol32=1e-5)
