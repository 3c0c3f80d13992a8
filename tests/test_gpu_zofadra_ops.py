"""Every Zofadra mechanism alone on the GPU (torch wrappers of pegainfer_amd/ops_blocks.py over the HIP blocks) against its
function in the plain restatement (oracle/zofadra_ref.py), in both storage types; and crafted inputs where random weights would
hide a fault: one far key whose score stands out among hundreds, marked keys just inside and just outside the window in prompts and
in decoding, a distance bias that decides the softmax, a state that one old token wrote and a fast decay forgets, chunk borders,
state regions used by another request before."""
import math

import pytest
import torch

import zofadra_common as C
from oracle import zofadra_ref as R

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


def states(n, d, seed):
    return C.bf16_round(torch.randn(n, d, generator=torch.Generator().manual_seed(seed)))


# ------------------------------------------------------------------ streams
@BOTH
@pytest.mark.parametrize("streams,d", [(1, 50), (2, 256), (2, 1030), (3, 1024), (4, 77), (5, 300), (16, 64), (3, 13000), (4, 2048), (6, 2048)])
def test_output_joins_the_mixed_streams_and_the_next_norm_reads_them(dtype, streams, d):
    g = torch.Generator().manual_seed(streams * d)
    rows, eps = 5, 1e-3
    X = torch.randn(rows, streams, d, generator=g) * 2 + 1
    y, gain = C.bf16_round(torch.randn(rows, d, generator=g)), C.bf16_round(torch.randn(d, generator=g))
    M, b, a = (C.bf16_round(torch.randn(*s, generator=g)) for s in ((streams, streams), (streams,), (streams,)))
    ref = R.write_streams(X.double().permute(1, 0, 2), M.double(), b.double(), y.double(), 0.3)
    u = R.read_streams(ref, a.double())
    kw = dict(y=dev(y, dtype), mix=dev(M, dtype), out_w=dev(b, dtype), mult=0.3, eps=eps)
    new, n, sm = B().stream_mix(X.cuda(), streams, d, DT[dtype], read_w=dev(a, dtype), gain=dev(gain, dtype), want_sum=True, **kw)
    close(new, ref.permute(1, 0, 2), "float32", tol32=3e-6)
    close(sm, ref.sum(0), "float32", tol32=3e-6)
    close(n, R.layer_norm(u, gain.double(), eps), dtype, tol16=1e-2)
    _, n, _ = B().stream_mix(X.cuda(), streams, d, DT[dtype], read_w=dev(a, dtype), gain=dev(gain, dtype), layer_norm=False, keep=False, **kw)
    close(n, R.rms(u, eps) * gain.double(), dtype, tol16=1e-2)
    new, n, sm = B().stream_mix(X.cuda(), streams, d, DT[dtype], **kw)                       # no norm follows
    close(new, ref.permute(1, 0, 2), "float32", tol32=3e-6)
    assert n is None and sm is None
    many = X.repeat(40, 1, 1)                                                                # enough rows for the narrow workgroups
    n2 = B().stream_mix(many.cuda(), streams, d, DT[dtype], read_w=dev(a, dtype), gain=dev(gain, dtype), **dict(kw, y=dev(y.repeat(40, 1), dtype)))[1]
    close(n2, R.layer_norm(u, gain.double(), eps).repeat(40, 1), dtype, tol16=1e-2)
    # the end: a plain sum, some rows only, in another order
    idx = torch.tensor([3, 0, 3], dtype=torch.int32, device="cuda")
    _, n, _ = B().stream_mix(X.cuda(), streams, d, DT[dtype], gain=dev(gain, dtype), eps=eps, row_index=idx, keep=False)
    close(n, R.layer_norm(X.double().sum(1), gain.double(), eps)[[3, 0, 3]], dtype, tol16=1e-2)


@BOTH
def test_streams_start_as_the_scaled_embedding(dtype):
    g = torch.Generator().manual_seed(3)
    E, a, gain = C.bf16_round(torch.randn(40, 72, generator=g)), C.bf16_round(torch.randn(3, generator=g)), C.bf16_round(torch.randn(72, generator=g))
    ids = torch.tensor([39, 0, 7], dtype=torch.int32, device="cuda")
    new, n, _ = B().stream_mix(None, 3, 72, DT[dtype], embed=dev(E, dtype), token_ids=ids, embed_scale=5.5, read_w=dev(a, dtype), gain=dev(gain, dtype))
    x = E[[39, 0, 7]].double() * 5.5
    close(new, torch.stack([x] * 3, 1), "float32", tol32=1e-6)
    close(n, R.layer_norm(x * float(a.double().sum()), gain.double(), 1e-5), dtype, tol16=1e-2)


@BOTH
@pytest.mark.parametrize("shape", [(1, 60), (1, 512), (1, 600), (2, 1500), (1, 4100)])        # a wave per head, then a workgroup per head
def test_norm_over_all_heads_times_gate(dtype, shape):
    heads, vd = shape
    g = torch.Generator().manual_seed(vd)
    o = torch.randn(9, heads * vd, generator=g) * 3
    z, w = C.bf16_round(torch.randn(9, heads * vd + 3, generator=g)), C.bf16_round(1 + 0.2 * torch.randn(vd, generator=g))
    got = B().head_rms_gate(o.cuda(), dev(w, dtype), dev(z, dtype)[:, 3:], "sigmoid", 1.0, 1e-3, heads, vd)
    ref = R.rms(o.double().view(9, heads, vd), 1e-3) * w.double() * torch.sigmoid(z[:, 3:].double()).view(9, heads, vd)
    close(got, ref.reshape(9, -1), dtype, tol16=2e-2)


# ------------------------------------------------------------------ attention
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
# portions that end just before, at and just after page (16), window (21 / 40 / 70) and key tile (32 / 64) borders, then token by token
PORTIONS = [15, 1, 1, 6, 2, 23, 1, 1, 14, 2, 14] + [1] * 70


def run_attention(m, w, p, h, dtype, plan, eps=1e-5, n_split=1, plain=False):
    Bk = B()
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    Wp = torch.cat([w[p + ".q"], w[p + ".k"], w[p + ".v"]])
    pc = Paged(PAGES, [G * d, G * dv], dtype)
    sl = torch.tensor(R.slopes(H), dtype=torch.float32).cuda()
    outs, at = [], 0
    for n in plan:
        rg = Bk.Ragged([n], starts=[at])
        proj = Bk.linear(dev(h[at:at + n], dtype), dev(Wp, dtype), plain=True)
        q = Bk.qk_prep_paged_form(proj, [0, H * d, (H + G) * d], H, G, d, dv, rg, pc.indptr, pc.pids, pc.cache, pc.page_stride, pc.offs[0],
                                  pc.offs[1], 16, q_norm=dev(w[p + ".q.norm"], dtype), k_norm=dev(w[p + ".k.norm"], dtype),
                                  norm_kind="all_weight", eps=eps)
        mix = Bk.paged_attention_opt(q, pc.cache, pc.page_stride, pc.offs[0], pc.offs[1], 16, rg, pc.indptr, pc.pids, G, dv, m["scale"],
                                     window=(m.get("mask") or {}).get("size", 0), dist_slope=sl, n_split=n_split, plain=plain)
        outs.append(Bk.linear(mix, dev(w[p + ".o"], dtype), plain=True))
        at += n
    return torch.cat(outs)


@BOTH
@pytest.mark.parametrize("layer", [("a", 0), ("a", 4), ("b", 1), ("b", 3), ("odd", 1), ("odd", 4), ("wide", 0)])
def test_windowed_attention_with_a_linear_bias_whole_and_in_portions(dtype, layer):
    cfg = C.CONFIGS[layer[0]]()
    w = C.random_weights(cfg, 4)
    p, m = "l%d.mix" % layer[1], cfg["layers"][layer[1]]["mixer"]
    n = 150
    h = states(n, cfg["width"], 8)
    ref = R.windowed_attention(h.double(), w64(w), p, m, 1e-5)
    close(run_attention(m, w, p, h, dtype, [n]), ref, dtype, tol32=1e-4, tol16=6e-2)
    close(run_attention(m, w, p, h, dtype, PORTIONS), ref, dtype, tol32=1e-4, tol16=6e-2)
    close(run_attention(m, w, p, h, dtype, [100] + [1] * 50, n_split=5), ref, dtype, tol32=1e-4, tol16=6e-2)
    if dtype == "bfloat16":
        close(run_attention(m, w, p, h, dtype, [n], plain=True), ref, dtype, tol16=6e-2)


def marked_read(dtype, n, plan, hot, window, slope, gain=40.0, n_split=1):
    """one head of 8 values: the key at `hot` scores `gain`, all others 0; its value row alone is 1.  Returns per row the weight the
    marked key got"""
    Bk = B()
    k, v, q = torch.zeros(n, 8), torch.zeros(n, 8), torch.zeros(n, 8)
    q[:, 0] = 1.0
    k[hot, 0] = gain
    v[hot, 0] = 1.0
    proj = dev(torch.cat([q, k, v], 1), dtype)
    pc = Paged(PAGES, [8, 8], dtype)
    outs, at = [], 0
    for c in plan:
        rg = Bk.Ragged([c], starts=[at])
        qq = Bk.qk_prep_paged_form(proj[at:at + c], [0, 8, 16], 1, 1, 8, 8, rg, pc.indptr, pc.pids, pc.cache, pc.page_stride, pc.offs[0],
                                   pc.offs[1], 16, norm_kind="head_weight")
        outs.append(Bk.paged_attention_opt(qq, pc.cache, pc.page_stride, pc.offs[0], pc.offs[1], 16, rg, pc.indptr, pc.pids, 1, 8, 1.0,
                                           window=window, dist_slope=torch.tensor([slope], dtype=torch.float32).cuda(), n_split=n_split))
        at += c
    return torch.cat(outs)[:, 0].double().cpu()


@BOTH
@pytest.mark.parametrize("window", [1, 2, 16, 17, 63, 64, 65, 100])
@pytest.mark.parametrize("hot", [0, 15, 64, 101])
def test_a_marked_key_is_seen_up_to_the_windows_edge_and_not_beyond(dtype, window, hot):
    n = 210
    for plan, split in (([n], 1), ([hot + 1, n - hot - 1], 1), ([100] + [1] * (n - 100), 4)):
        got = marked_read(dtype, n, plan, hot, window, slope=0.0, n_split=split)
        i = torch.arange(n)
        seen = (i >= hot) & (i - hot < window)
        assert (got[seen] > 0.99).all() and (got[~seen] == 0).all(), (window, hot)


@BOTH
def test_the_distance_bias_decides_the_softmax(dtype):
    """a key 30 better than all others, and a slope of 1/4 per token: it wins up to a distance of about 120 and is gone beyond 200 -
    against softmax weights computed directly"""
    n, hot, slope = 420, 3, 0.25
    i = torch.arange(n, dtype=torch.float64)
    d = i[:, None] - i[None]
    s = torch.where(d >= 0, -slope * d, torch.full_like(d, -math.inf))
    s[:, hot] += torch.where(i >= hot, 30.0, 0.0)
    ref = torch.softmax(s, -1)[:, hot]
    assert ref[100] > 0.9 and ref[400] < 1e-9
    for plan, split in (([n], 1), ([400] + [1] * 20, 7)):
        got = marked_read(dtype, n, plan, hot, 0, slope, gain=30.0, n_split=split)
        assert float((got[hot:] - ref[hot:]).abs().max()) < (1e-5 if dtype == "float32" else 1e-2)


def run_latent(m, w, p, h, dtype, plan, eps=1e-5, n_split=1, tiled=True, pc=None, own=True):
    """the mixer as the runtime strings it together; own=False reads the entries another run has left in pc"""
    Bk = B()
    H, d, dr, dv, r, qr = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
    pc = pc or Paged(PAGES, [r + dr], dtype)
    f = torch.tensor([m["rot"]["base"] ** (-2.0 * i / dr) for i in range(dr // 2)], dtype=torch.float32).cuda()
    Wp = torch.cat([w[p + ".dq"]] + ([w[p + ".dkv"]] if own else []))
    uk = dev(w[p + ".uk"].view(H, d, r).transpose(1, 2), dtype)
    args = (pc.indptr, pc.pids, pc.cache, pc.page_stride, pc.offs[0], 16, H, d, dr, r, eps, f, True)
    outs, at = [], 0
    for n in plan:
        rg = Bk.Ragged([n], starts=[at])
        proj = Bk.linear(dev(h[at:at + n], dtype), dev(Wp, dtype), plain=True)
        kw = dict(dkv=proj[:, qr:], c_norm_w=dev(w[p + ".dkv.norm"], dtype)) if own else {}
        cq = Bk.latent_prep_form(rg, *args, ql=proj[:, :qr], ql_norm_w=dev(w[p + ".dq.norm"], dtype), **kw)
        q = Bk.linear(cq, dev(w[p + ".uq"], dtype), plain=True)
        qc = torch.full((n, H, r + dr), float("nan"), dtype=torch.float32, device="cuda")
        Bk.latent_prep_form(rg, *args, q=q, qc=qc)
        g = Bk.GemmDesc(x=q.data_ptr(), w=uk.data_ptr(), y=qc.data_ptr(), x_dtype=Bk._dt(q), w_dtype=Bk._dt(uk), y_dtype=1, m=r, k=d, rows=n,
                        groups=H, x_row_stride=H * (d + dr), x_group_stride=d + dr, w_m_stride=d, w_k_stride=1, w_group_stride=d * r,
                        y_row_stride=H * (r + dr), y_group_stride=r + dr)
        Bk.gemm_strided(g)
        ok = tiled and r % 16 == 0 and dr % 8 == 0 and dtype == "bfloat16"
        ol = Bk.latent_attention_dealt(qc, pc.cache, pc.page_stride, pc.offs[0], 16, rg, pc.indptr, pc.pids, r, dr, m["scale"], n_split=n_split,
                                       tiles=Bk.row_tiles([n], H) if ok else None)
        o = torch.matmul(ol.cpu().double().transpose(0, 1), w[p + ".uv"].double().view(H, dv, r).transpose(1, 2)).transpose(0, 1)
        outs.append(o.reshape(n, H * dv) @ w[p + ".o"].double().T)
        at += n
    return torch.cat(outs), pc


@BOTH
@pytest.mark.parametrize("layer", [("a", 1), ("b", 2), ("odd", 0), ("wide", 1), ("borrow", 1)])
def test_latent_attention_whole_in_portions_and_dealt(dtype, layer):
    cfg = C.CONFIGS[layer[0]]()
    w = C.random_weights(cfg, 5)
    p, m = "l%d.mix" % layer[1], cfg["layers"][layer[1]]["mixer"]
    n = 150
    h = states(n, cfg["width"], 9)
    ref = R.latent_attention(h.double(), w64(w), p, m, 1e-5, R.make_latents(h.double(), w64(w), p, m, 1e-5))
    tol = dict(tol32=1e-4, tol16=6e-2)
    close(run_latent(m, w, p, h, dtype, [n])[0], ref, dtype, **tol)
    close(run_latent(m, w, p, h, dtype, [n], n_split=3)[0], ref, dtype, **tol)
    close(run_latent(m, w, p, h, dtype, PORTIONS, n_split=4)[0], ref, dtype, **tol)
    close(run_latent(m, w, p, h, dtype, [33, 32, 31, 2, 2, 50], n_split=64)[0], ref, dtype, **tol)
    if dtype == "bfloat16":
        close(run_latent(m, w, p, h, dtype, [100, 50], n_split=2, tiled=False)[0], ref, dtype, **tol)


@BOTH
def test_borrowed_latents_are_read_from_the_sources_entries(dtype):
    cfg = C.config_a()
    w = C.random_weights(cfg, 6)
    src, m = cfg["layers"][1]["mixer"], cfg["layers"][3]["mixer"]
    h1, h3 = states(70, cfg["width"], 10), states(70, cfg["width"], 11)
    _, pc = run_latent(src, w, "l1.mix", h1, dtype, [70])
    before = pc.cache.clone()
    ref = R.latent_attention(h3.double(), w64(w), "l3.mix", m, 1e-5, R.make_latents(h1.double(), w64(w), "l1.mix", src, 1e-5))
    got, _ = run_latent(m, w, "l3.mix", h3, dtype, [40, 2, 28], pc=pc, own=False, n_split=2)
    close(got, ref, dtype, tol32=1e-4, tol16=6e-2)
    assert torch.equal(torch.nan_to_num(before.float()), torch.nan_to_num(pc.cache.float()))          # nothing was written


@BOTH
@pytest.mark.parametrize("hot", [0, 31, 32, 255, 256, 300])
def test_one_far_latent_stands_out_among_hundreds(dtype, hot):
    """entries whose latent is zero but for the marked one; its score is 40 above the rest: every later query reads it alone"""
    Bk = B()
    n, H, r, dr = 420, 3, 32, 8
    pc = Paged(PAGES, [r + dr], dtype)
    rg = Bk.Ragged([n])
    dkv = torch.zeros(n, r + dr)
    dkv[:, 1] = 1.0
    dkv[hot, :2] = torch.tensor([1.0, 0.0])
    f = torch.ones(dr // 2).cuda()
    Bk.latent_prep_form(rg, pc.indptr, pc.pids, pc.cache, pc.page_stride, pc.offs[0], 16, H, 8, dr, r, 0.0, f, True, dkv=dev(dkv, dtype),
                        c_norm_w=dev(torch.ones(r), dtype))
    unit = float(C.bf16_round(torch.tensor([r ** 0.5])))       # a latent with one value of 1 has norm weight sqrt(r)
    for rows, start in ((n - hot, hot), (1, n - 1)):
        q = torch.zeros(rows, H, r + dr, device="cuda")
        q[:, :, 0] = 40.0 / unit
        rq = Bk.Ragged([rows], starts=[start])
        for split, tiles in ((1, None), (5, None), (1, Bk.row_tiles([rows], H)), (9, Bk.row_tiles([rows], H))):
            if tiles is not None and dtype == "float32":
                continue
            o = Bk.latent_attention_dealt(q, pc.cache, pc.page_stride, pc.offs[0], 16, rq, pc.indptr, pc.pids, r, dr, 1.0, n_split=split, tiles=tiles)
            assert float(o[:, :, 0].min()) > 0.98 * unit and float(o[:, :, 1].abs().max()) < 1e-3, (hot, split, tiles is not None)


# ------------------------------------------------------------------ linear attention with a constant decay
def run_decay(m, qkv, dtype, plans, slots, scan_max, dirty=5.0):
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
        x = dev(torch.cat([qkv[i][at[i]:at[i] + plans[i][k]] for i in live]), dtype)
        o = Bk.decay_attention(x, [0, H * dk, 2 * H * dk], m["decay"], state, H, dk, dv, rg, scan_max=scan_max)
        row = 0
        for i in live:
            n = plans[i][k]
            outs[i].append(o[row:row + n])
            row += n
            at[i] += n
    assert float((state[max(slots) + 1] - dirty).abs().max()) == 0.0          # a slot outside the step stays as it was
    return [torch.cat(o) for o in outs], state


def decay_ref(m, qkv):
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    n = qkv.shape[0]
    x = R.silu(qkv.double())
    q, k, v = x[:, :H * dk].view(n, H, dk), x[:, H * dk:2 * H * dk].view(n, H, dk), x[:, 2 * H * dk:].view(n, H, dv)
    y, end = torch.zeros(n, H, dv, dtype=torch.float64), []
    for h in range(H):
        S = torch.zeros(dk, dv, dtype=torch.float64)
        for t in range(n):
            S = m["decay"][h] * S + torch.outer(k[t, h], v[t, h])
            y[t, h] = S.T @ q[t, h]
        end.append(S.reshape(-1))
    return y.reshape(n, H * dv), torch.cat(end)


SIZES = [dict(heads=3, dim=12, vdim=20, decay=[0.5, 0.97, 0.999]), dict(heads=1, dim=24, vdim=16, decay=[1.0]),
         dict(heads=5, dim=7, vdim=9, decay=[0.99, 0.2, 0.75, 0.999, 1e-4]), dict(heads=2, dim=72, vdim=136, decay=[0.98, 0.6]),
         dict(heads=2, dim=128, vdim=64, decay=[0.99, 0.9]), dict(heads=1, dim=64, vdim=256, decay=[0.95])]


@BOTH
@pytest.mark.parametrize("m", SIZES, ids=lambda m: "%dx%dx%d" % (m["heads"], m["dim"], m["vdim"]))
def test_decayed_linear_attention_token_by_token_and_in_chunks(dtype, m):
    w = m["heads"] * (2 * m["dim"] + m["vdim"])
    qkv = [states(200, w, 20), states(77, w, 21), states(9, w, 22)]
    refs = [decay_ref(m, x) for x in qkv]
    for plans, scan_max in (([[200], [77], [9]], 0), ([[200], [77], [9]], 32), ([[64, 63, 65, 8], [1, 76], [2, 2, 5]], 32),
                            ([[128, 1, 1, 70], [33, 44], [3, 1, 1, 4]], 32), ([[2, 100, 98], [40, 1, 36], [9]], 1)):
        outs, state = run_decay(m, qkv, dtype, plans, [2, 0, 3], scan_max)
        for i in range(3):
            close(outs[i], refs[i][0], "float32", tol32=1e-5)              # bf16: the stored inputs are exact, everything else is fp32
            close(state[[2, 0, 3][i]], refs[i][1], "float32", tol32=1e-5)


@BOTH
@pytest.mark.parametrize("scan_max", [0, 32])
def test_an_old_write_is_kept_by_a_slow_head_and_forgotten_by_a_fast_one(dtype, scan_max):
    m = dict(heads=3, dim=8, vdim=8, decay=[0.999, 0.5, 1.0])
    H, n, hot = 3, 500, 40
    x = torch.zeros(n, 3 * 24)                                    # silu(0) = 0: a token that writes and reads nothing
    for h in range(H):
        x[:, h * 8] = 8.0                                         # every query asks for key direction 0
        x[hot, 24 + h * 8] = 8.0                                  # one token writes there
        x[hot, 48 + h * 8 + 3] = 8.0
    ref, _ = decay_ref(m, x)
    for plan in ([n], [41, 459], [40, 1, 130, 1, 1, 327]):
        out = run_decay(m, [x], dtype, [plan], [0], scan_max)[0][0].double().cpu().view(n, H, 8)
        close(out, ref.view(n, H, 8), "float32", tol32=1e-5)
        peak = float(out[hot, 2, 3])
        assert (out[:hot] == 0).all() and abs(float(out[n - 1, 2, 3]) / peak - 1.0) < 1e-5
        assert abs(float(out[n - 1, 0, 3]) / peak - 0.999 ** (n - 1 - hot)) < 1e-4 and float(out[n - 1, 1, 3]) < 1e-30
