"""Torch-tensor wrappers over include/pegainfer_kernels_blocks.h: the model-independent blocks that exist in a bf16 and a
true-fp32 instance (Dynamic-Tanh norms over an fp32 stream, activations, the strided / batched / grouped GEMM, attention
over a paged latent cache, routing; time convolutions with carried tails, grouped output norms with a depth-weighted
sum, clamp-GLU, recurrent matrix memories over per-request state, attention over a paged key/value cache).  Tensors are torch CUDA tensors used as device memory; the
storage type of a call (bf16 / fp32) is taken from the activation tensor.  Work is enqueued on torch's current stream.
No CPU fallback: without the HIP library every call raises ImportError.
"""
import ctypes

import torch

from . import ffi
from .ops import _chk, _p, _stream

EPI_NONE, EPI_RELU_SQ, EPI_SIGMOID_GATE, EPI_GELU_ERF = 0, 1, 2, 3


def _dt(t):
    if t.dtype == torch.bfloat16:
        return 0
    if t.dtype == torch.float32:
        return 1
    raise TypeError("bf16 or fp32 tensors only")


class GemmDesc(ctypes.Structure):
    _fields_ = [("x", ctypes.c_void_p), ("w", ctypes.c_void_p), ("y", ctypes.c_void_p),
                ("x_dtype", ctypes.c_int32), ("w_dtype", ctypes.c_int32), ("y_dtype", ctypes.c_int32),
                ("m", ctypes.c_int32), ("k", ctypes.c_int32), ("rows", ctypes.c_int32), ("groups", ctypes.c_int32),
                ("x_row_stride", ctypes.c_int64), ("x_group_stride", ctypes.c_int64),
                ("w_m_stride", ctypes.c_int64), ("w_k_stride", ctypes.c_int64), ("w_group_stride", ctypes.c_int64),
                ("y_row_stride", ctypes.c_int64), ("y_group_stride", ctypes.c_int64),
                ("tile_group", ctypes.c_void_p), ("tile_row0", ctypes.c_void_p), ("tile_rows", ctypes.c_void_p),
                ("n_tiles", ctypes.c_void_p), ("max_tiles", ctypes.c_int32),
                ("x_row_index", ctypes.c_void_p), ("y_row_index", ctypes.c_void_p),
                ("epilogue", ctypes.c_int32), ("gate", ctypes.c_void_p), ("gate_dtype", ctypes.c_int32),
                ("gate_row_stride", ctypes.c_int64), ("max_tile_rows", ctypes.c_int32), ("tile_rows_cap", ctypes.c_int32),
                ("plain", ctypes.c_int32)]


def embed_f32(embed, token_ids_u32):
    out = torch.empty((token_ids_u32.numel(), embed.shape[1]), dtype=torch.float32, device=embed.device)
    _chk(ffi.lib().pegainfer_embed_f32(_p(embed), _p(token_ids_u32), _p(out), embed.shape[1], token_ids_u32.numel(),
                                       _dt(embed), _stream()), "embed_f32")
    return out


def dyt_norm(x_f32, alpha, w, b):
    """out = tanh(alpha x) w + b; x fp32 [rows, d]; alpha / w / b (and the result) in the storage type of w"""
    assert x_f32.dtype == torch.float32 and x_f32.is_contiguous()
    out = torch.empty(x_f32.shape, dtype=w.dtype, device=x_f32.device)
    _chk(ffi.lib().pegainfer_dyt_norm(_p(x_f32), _p(alpha), _p(w), _p(b), _p(out), x_f32.shape[-1],
                                      x_f32.numel() // x_f32.shape[-1], _dt(w), _stream()), "dyt_norm")
    return out


def dyt_add_norm(x_f32, y, post, nxt=None):
    """x += dyt(y; post) in place; returns dyt(x; nxt) when nxt = (alpha, w, b) is given"""
    assert x_f32.dtype == torch.float32 and x_f32.is_contiguous() and y.is_contiguous()
    out = torch.empty(y.shape, dtype=y.dtype, device=y.device) if nxt else None
    n = nxt or (None, None, None)
    _chk(ffi.lib().pegainfer_dyt_add_norm(_p(x_f32), _p(y), _p(post[0]), _p(post[1]), _p(post[2]), _p(n[0]), _p(n[1]), _p(n[2]),
                                          _p(out), y.shape[-1], y.numel() // y.shape[-1], _dt(y), _stream()), "dyt_add_norm")
    return out


def relu_sq(x):
    out = torch.empty_like(x)
    _chk(ffi.lib().pegainfer_relu_sq(_p(x), _p(out), x.numel(), _dt(x), _stream()), "relu_sq")
    return out


def silu_mul_rows(gate_up):
    rows, two_i = gate_up.shape
    out = torch.empty((rows, two_i // 2), dtype=gate_up.dtype, device=gate_up.device)
    _chk(ffi.lib().pegainfer_silu_mul_rows(_p(gate_up), _p(out), two_i // 2, rows, _dt(gate_up), _stream()), "silu_mul_rows")
    return out


def gemm_strided(desc):
    _chk(ffi.lib().pegainfer_gemm_strided(ctypes.addressof(desc), _stream()), "gemm_strided")


def linear(x, w, out_dtype=None, epilogue=EPI_NONE, plain=False):
    """y[T, M] = x[T, K] w[M, K]^T through pegainfer_gemm_strided (any sizes, bf16 or fp32 operands, fp32 accumulation; x may be
    a column range of a wider matrix); plain = the fp32-FMA tile kernel whatever the shape"""
    T, K = x.shape
    M = w.shape[0]
    y = torch.empty((T, M), dtype=out_dtype or x.dtype, device=x.device)
    d = GemmDesc(x=_p(x), w=_p(w), y=_p(y), x_dtype=_dt(x), w_dtype=_dt(w), y_dtype=_dt(y), m=M, k=K, rows=T, groups=1,
                 x_row_stride=x.stride(0), w_m_stride=K, w_k_stride=1, y_row_stride=M, epilogue=epilogue, plain=int(plain))
    gemm_strided(d)
    return y


def latent_prep(proj, dkv_offset, c_norm_w, eps, inv_freq, rot_dims, positions, token_req, page_indptr, page_ids, cache,
                page_stride, layer_off, page_size, qc, heads, nope, rot, rank):
    _chk(ffi.lib().pegainfer_latent_prep(_p(proj), proj.shape[1], dkv_offset, _p(c_norm_w), float(eps), _p(inv_freq), rot_dims,
                                         _p(positions), _p(token_req), _p(page_indptr), _p(page_ids), _p(cache), page_stride,
                                         layer_off, page_size, _p(qc), heads, nope, rot, rank, proj.shape[0], _dt(proj),
                                         _stream()), "latent_prep")


def row_tiles(lens, heads, device="cuda"):
    """the flattened (token, head) rows of a step with entries of `lens` tokens, cut into runs of <= 64 rows inside one entry"""
    row0, rows, at = [], [], 0
    for n in lens:
        for r in range(0, n * heads, 64):
            row0.append(at * heads + r)
            rows.append(min(64, n * heads - r))
        at += n
    return (torch.tensor(row0, dtype=torch.int32, device=device), torch.tensor(rows, dtype=torch.int32, device=device))


def latent_attention(qc, cache, page_stride, layer_off, page_size, positions, token_req, page_indptr, page_ids, rank, rot,
                     scale, max_kv_len, split_keys=0, tiles=None):
    """qc fp32 [T, heads, rank + rot] -> o_lat fp32 [T, heads, rank]; tiles = row_tiles(...) selects the matrix-core form"""
    T, H, E = qc.shape
    assert E == rank + rot and qc.dtype == torch.float32
    o = torch.empty((T, H, rank), dtype=torch.float32, device=qc.device)
    n = ffi.lib().pegainfer_latent_attention_workspace(T, H, rank, max_kv_len, split_keys)
    ws = torch.empty(max(int(n), 1), dtype=torch.float32, device=qc.device)
    t0, tr = tiles if tiles is not None else (None, None)
    _chk(ffi.lib().pegainfer_latent_attention(_p(qc), _p(o), _p(cache), page_stride, layer_off, page_size, _p(positions),
                                              _p(token_req), _p(page_indptr), _p(page_ids), H, rank, rot, float(scale), T,
                                              max_kv_len, split_keys, _p(ws), _p(t0), _p(tr), 0 if t0 is None else t0.numel(),
                                              _dt(cache), _stream()), "latent_attention")
    return o


def route(h, w_router, correction, n_groups, keep_groups, top):
    rows, d = h.shape
    e = torch.empty((rows, top), dtype=torch.int32, device=h.device)
    w = torch.empty((rows, top), dtype=torch.float32, device=h.device)
    _chk(ffi.lib().pegainfer_route_sigmoid_grouped(_p(h), _p(w_router), _p(correction), _p(e), _p(w), d, w_router.shape[0],
                                                   n_groups, keep_groups, top, rows, _dt(h), _stream()), "route")
    return e, w


def route_sort(expert, experts, rows_per_tile=64):
    """-> pos_pair, pos_row, tile_group, tile_row0, tile_rows, n_tiles (int32 device tensors), max_tiles"""
    rows, top = expert.shape
    P = rows * top
    max_tiles = (P + rows_per_tile - 1) // rows_per_tile + experts
    dev = expert.device
    pos_pair, pos_row = torch.empty(P, dtype=torch.int32, device=dev), torch.empty(P, dtype=torch.int32, device=dev)
    tg, t0, tr = (torch.zeros(max_tiles, dtype=torch.int32, device=dev) for _ in range(3))
    nt = torch.zeros(1, dtype=torch.int32, device=dev)
    _chk(ffi.lib().pegainfer_route_sort(_p(expert), P, top, experts, _p(pos_pair), _p(pos_row), _p(tg), _p(t0), _p(tr), _p(nt),
                                        max_tiles, rows_per_tile, _stream()), "route_sort")
    return pos_pair, pos_row, tg, t0, tr, nt, max_tiles


def route_combine(y_pairs, weight, out_dtype):
    rows, top = weight.shape
    d = y_pairs.shape[1]
    out = torch.empty((rows, d), dtype=out_dtype, device=y_pairs.device)
    _chk(ffi.lib().pegainfer_route_combine(_p(y_pairs), _p(weight), _p(out), d, top, rows, _dt(out), _stream()), "route_combine")
    return out


# ---- sequences with state: ragged batches (entry e = rows entry_row0[e] .. entry_row0[e + 1] - 1, state slot entry_slot[e]) ----
class Ragged:
    """device index arrays of a step whose entries have `lens` rows and use the state slots `slots`; positions start at
    `starts` (default 0)"""

    def __init__(self, lens, slots=None, starts=None, device="cuda"):
        slots = list(range(len(lens))) if slots is None else slots
        starts = [0] * len(lens) if starts is None else starts
        row0, ent, pos = [0], [], []
        for i, n in enumerate(lens):
            row0.append(row0[-1] + n)
            ent += [i] * n
            pos += list(range(starts[i], starts[i] + n))
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
        self.lens, self.n, self.rows = list(lens), len(lens), row0[-1]
        self.entry_row0, self.entry_slot, self.row_entry, self.positions = i32(row0), i32(slots), i32(ent), i32(pos)


def time_conv(x, w, state, rg, residual=False, silu=False, out_dtype=None, channels=None, in_bias=None, out_bias=None):
    """causal per-channel convolution over time; state fp32 [slots, taps - 1, C] is read, then moved on by the step's rows.
    in_bias [C] joins every real input (and so the carried ones), out_bias [C] the sum before the activation; both in w's type"""
    C = channels or w.shape[0]
    taps = w.shape[1]
    out = torch.empty((x.shape[0], C), dtype=out_dtype or x.dtype, device=x.device)
    slot_stride = state.shape[1] * state.shape[2] if state.dim() == 3 else 0
    L = ffi.lib()
    if all(n == 1 for n in rg.lens):      # decoding: output and the moved-on tail in one launch
        _chk(L.pegainfer_time_conv_step_biased(_p(x), _dt(x), x.stride(0), _p(w), _dt(w), _p(in_bias), _p(out_bias), _p(state),
                                               slot_stride, _p(out), _dt(out), C, C, taps, (1 if residual else 0) | (2 if silu else 0),
                                               _p(rg.entry_slot), rg.n, _stream()), "time_conv_step")
        return out
    _chk(L.pegainfer_time_conv_biased(_p(x), _dt(x), x.stride(0), _p(w), _dt(w), _p(in_bias), _p(out_bias), _p(state), slot_stride,
                                      _p(out), _dt(out), C, C, taps, (1 if residual else 0) | (2 if silu else 0), _p(rg.row_entry),
                                      _p(rg.entry_row0), _p(rg.entry_slot), x.shape[0], _stream()), "time_conv")
    _chk(L.pegainfer_time_conv_commit_biased(_p(x), _dt(x), x.stride(0), _p(in_bias), _dt(w), _p(state), slot_stride, C, taps,
                                             _p(rg.entry_row0), _p(rg.entry_slot), rg.n, _stream()), "time_conv_commit")
    return out


def group_rms_add(y, w, groups, eps, x=None, stack=None, coef=None):
    """r = (x or 0) + grouped_rms(y) * w  -> (r fp32, r in w's dtype, mix fp32 or None) with
    mix = sum_j coef[j] stack[j] + coef[-1] r over the len(coef) - 1 streams of `stack` (fp32 [n, rows, d])"""
    rows, d = y.shape
    r32 = torch.empty((rows, d), dtype=torch.float32, device=y.device)
    rb = torch.empty((rows, d), dtype=w.dtype, device=y.device)
    n_mix = 0 if coef is None else coef.numel()
    mix = torch.empty((rows, d), dtype=torch.float32, device=y.device) if n_mix else None
    _chk(ffi.lib().pegainfer_group_rms_add(_p(x), _p(y), _dt(y), _p(w), groups, float(eps), _p(r32), _p(rb), d, rows, _dt(w),
                                           _p(stack), 0 if stack is None else stack.stride(0), _p(coef), n_mix, _p(mix), None,
                                           _stream()), "group_rms_add")
    return r32, rb, mix


def clamp_glu_rows(gate_up, limit, alpha=1.702):
    rows, two_i = gate_up.shape
    out = torch.empty((rows, two_i // 2), dtype=gate_up.dtype, device=gate_up.device)
    _chk(ffi.lib().pegainfer_clamp_glu_rows(_p(gate_up), _p(out), two_i // 2, rows, float(limit), float(alpha), _dt(gate_up),
                                            _stream()), "clamp_glu_rows")
    return out


def route_topk(h, w_router, top, score="softmax", correction=None, n_groups=1, keep_groups=1):
    rows, d = h.shape
    e = torch.empty((rows, top), dtype=torch.int32, device=h.device)
    w = torch.empty((rows, top), dtype=torch.float32, device=h.device)
    _chk(ffi.lib().pegainfer_route_topk(_p(h), _p(w_router), _p(correction), _p(e), _p(w), d, w_router.shape[0], n_groups,
                                        keep_groups, top, rows, 1 if score == "softmax" else 0, _dt(h), _stream()), "route_topk")
    return e, w


def route_from_logits(logits_f32, top, score="softmax", correction=None, n_groups=1, keep_groups=1, dtype=torch.bfloat16):
    rows, E = logits_f32.shape
    e = torch.empty((rows, top), dtype=torch.int32, device=logits_f32.device)
    w = torch.empty((rows, top), dtype=torch.float32, device=logits_f32.device)
    _chk(ffi.lib().pegainfer_route_from_logits(_p(logits_f32), _p(correction), _p(e), _p(w), E, n_groups, keep_groups, top, rows,
                                               1 if score == "softmax" else 0, 0 if dtype == torch.bfloat16 else 1, _stream()),
         "route_from_logits")
    return e, w


def route_combine_add(y_pairs, weight, add, out_dtype):
    rows, top = weight.shape
    d = y_pairs.shape[1]
    out = torch.empty((rows, d), dtype=out_dtype, device=y_pairs.device)
    _chk(ffi.lib().pegainfer_route_combine_add(_p(y_pairs), _p(weight), _p(add), _p(out), d, top, rows, _dt(out), _stream()),
         "route_combine_add")
    return out


def delta_rule(qkv_f32, proj, b_off, a_off, A_log, dt_bias, state, heads, kv_heads, dim, vdim, rg):
    """qkv fp32 [rows, 2 kv dim + heads vdim] (after convolution and silu), proj [rows, *] with the beta / decay inputs;
    state fp32 [slots, heads, dim, vdim] is updated in place, and so are the q / k parts of qkv (made unit vectors);
    returns o fp32 [rows, heads * vdim]"""
    o = torch.empty((qkv_f32.shape[0], heads * vdim), dtype=torch.float32, device=proj.device)
    gates = torch.empty((qkv_f32.shape[0], 2 * heads), dtype=torch.float32, device=proj.device)
    _chk(ffi.lib().pegainfer_delta_rule(_p(qkv_f32), qkv_f32.stride(0), _p(proj), proj.stride(0), b_off, a_off, _p(A_log),
                                        _p(dt_bias), _p(gates), _p(state), state.stride(0), _p(o), heads, kv_heads, dim, vdim,
                                        qkv_f32.shape[0], _p(rg.entry_row0), _p(rg.entry_slot), rg.n, _dt(proj), _stream()),
         "delta_rule")
    return o


def gated_matrix_memory(proj, offs, i_bias, f_bias, cap, state, heads, dim, vdim, rg):
    """proj [rows, *] with q / k / v / i / f at the column offsets `offs`; state fp32 [slots, heads (dim vdim + dim + 1)] laid
    out [S of all heads | n of all heads | m of all heads]; returns o fp32 [rows, heads * vdim]"""
    o = torch.empty((proj.shape[0], heads * vdim), dtype=torch.float32, device=proj.device)
    _chk(ffi.lib().pegainfer_gated_matrix_memory(_p(proj), proj.stride(0), offs[0], offs[1], offs[2], offs[3], offs[4], _p(i_bias),
                                                 _p(f_bias), float(cap), _p(state), state.stride(0), _p(o), heads, dim, vdim,
                                                 _p(rg.entry_row0), _p(rg.entry_slot), rg.n, _dt(proj), _stream()),
         "gated_matrix_memory")
    return o


def head_rms_gate(o_f32, w, gate, gate_kind, factor, eps, heads, vdim, out=None):
    """gate: a [rows, heads * vdim] view (row stride free) in w's dtype; gate_kind "silu" | "sigmoid" """
    rows = o_f32.shape[0]
    out = torch.empty((rows, heads * vdim), dtype=w.dtype, device=w.device) if out is None else out
    _chk(ffi.lib().pegainfer_head_rms_gate(_p(o_f32), _p(w), int(w.numel() != vdim),
                                           _p(gate), gate.stride(0), 0 if gate_kind == "silu" else 1, float(factor), float(eps),
                                           _p(out), out.stride(0), heads, vdim, rows, _dt(w), _stream()), "head_rms_gate")
    return out


def attention_tiles(lens, per_group, device="cuda", rows=16):
    """row tiles of pegainfer_paged_attention for entries of `lens` rows: runs of token rows times runs of the per_group query
    heads of a key/value head, at most `rows` rows each"""
    row0, ntok, qh0, nqh, at = [], [], [], [], 0
    for n in lens:
        tpt = max(1, rows // per_group)
        for t0 in range(0, n, tpt):
            for q0 in range(0, per_group, rows):
                row0.append(at + t0); ntok.append(min(tpt, n - t0)); qh0.append(q0); nqh.append(min(rows, per_group - q0))  # noqa: E702
        at += n
    return tuple(torch.tensor(v, dtype=torch.int32, device=device) for v in (row0, ntok, qh0, nqh))


def qk_norm_rope_paged(proj, offs, heads, kv_heads, dim, vdim, q_norm, k_norm, eps, inv_freq, rot_dims, rg, page_indptr,
                       page_ids, cache, page_stride, k_off, v_off, page_size):
    q = torch.empty((proj.shape[0], heads, dim), dtype=torch.float32, device=proj.device)
    _chk(ffi.lib().pegainfer_qk_norm_rope_paged(_p(proj), proj.stride(0), offs[0], offs[1], offs[2], heads, kv_heads, dim, vdim,
                                                _p(q_norm), _p(k_norm), float(eps), _p(inv_freq), rot_dims, _p(rg.positions),
                                                _p(rg.row_entry), _p(page_indptr), _p(page_ids), _p(cache), page_stride, k_off,
                                                v_off, page_size, _p(q), None, proj.shape[0], _dt(proj), _stream()), "qk_norm_rope_paged")
    return q


def paged_attention(q, cache, page_stride, k_off, v_off, page_size, rg, page_indptr, page_ids, kv_heads, vdim, scale, factor=1.0):
    T, H, dim = q.shape
    out = torch.empty((T, H * vdim), dtype=cache.dtype, device=q.device)
    t = attention_tiles(rg.lens, H // kv_heads, q.device)
    _chk(ffi.lib().pegainfer_paged_attention(_p(q), _p(cache), page_stride, k_off, v_off, page_size, _p(rg.positions),
                                             _p(rg.row_entry), _p(page_indptr), _p(page_ids), H, kv_heads, dim, vdim,
                                             float(scale), float(factor), _p(t[0]), _p(t[1]), _p(t[2]), _p(t[3]), t[0].numel(),
                                             _p(out), out.stride(0), _dt(cache), _stream()), "paged_attention")
    return out


# ---- one-number RMS gains, attention with options, channel decays, group-limited routing ----
def scalar_rms_add(x, gain, eps, y=None, bias=None, mult=1.0, add_rows=None, add_vec=None, norm=True):
    """r = x + mult (y + bias) + add_rows + add_vec (fp32), n = r / rms(r) * gain[0] (fp32) -> (r, n or None);
    x fp32 [rows, d]; y / bias / add_vec / gain in the storage type of gain"""
    rows, d = x.shape
    r = torch.empty_like(x)
    n = torch.empty_like(x) if norm else None
    _chk(ffi.lib().pegainfer_scalar_rms_add(_p(x), _p(y), _dt(y) if y is not None else _dt(gain), _p(bias), float(mult), _p(add_rows),
                                            _p(add_vec), _p(r), _p(gain) if norm else None, float(eps), _p(n), d, rows, _dt(gain),
                                            _stream()), "scalar_rms_add")
    return r, n


def qk_prep_paged(proj, offs, heads, kv_heads, dim, vdim, rg, page_indptr, page_ids, cache, page_stride, k_off, v_off, page_size,
                  q_norm=None, k_norm=None, eps=0.0, q_bias=None, k_bias=None, v_bias=None, qt_coef=0.0, qt_every=0, inv_freq=None,
                  rot_dims=0):
    """queries -> fp32 [rows, heads, dim]; keys and values -> the cache entry of (request, position).  dim counts ALL values of
    a query / key head (both maps of a two-map attention)"""
    q = torch.empty((proj.shape[0], heads, dim), dtype=torch.float32, device=proj.device)
    _chk(ffi.lib().pegainfer_qk_prep_paged(_p(proj), proj.stride(0), offs[0], offs[1], offs[2], heads, kv_heads, dim, vdim, _p(q_norm),
                                           _p(k_norm), float(eps), _p(q_bias), _p(k_bias), _p(v_bias), float(qt_coef), int(qt_every),
                                           _p(inv_freq), rot_dims, _p(rg.positions), _p(rg.row_entry), _p(page_indptr), _p(page_ids),
                                           _p(cache), page_stride, k_off, v_off, page_size, _p(q), None, proj.shape[0], _dt(proj),
                                           _stream()), "qk_prep_paged")
    return q


def paged_attention_ex(q, cache, page_stride, k_off, v_off, page_size, rg, page_indptr, page_ids, kv_heads, vdim, scale, factor=1.0,
                       maps=1, lam=0.0, block=0, sink=None, head_norm=False, norm_eps=0.0, n_split=1, plain=False):
    """q fp32 [rows, heads, maps * dim]; n_split > 1: the keys of every tile dealt to that many workgroups, then merged; a bf16 cache runs on
    the matrix cores unless plain"""
    T, H, qd = q.shape
    out = torch.empty((T, H * vdim), dtype=cache.dtype, device=q.device)
    t = attention_tiles(rg.lens, H // kv_heads, q.device)
    ws = None
    if n_split > 1:
        ws = torch.empty(ffi.lib().pegainfer_paged_attention_workspace(t[0].numel(), kv_heads, vdim, maps, n_split),
                         dtype=torch.float32, device=q.device)
    _chk(ffi.lib().pegainfer_paged_attention_ex(_p(q), _p(cache), page_stride, k_off, v_off, page_size, _p(rg.positions),
                                                _p(rg.row_entry), _p(page_indptr), _p(page_ids), H, kv_heads, qd // maps, vdim,
                                                float(scale), float(factor), _p(t[0]), _p(t[1]), _p(t[2]), _p(t[3]), t[0].numel(),
                                                _p(out), out.stride(0), maps, float(lam), int(block), _p(sink), int(bool(head_norm)),
                                                float(norm_eps), int(n_split), _p(ws), int(bool(plain)), _dt(cache), _stream()), "paged_attention_ex")
    return out


def delta_rule_channel(qkv_f32, proj, b_off, a_f32, A_log, dt_bias, state, heads, kv_heads, dim, vdim, rg):
    """the gated delta rule with a decay per (head, key channel); a_f32 [rows, heads * dim] the decay inputs; otherwise as
    delta_rule"""
    o = torch.empty((qkv_f32.shape[0], heads * vdim), dtype=torch.float32, device=proj.device)
    gates = torch.empty((qkv_f32.shape[0], heads * dim + heads), dtype=torch.float32, device=proj.device)
    _chk(ffi.lib().pegainfer_delta_rule_channel(_p(qkv_f32), qkv_f32.stride(0), _p(proj), proj.stride(0), b_off, _p(a_f32),
                                                a_f32.stride(0), _p(A_log), _p(dt_bias), _p(gates), _p(state), state.stride(0), _p(o),
                                                heads, kv_heads, dim, vdim, qkv_f32.shape[0], _p(rg.entry_row0), _p(rg.entry_slot),
                                                rg.n, _dt(proj), _stream()), "delta_rule_channel")
    return o


def route_from_logits_ex(logits_f32, experts, top, n_groups=1, keep_groups=1, score="softmax", group="max", renorm=True,
                         dtype=torch.bfloat16):
    """logits fp32 [rows, >= experts] (columns beyond `experts` are not read)"""
    rows = logits_f32.shape[0]
    e = torch.empty((rows, top), dtype=torch.int32, device=logits_f32.device)
    w = torch.empty((rows, top), dtype=torch.float32, device=logits_f32.device)
    _chk(ffi.lib().pegainfer_route_from_logits_ex(_p(logits_f32), logits_f32.stride(0), None, _p(e), _p(w), experts, n_groups,
                                                  keep_groups, top, rows, 1 if score == "softmax" else 0, 1 if group == "max" else 0,
                                                  int(bool(renorm)), 0 if dtype == torch.bfloat16 else 1, _stream()),
         "route_from_logits_ex")
    return e, w


def route_combine_gated(y_pairs, weight, add, add_gate_f32, out_dtype):
    """sum_c weight[row, c] y_pairs[row * top + c] + sigmoid(add_gate[row]) * add[row]; add_gate: an fp32 [rows] view (stride free)"""
    rows, top = weight.shape
    d = y_pairs.shape[1]
    out = torch.empty((rows, d), dtype=out_dtype, device=y_pairs.device)
    _chk(ffi.lib().pegainfer_route_combine_gated(_p(y_pairs), _p(weight), _p(add), _p(add_gate_f32),
                                                 0 if add_gate_f32 is None else add_gate_f32.stride(0), _p(out), d, top, rows,
                                                 _dt(out), _stream()), "route_combine_gated")
    return out


# ---- several sublayers behind one norm, attention with shaped scores and gates, state-space scan ----
class SumTerm(ctypes.Structure):
    _fields_ = [("y", ctypes.c_void_p), ("y_row_stride", ctypes.c_int64), ("bias", ctypes.c_void_p), ("norm_w", ctypes.c_void_p),
                ("factor", ctypes.c_float)]


def terms_rms_add(x, terms, gain=None, eps=1e-6, out_dtype=None):
    """r = x + sum_t factor_t * (norm_w_t ? rms_norm(y_t + bias_t) * norm_w_t : y_t + bias_t);  n = rms_norm(r) * gain.
    x fp32 [rows, d] or None; terms: up to three (y, bias or None, norm_w or None, factor); -> (r fp32, n in out_dtype or None)"""
    ref = terms[0][0] if terms else gain
    rows, d = (x.shape if x is not None else terms[0][0].shape)
    arr = (SumTerm * max(1, len(terms)))()
    for i, (y, bias, nw, f) in enumerate(terms):
        arr[i] = SumTerm(_p(y), y.stride(0), _p(bias), _p(nw), float(f))
    r = torch.empty((rows, d), dtype=torch.float32, device=ref.device)
    n = torch.empty((rows, d), dtype=out_dtype or ref.dtype, device=ref.device) if gain is not None else None
    _chk(ffi.lib().pegainfer_terms_rms_add(_p(x), ctypes.addressof(arr) if terms else None, len(terms), _p(r), _p(gain), float(eps), _p(n),
                                           _dt(n) if n is not None else 0, d, rows, _dt(ref), _stream()), "terms_rms_add")
    return r, n


ACTS = {"silu": 0, "relu": 1, "gelu_tanh": 2, "gelu_erf": 3}


def glu_rows(gate, up, act="relu"):
    """act(gate) * up; gate and up are [rows, I] views of rows with one stride (column ranges of a wider matrix)"""
    rows, I = gate.shape
    assert gate.stride(0) == up.stride(0)
    out = torch.empty((rows, I), dtype=gate.dtype, device=gate.device)
    _chk(ffi.lib().pegainfer_glu_rows(_p(gate), _p(up), gate.stride(0), _p(out), I, I, rows, ACTS[act],
                                      _dt(gate), _stream()), "glu_rows")
    return out


def softcap_rows(x_f32, cap):
    out = torch.empty_like(x_f32)
    _chk(ffi.lib().pegainfer_softcap_rows(_p(x_f32), _p(out), x_f32.numel(), float(cap), _stream()), "softcap_rows")
    return out


def head_gate_rms(o_f32, w, gate, gate_kind, eps, heads, vdim, gate_first=True, factor=1.0):
    """head_rms_gate with the order chosen: gate_first norms the gated values"""
    rows = o_f32.shape[0]
    out = torch.empty((rows, heads * vdim), dtype=w.dtype, device=w.device)
    _chk(ffi.lib().pegainfer_head_gate_rms(_p(o_f32), _p(w), int(w.numel() != vdim), _p(gate), gate.stride(0),
                                           0 if gate_kind == "silu" else 1, int(bool(gate_first)), float(factor), float(eps), _p(out),
                                           out.stride(0), heads, vdim, rows, _dt(w), _stream()), "head_gate_rms")
    return out


QKNORM = {"head_weight": 0, "head_unit_after": 1, "all_weight": 2}


def qk_prep_paged_form(proj, offs, heads, kv_heads, dim, vdim, rg, page_indptr, page_ids, cache, page_stride, k_off, v_off, page_size,
                       q_norm=None, k_norm=None, norm_kind="head_weight", eps=0.0, q_bias=None, k_bias=None, v_bias=None, inv_freq=None,
                       rot_dims=0, halves=False):
    """proj: rows of the cache's type or fp32 (what a convolution left); queries -> fp32 [rows, heads, dim]; keys and values -> the
    cache entry of (request, position)"""
    q = torch.empty((proj.shape[0], heads, dim), dtype=torch.float32, device=proj.device)
    _chk(ffi.lib().pegainfer_qk_prep_paged_form(_p(proj), _dt(proj), proj.stride(0), offs[0], offs[1], offs[2], heads, kv_heads, dim, vdim,
                                                _p(q_norm), _p(k_norm), QKNORM[norm_kind], float(eps), _p(q_bias), _p(k_bias), _p(v_bias),
                                                0.0, 0, _p(inv_freq), rot_dims, int(bool(halves)), _p(rg.positions), _p(rg.row_entry),
                                                _p(page_indptr), _p(page_ids), _p(cache), page_stride, k_off, v_off, page_size, _p(q), None,
                                                proj.shape[0], _dt(cache), _stream()), "qk_prep_paged_form")
    return q


def paged_attention_masked(q, cache, page_stride, k_off, v_off, page_size, rg, page_indptr, page_ids, kv_heads, vdim, scale, softcap=0.0,
                           window=0, keep_first=0, dist_bias=None, gate=None, gate_per_head=False, block=0, sink=None, n_split=1,
                           plain=False):
    """q fp32 [rows, heads, dim]; dist_bias fp32 [n_dist, heads]; gate: a view of rows in the cache's type ([rows, heads * vdim] or
    [rows, heads])"""
    T, H, dim = q.shape
    out = torch.empty((T, H * vdim), dtype=cache.dtype, device=q.device)
    t = attention_tiles(rg.lens, H // kv_heads, q.device)
    ws = None
    if n_split > 1:
        ws = torch.empty(ffi.lib().pegainfer_paged_attention_workspace(t[0].numel(), kv_heads, vdim, 1, n_split), dtype=torch.float32,
                         device=q.device)
    _chk(ffi.lib().pegainfer_paged_attention_masked(_p(q), _p(cache), page_stride, k_off, v_off, page_size, _p(rg.positions),
                                                    _p(rg.row_entry), _p(page_indptr), _p(page_ids), H, kv_heads, dim, vdim, float(scale),
                                                    1.0, _p(t[0]), _p(t[1]), _p(t[2]), _p(t[3]), t[0].numel(), _p(out), out.stride(0), 1,
                                                    0.0, int(block), _p(sink), 0, 0.0, float(softcap), int(window), int(keep_first),
                                                    _p(dist_bias), 0 if dist_bias is None else dist_bias.shape[0], _p(gate),
                                                    0 if gate is None else gate.stride(0),
                                                    0 if gate is None else (2 if gate_per_head else 1), int(n_split), _p(ws),
                                                    int(bool(plain)), _dt(cache), _stream()), "paged_attention_masked")
    return out


def ssd_scan(xbc_f32, proj, dt_off, A_log, dt_bias, D, state, heads, groups, n_state, vdim, rg):
    """selective state-space scan; xbc fp32 [rows, heads * vdim + 2 * groups * n_state]; proj rows (storage type) hold the raw step
    sizes at dt_off; state fp32 [slots, heads * n_state * vdim] is read and moved on; -> y fp32 [rows, heads * vdim]"""
    y = torch.empty((xbc_f32.shape[0], heads * vdim), dtype=torch.float32, device=proj.device)
    _chk(ffi.lib().pegainfer_ssd_scan(_p(xbc_f32), xbc_f32.stride(0), _p(proj), proj.stride(0), dt_off, _p(A_log), _p(dt_bias), _p(D),
                                      _p(state), state.stride(0), _p(y), heads, groups, n_state, vdim, _p(rg.entry_row0), _p(rg.entry_slot),
                                      rg.n, _dt(proj), _stream()), "ssd_scan")
    return y


# ---- several residual streams, latent attention with a query latent, a linear distance bias, constant decays ----
def _struct(name, fields):
    kinds = {"p": ctypes.c_void_p, "i": ctypes.c_int32, "l": ctypes.c_int64, "f": ctypes.c_float}
    return type(name, (ctypes.Structure,), {"_fields_": [(n, kinds[k]) for k, ns in fields for n in ns.split()]})


AttnOptions = _struct("AttnOptions", [("i", "maps"), ("f", "lambda_"), ("i", "block"), ("p", "sink"), ("i", "head_norm"), ("f", "norm_eps softcap"),
                                      ("i", "window keep_first"), ("p", "dist_bias"), ("i", "n_dist"), ("p", "dist_slope gate"),
                                      ("l", "gate_stride"), ("i", "gate_kind n_split"), ("p", "workspace"), ("i", "plain shared_tail tile_rows")])
LatentPrepDesc = _struct("LatentPrepDesc", [("p", "dkv"), ("l", "dkv_stride"), ("p", "c_norm_w ql"), ("l", "ql_stride"), ("p", "ql_norm_w ql_out"),
                                            ("i", "q_rank"), ("p", "q"), ("l", "q_stride"), ("p", "qc"), ("f", "eps"), ("p", "inv_freq"),
                                            ("i", "rot_dims rot_layout"), ("p", "positions token_req page_indptr page_ids cache"),
                                            ("l", "page_stride layer_off"), ("i", "page_size heads nope rot rank n_tokens dtype")])
StreamMixDesc = _struct("StreamMixDesc", [("p", "x_in embed token_ids"), ("f", "embed_scale"), ("p", "row_index y"), ("l", "y_row_stride"),
                                          ("p", "mix out_w"), ("f", "mult"), ("p", "x_out sum_out read_w gain n_out"), ("f", "eps"),
                                          ("i", "norm_kind streams d rows dtype")])
DecayAttentionDesc = _struct("DecayAttentionDesc", [("p", "proj"), ("l", "proj_stride q_off k_off v_off"), ("i", "silu"), ("p", "decay_pow"),
                                                    ("i", "pow_n"), ("p", "state"), ("l", "slot_stride"), ("p", "o"), ("i", "heads dim vdim"),
                                                    ("p", "entry_row0 entry_slot"), ("i", "n_entries scan_max"), ("p", "chunk_row0 chunk_rows"),
                                                    ("i", "n_chunks"), ("p", "long_chunk0 long_slot"), ("i", "n_long"), ("p", "workspace"),
                                                    ("i", "dtype")])


def paged_attention_opt(q, cache, page_stride, k_off, v_off, page_size, rg, page_indptr, page_ids, kv_heads, vdim, scale, window=0,
                        dist_slope=None, softcap=0.0, n_split=1, plain=False, sink=None, gate=None, factor=1.0, shared_tail=0, tile_rows=16):
    """q fp32 [rows, heads, dim]; dist_slope fp32 [heads]: slope * distance is taken off the scores; gate: a [rows, heads] view in the
    cache's type, one output gate logit per head; shared_tail: values of a key that are read from its value"""
    T, H, dim = q.shape
    out = torch.empty((T, H * vdim), dtype=cache.dtype, device=q.device)
    t = attention_tiles(rg.lens, H // kv_heads, q.device, tile_rows)
    ws = None
    if n_split > 1:
        ws = torch.empty(ffi.lib().pegainfer_paged_attention_workspace(t[0].numel(), kv_heads, vdim, 1, n_split), dtype=torch.float32,
                         device=q.device)
    o = AttnOptions(window=int(window), dist_slope=_p(dist_slope), softcap=float(softcap), n_split=int(n_split), workspace=_p(ws),
                    plain=int(bool(plain)), sink=_p(sink), gate=_p(gate), gate_stride=0 if gate is None else gate.stride(0),
                    gate_kind=0 if gate is None else 2, shared_tail=int(shared_tail), tile_rows=tile_rows if tile_rows > 16 else 0)
    _chk(ffi.lib().pegainfer_paged_attention_opt(_p(q), _p(cache), page_stride, k_off, v_off, page_size, _p(rg.positions), _p(rg.row_entry),
                                                 _p(page_indptr), _p(page_ids), H, kv_heads, dim, vdim, float(scale), float(factor), _p(t[0]),
                                                 _p(t[1]), _p(t[2]), _p(t[3]), t[0].numel(), _p(out), out.stride(0), ctypes.addressof(o), _dt(cache),
                                                 _stream()), "paged_attention_opt")
    return out


def latent_prep_form(rg, page_indptr, page_ids, cache, page_stride, layer_off, page_size, heads, nope, rot, rank, eps, inv_freq, pairs,
                     dkv=None, c_norm_w=None, ql=None, ql_norm_w=None, q=None, qc=None):
    """dkv [rows, rank + rot] -> cache; ql [rows, q_rank] -> returned normed; q [rows, heads * (nope + rot)] -> qc[:, :, rank:]"""
    T = rg.positions.numel()
    out = torch.empty((T, ql.shape[1]), dtype=cache.dtype, device=cache.device) if ql is not None else None
    d = LatentPrepDesc(eps=float(eps), inv_freq=_p(inv_freq), rot_dims=rot, rot_layout=0 if pairs else 1, positions=_p(rg.positions),
                       token_req=_p(rg.row_entry), page_indptr=_p(page_indptr), page_ids=_p(page_ids), cache=_p(cache),
                       page_stride=page_stride, layer_off=layer_off, page_size=page_size, heads=heads, nope=nope, rot=rot, rank=rank,
                       n_tokens=T, dtype=_dt(cache))
    if dkv is not None:
        d.dkv, d.dkv_stride, d.c_norm_w = _p(dkv), dkv.stride(0), _p(c_norm_w)
    if ql is not None:
        d.ql, d.ql_stride, d.ql_norm_w, d.ql_out, d.q_rank = _p(ql), ql.stride(0), _p(ql_norm_w), _p(out), ql.shape[1]
    if q is not None:
        d.q, d.q_stride, d.qc = _p(q), q.stride(0), _p(qc)
    _chk(ffi.lib().pegainfer_latent_prep_form(ctypes.addressof(d), _stream()), "latent_prep_form")
    return out


def latent_attention_dealt(qc, cache, page_stride, layer_off, page_size, rg, page_indptr, page_ids, rank, rot, scale, n_split=1, tiles=None):
    """qc fp32 [T, heads, rank + rot] -> o_lat fp32 [T, heads, rank]; the keys dealt to n_split workgroups per row (tile)"""
    T, H, _ = qc.shape
    o = torch.empty((T, H, rank), dtype=torch.float32, device=qc.device)
    ws = torch.empty(max(1, int(ffi.lib().pegainfer_latent_attention_dealt_workspace(T, H, rank, n_split))), dtype=torch.float32, device=qc.device)
    t0, tr = tiles if tiles is not None else (None, None)
    _chk(ffi.lib().pegainfer_latent_attention_dealt(_p(qc), _p(o), _p(cache), page_stride, layer_off, page_size, _p(rg.positions),
                                                    _p(rg.row_entry), _p(page_indptr), _p(page_ids), H, rank, rot, float(scale), T, n_split,
                                                    _p(ws), _p(t0), _p(tr), 0 if t0 is None else t0.numel(), _dt(cache), _stream()),
         "latent_attention_dealt")
    return o


def stream_mix(x, streams, d, dtype, y=None, mix=None, out_w=None, mult=1.0, read_w=None, gain=None, eps=1e-5, layer_norm=True, embed=None,
               token_ids=None, embed_scale=1.0, row_index=None, want_sum=False, keep=True):
    """x fp32 [rows, streams, d] or None (then embed[token_ids] * embed_scale) -> (new streams or None, normed row or None, sum or None)"""
    rows = row_index.numel() if row_index is not None else (token_ids.numel() if x is None else x.shape[0])
    new = torch.empty((rows, streams, d), dtype=torch.float32, device="cuda") if keep else None
    n = torch.empty((rows, d), dtype=dtype, device="cuda") if gain is not None else None
    sm = torch.empty((rows, d), dtype=torch.float32, device="cuda") if want_sum else None
    q = StreamMixDesc(x_in=_p(x), embed=_p(embed), token_ids=_p(token_ids), embed_scale=float(embed_scale), row_index=_p(row_index), y=_p(y),
                      y_row_stride=y.stride(0) if y is not None else 0, mix=_p(mix), out_w=_p(out_w), mult=float(mult), x_out=_p(new),
                      sum_out=_p(sm), read_w=_p(read_w), gain=_p(gain), n_out=_p(n), eps=float(eps), norm_kind=int(bool(layer_norm)),
                      streams=streams, d=d, rows=rows, dtype=0 if dtype == torch.bfloat16 else 1)
    _chk(ffi.lib().pegainfer_stream_mix(ctypes.addressof(q), _stream()), "stream_mix")
    return new, n, sm


def _chunk_tables(d, rg, scan_max, workspace, heads, dim, vdim, chunk=64):
    """the chunk tables of a step's entries of more than scan_max rows, put into the descriptor d; returns the tensors behind them"""
    row0, rows, first, slot, at = [], [], [0], [], 0
    slots = rg.entry_slot.tolist()
    for i, n in enumerate(rg.lens if scan_max > 0 else []):
        if n > scan_max:
            for k in range(0, n, chunk):
                row0.append(at + k)
                rows.append(min(chunk, n - k))
            first.append(len(row0))
            slot.append(slots[i])
        at += n
    if not slot:
        return []
    dev = rg.entry_slot.device
    keep = [torch.tensor(v, dtype=torch.int32, device=dev) for v in (row0, rows, first, slot)]
    keep.append(torch.full((int(workspace(len(row0), heads, dim, vdim)),), float("nan"), dtype=torch.float32, device=dev))
    d.scan_max, d.chunk_row0, d.chunk_rows, d.n_chunks = scan_max, _p(keep[0]), _p(keep[1]), len(row0)
    d.long_chunk0, d.long_slot, d.n_long, d.workspace = _p(keep[2]), _p(keep[3]), len(slot), _p(keep[4])
    return keep


def decay_attention(proj, offs, decay, state, heads, dim, vdim, rg, silu=True, scan_max=0):
    """proj rows [.. q at offs[0] | k at offs[1] | v at offs[2] ..]; decay: one number per head; state fp32 [slots, heads * dim * vdim];
    scan_max > 0: entries of more rows take the chunk form -> fp32 [rows, heads * vdim]"""
    C = 64
    pw = torch.tensor([[float(g) ** n for n in range(C + 1)] for g in decay], dtype=torch.float32, device=proj.device)
    o = torch.empty((proj.shape[0], heads * vdim), dtype=torch.float32, device=proj.device)
    d = DecayAttentionDesc(proj=_p(proj), proj_stride=proj.stride(0), q_off=offs[0], k_off=offs[1], v_off=offs[2], silu=int(bool(silu)),
                           decay_pow=_p(pw), pow_n=C + 1, state=_p(state), slot_stride=state.stride(0), o=_p(o), heads=heads, dim=dim,
                           vdim=vdim, entry_row0=_p(rg.entry_row0), entry_slot=_p(rg.entry_slot), n_entries=len(rg.lens), dtype=_dt(proj))
    keep = _chunk_tables(d, rg, scan_max, ffi.lib().pegainfer_decay_attention_workspace, heads, dim, vdim)  # noqa: F841 (alive until enqueued)
    _chk(ffi.lib().pegainfer_decay_attention(ctypes.addressof(d), _stream()), "decay_attention")
    return o


# ---- norms with offset gains, rows of token pairs, identity experts, values that are keys, gated linear attention ----
TermsRmsDesc = _struct("TermsRmsDesc", [("p", "x_in row_index embed token_ids"), ("f", "embed_scale"), ("p", "pair_table prev_ids"),
                                        ("l", "mul_prev mul_cur buckets"), ("p", "terms"), ("i", "n_terms"), ("p", "x_out gain"),
                                        ("f", "eps gain_offset"), ("p", "n_out"), ("i", "n_dtype d rows dtype")])
RoutePlanDesc = _struct("RoutePlanDesc", [("p", "logits"), ("l", "logits_stride"), ("p", "correction out_expert out_weight"),
                                          ("i", "experts n_groups keep_groups top rows score_kind group_kind renorm"), ("f", "factor"),
                                          ("i", "sort_experts"), ("p", "pos_pair pos_row tile_group tile_row0 tile_rows n_tiles"),
                                          ("i", "max_tiles rows_per_tile dtype")])
QkPrepDesc = _struct("QkPrepDesc", [("p", "proj"), ("i", "proj_dtype"), ("l", "proj_stride q_off k_off v_off"), ("i", "heads kv_heads dim vdim"),
                                    ("p", "q_norm k_norm"), ("i", "norm_kind"), ("f", "eps"), ("p", "q_bias k_bias v_bias"), ("f", "qt_coef"),
                                    ("i", "qt_every"), ("p", "inv_freq"), ("i", "rot_dims rot_layout"), ("f", "rot_amp"),
                                    ("p", "positions row_entry page_indptr page_ids cache"), ("l", "page_stride k_cache_off v_cache_off"),
                                    ("i", "page_size shared_tail"), ("p", "q_out q_out_stored"), ("i", "n_rows dtype")])
GatedLinearDesc = _struct("GatedLinearDesc", [("p", "proj"), ("l", "proj_stride q_off k_off v_off"), ("f", "q_scale"), ("p", "z"), ("l", "z_stride"),
                                              ("p", "z_bias"), ("f", "tau"), ("p", "w_up"), ("l", "low_off"), ("i", "rank rank_stride"), ("p", "state"),
                                              ("l", "slot_stride"), ("p", "o"), ("i", "heads dim vdim"), ("p", "entry_row0 entry_slot"), ("i", "n_entries scan_max"),
                                              ("p", "chunk_row0 chunk_rows"), ("i", "n_chunks"), ("p", "long_chunk0 long_slot"), ("i", "n_long"),
                                              ("p", "workspace"), ("i", "dtype")])


def terms_rms(dtype, d, x=None, row_index=None, embed=None, token_ids=None, embed_scale=1.0, pair_table=None, prev_ids=None, muls=(0, 0),
              terms=(), gain=None, eps=1e-5, gain_offset=0.0, out_dtype=None):
    """terms_rms_add with its options: gain_offset, x rows picked by row_index, or the stream started from embedding rows (and the rows of
    pair_table [buckets + 1, d]) -> (stream fp32, normed row or None)"""
    rows = row_index.numel() if row_index is not None else token_ids.numel() if x is None else x.shape[0]
    arr = (SumTerm * max(1, len(terms)))()
    for i, (y, bias, nw, f) in enumerate(terms):
        arr[i] = SumTerm(_p(y), y.stride(0), _p(bias), _p(nw), float(f))
    r = torch.empty((rows, d), dtype=torch.float32, device="cuda")
    n = torch.empty((rows, d), dtype=out_dtype or dtype, device="cuda") if gain is not None else None
    q = TermsRmsDesc(x_in=_p(x), row_index=_p(row_index), embed=_p(embed), token_ids=_p(token_ids), embed_scale=float(embed_scale),
                     pair_table=_p(pair_table), prev_ids=_p(prev_ids), mul_prev=int(muls[0]), mul_cur=int(muls[1]),
                     buckets=0 if pair_table is None else pair_table.shape[0] - 1, terms=ctypes.addressof(arr) if terms else None,
                     n_terms=len(terms), x_out=_p(r), gain=_p(gain), eps=float(eps), gain_offset=float(gain_offset), n_out=_p(n),
                     n_dtype=_dt(n) if n is not None else 0, d=d, rows=rows, dtype=0 if dtype == torch.bfloat16 else 1)
    _chk(ffi.lib().pegainfer_terms_rms(ctypes.addressof(q), _stream()), "terms_rms")
    return r, n


JoinRmsDesc = _struct("JoinRmsDesc", [("p", "x y"), ("l", "y_row_stride"), ("p", "y_pairs weight expert"), ("i", "top same_from"), ("p", "same"),
                                      ("l", "same_stride"), ("p", "add add_gate"), ("l", "add_gate_stride"), ("p", "post gain"),
                                      ("f", "eps gain_offset"), ("p", "n_out"), ("i", "d rows dtype")])


def join_rms(x_f32, post, gain=None, eps=1e-5, gain_offset=0.0, y=None, y_pairs=None, weight=None, expert=None, same_from=0, same=None, add=None,
             add_gate_f32=None):
    """x (in place) += rms_norm(y) * (gain_offset + post); -> rms_norm(x) * (gain_offset + gain) or None.  y: rows of the weights' type, or the
    weighted sum of routed experts from y_pairs fp32 [rows * top, d]"""
    rows, d = x_f32.shape
    n = torch.empty((rows, d), dtype=post.dtype, device=post.device) if gain is not None else None
    q = JoinRmsDesc(x=_p(x_f32), y=_p(y), y_row_stride=0 if y is None else y.stride(0), y_pairs=_p(y_pairs), weight=_p(weight), expert=_p(expert),
                    top=0 if weight is None else weight.shape[1], same_from=same_from, same=_p(same), same_stride=0 if same is None else same.stride(0),
                    add=_p(add), add_gate=_p(add_gate_f32), add_gate_stride=0 if add_gate_f32 is None else add_gate_f32.stride(0), post=_p(post),
                    gain=_p(gain), eps=float(eps), gain_offset=float(gain_offset), n_out=_p(n), d=d, rows=rows, dtype=_dt(post))
    _chk(ffi.lib().pegainfer_join_rms(ctypes.addressof(q), _stream()), "join_rms")
    return n


def act_rows(x, act):
    """x: a [rows, I] view of rows with one stride"""
    out = torch.empty(x.shape, dtype=x.dtype, device=x.device)
    _chk(ffi.lib().pegainfer_act_rows(_p(x), x.stride(0), _p(out), out.stride(0), x.shape[1], x.shape[0], ACTS[act], _dt(x), _stream()), "act_rows")
    return out


def route_plan(logits_f32, experts, top, sort_experts, correction=None, score="softmax", renorm=True, factor=1.0, rows_per_tile=64,
               dtype=torch.bfloat16):
    """selection and sort -> (expert [rows, top], weight, dict of the sort's arrays)"""
    rows, dev = logits_f32.shape[0], logits_f32.device
    P = rows * top
    max_tiles = (P + rows_per_tile - 1) // rows_per_tile + sort_experts
    i32 = lambda *n: torch.full(n, -7, dtype=torch.int32, device=dev)  # noqa: E731
    e, w = i32(rows, top), torch.empty((rows, top), dtype=torch.float32, device=dev)
    s = {"pos_pair": i32(P), "pos_row": i32(P), "tile_group": i32(max_tiles), "tile_row0": i32(max_tiles), "tile_rows": i32(max_tiles), "n_tiles": i32(1)}
    q = RoutePlanDesc(logits=_p(logits_f32), logits_stride=logits_f32.stride(0), correction=_p(correction), out_expert=_p(e), out_weight=_p(w),
                      experts=experts, n_groups=1, keep_groups=1, top=top, rows=rows, score_kind=1 if score == "softmax" else 0,
                      renorm=int(bool(renorm)), factor=float(factor), sort_experts=sort_experts, max_tiles=max_tiles,
                      rows_per_tile=rows_per_tile, dtype=0 if dtype == torch.bfloat16 else 1, **{k: _p(v) for k, v in s.items()})
    _chk(ffi.lib().pegainfer_route_plan(ctypes.addressof(q), _stream()), "route_plan")
    s["max_tiles"] = max_tiles
    return e, w, s


def route_combine_same(y_pairs, weight, expert, same_from, same, add=None, add_gate_f32=None):
    """pairs of expert numbers >= same_from take their row of `same`"""
    rows, top = weight.shape
    d = same.shape[1]
    out = torch.empty((rows, d), dtype=same.dtype, device=same.device)
    _chk(ffi.lib().pegainfer_route_combine_same(_p(y_pairs), _p(weight), _p(expert), same_from, _p(same), same.stride(0), _p(add),
                                                _p(add_gate_f32), 0 if add_gate_f32 is None else add_gate_f32.stride(0), _p(out), d, top, rows,
                                                _dt(out), _stream()), "route_combine_same")
    return out


def qk_prep(proj, offs, heads, kv_heads, dim, vdim, rg, page_indptr, page_ids, cache, page_stride, k_off, v_off, page_size, inv_freq=None,
            rot_dims=0, halves=True, rot_amp=1.0, shared_tail=0):
    """queries -> fp32 [rows, heads, dim]; keys (without their last shared_tail values) and values -> the cache"""
    q = torch.empty((proj.shape[0], heads, dim), dtype=torch.float32, device=proj.device)
    p = QkPrepDesc(proj=_p(proj), proj_dtype=_dt(proj), proj_stride=proj.stride(0), q_off=offs[0], k_off=offs[1], v_off=offs[2], heads=heads,
                   kv_heads=kv_heads, dim=dim, vdim=vdim, inv_freq=_p(inv_freq), rot_dims=rot_dims, rot_layout=int(bool(halves)),
                   rot_amp=float(rot_amp), positions=_p(rg.positions), row_entry=_p(rg.row_entry), page_indptr=_p(page_indptr),
                   page_ids=_p(page_ids), cache=_p(cache), page_stride=page_stride, k_cache_off=k_off, v_cache_off=v_off, page_size=page_size,
                   shared_tail=shared_tail, q_out=_p(q), n_rows=proj.shape[0], dtype=_dt(cache))
    _chk(ffi.lib().pegainfer_qk_prep(ctypes.addressof(p), _stream()), "qk_prep")
    return q


def gated_linear(proj, offs, z_f32, z_bias, tau, q_scale, state, heads, dim, vdim, rg, scan_max=0, w_up=None, low_off=0, rank=0):
    """proj rows [.. q at offs[0] | k at offs[1] | v at offs[2] ..]; z fp32 [rows, heads * dim], or None: w_up [heads * dim, rank padded to 8]
    times the row's rank values at low_off; state fp32 [slots, heads * dim * vdim]; scan_max > 0: entries of more rows take the chunk form
    -> fp32 [rows, heads * vdim]"""
    o = torch.empty((proj.shape[0], heads * vdim), dtype=torch.float32, device=proj.device)
    d = GatedLinearDesc(proj=_p(proj), proj_stride=proj.stride(0), q_off=offs[0], k_off=offs[1], v_off=offs[2], q_scale=float(q_scale),
                        z=_p(z_f32), z_stride=0 if z_f32 is None else z_f32.stride(0), z_bias=_p(z_bias), tau=float(tau), w_up=_p(w_up),
                        low_off=low_off, rank=rank, rank_stride=0 if w_up is None else w_up.stride(0), state=_p(state),
                        slot_stride=state.stride(0), o=_p(o), heads=heads, dim=dim, vdim=vdim, entry_row0=_p(rg.entry_row0),
                        entry_slot=_p(rg.entry_slot), n_entries=len(rg.lens), dtype=_dt(proj))
    keep = _chunk_tables(d, rg, scan_max, ffi.lib().pegainfer_gated_linear_workspace, heads, dim, vdim)  # noqa: F841 (alive until enqueued)
    _chk(ffi.lib().pegainfer_gated_linear(ctypes.addressof(d), _stream()), "gated_linear")
    return o
