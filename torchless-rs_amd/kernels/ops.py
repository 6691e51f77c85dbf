"""Python faces of the HIP kernels.

Every function checks on the host that its operands are on the GPU,
contiguous, of the type and shape that the kernel and its grid assume, and
launches on torch's current stream.  A failure of the launcher raises
`KernelError` with the library's message.  There is no fallback: without the
library nothing here runs.
"""
from __future__ import annotations

import ctypes
import functools
from typing import Optional

import torch

from .build import load, load_measure
from .page import PAGE, require_same

DT_F32, DT_BF16 = 0, 1
_CODES = {torch.float32: DT_F32, torch.bfloat16: DT_BF16}


class KernelError(RuntimeError):
    pass


_configured = False


def lib() -> ctypes.CDLL:
    global _configured
    L = load()
    if not _configured:
        L.tl_last_error.restype = ctypes.c_char_p
        require_same(L.tl_page_size(), "the kernels' library")
        _configured = True
    return L


def _check(rc: int) -> None:
    if rc != 0:
        raise KernelError(lib().tl_last_error().decode())


def _code(dt: torch.dtype) -> int:
    if dt not in _CODES:
        raise KernelError(f"dtype {dt} is not served by the kernels (float32 and bfloat16 are)")
    return _CODES[dt]


def _p(t: Optional[torch.Tensor]) -> ctypes.c_void_p:
    return ctypes.c_void_p(0 if t is None else t.data_ptr())


_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)


def _stream() -> ctypes.c_void_p:
    """The current stream's handle (the short way where torch has it: a stream object for every launch
    costs the host a fifth of a step that is not a captured graph)."""
    if _raw_stream is not None:
        return ctypes.c_void_p(_raw_stream(torch.cuda.current_device()))
    return ctypes.c_void_p(torch.cuda.current_stream().cuda_stream)


def _req(t: torch.Tensor, name: str, dtype=None, shape=None) -> None:
    # one test on the usual way (every launch asks several times); what is wrong is named below
    if (t.is_cuda and t.is_contiguous() and (dtype is None or t.dtype == dtype)
            and (shape is None or t.shape == tuple(shape))):
        return
    if not t.is_cuda:
        raise KernelError(f"{name}: must be on the GPU")
    if not t.is_contiguous():
        raise KernelError(f"{name}: must be contiguous")
    if dtype is not None and t.dtype != dtype:
        raise KernelError(f"{name}: dtype {t.dtype}, kernel needs {dtype}")
    raise KernelError(f"{name}: shape {tuple(t.shape)}, kernel needs {tuple(shape)}")


def embed(table: torch.Tensor, ids: torch.Tensor, out: torch.Tensor, scale: float = 1.0) -> None:
    """out[n, :] = table[ids[n], :] widened to float32, times `scale`."""
    n, H = ids.shape[0], table.shape[1]
    _req(table, "embed.table")
    _req(ids, "embed.ids", torch.int32, (n,))
    _req(out, "embed.out", torch.float32, (n, H))
    _check(lib().tl_embed(_p(table), _code(table.dtype), _p(ids), n, H, ctypes.c_float(scale), _p(out), _stream()))


class PairTable:
    """A second embedding table read by pairs of tokens: row (previous * mul_prev + current * mul_cur) mod `buckets` of `table`
    [buckets + 1, H]; a sequence's first token reads the last row.  The previous token of a sequence's first row of
    a step is what the step before left in the sequence's block."""

    def __init__(self, table: torch.Tensor, buckets: int, mul_prev: int, mul_cur: int):
        self.table, self.buckets = table, int(buckets)
        self.mul_prev, self.mul_cur = int(mul_prev) % self.buckets, int(mul_cur) % self.buckets     # (the same rows, smaller products)


def embed_pairs(table: torch.Tensor, ids: torch.Tensor, scale: float, pairs: Optional[PairTable], row_pos, row_seq, cu_seqlens,
                slots, last: Optional[torch.Tensor], norm_weight: Optional[torch.Tensor], eps: float, out: torch.Tensor) -> None:
    """out[n, :] = table[ids[n], :] * scale, plus the pair's row (`pairs`), then divided by the row's root mean square and times
    `norm_weight` (float32 [H]; None: no norm), all in float32.  `last` (int32 [slots, 1]): every sequence's last token, read for
    its first row (unless that is position 0) and left behind by this step."""
    n, H = ids.shape[0], table.shape[1]
    B = slots.shape[0]
    _req(table, "embed_pairs.table")
    _req(ids, "embed_pairs.ids", torch.int32, (n,))
    if pairs is not None:
        _req(pairs.table, "embed_pairs.pairs", table.dtype, (pairs.buckets + 1, H))
        _req(row_pos, "embed_pairs.row_pos", torch.int32, (n,))
        _req(row_seq, "embed_pairs.row_seq", torch.int32, (n,))
        _req(cu_seqlens, "embed_pairs.cu_seqlens", torch.int32, (B + 1,))
        _req(slots, "embed_pairs.slots", torch.int32)
        if last is None:
            raise KernelError("embed_pairs: pairs need the sequences' last tokens")
        _req(last, "embed_pairs.last", torch.int32, (last.shape[0], 1))
    if norm_weight is not None:
        _req(norm_weight, "embed_pairs.norm_weight", torch.float32, (H,))
    _req(out, "embed_pairs.out", torch.float32, (n, H))
    p = pairs
    _check(lib().tl_embed_pairs(_p(table), _code(table.dtype), _p(ids), n, H, ctypes.c_float(scale), _p(p.table) if p else None,
                                ctypes.c_longlong(p.buckets if p else 1), ctypes.c_longlong(p.mul_prev if p else 0),
                                ctypes.c_longlong(p.mul_cur if p else 0), _p(row_pos), _p(row_seq), _p(cu_seqlens), _p(slots),
                                _p(last), _p(norm_weight), ctypes.c_float(eps), _p(out), _stream()))


def rmsnorm_add(z: torch.Tensor, w: torch.Tensor, eps: float, x: torch.Tensor, w_next: Optional[torch.Tensor] = None,
                eps_next: float = 0.0, out: Optional[torch.Tensor] = None) -> None:
    """The RMS norm of a sublayer's output added to the stream: x += z / sqrt(mean(z^2) + eps) * w
    (z, x float32 [n, H]).  With `w_next` the norm that reads the stream next runs in the same
    kernel: out = x / sqrt(mean(x^2) + eps_next) * w_next, in `out`'s dtype."""
    n, H = z.shape
    _req(z, "rmsnorm_add.z", torch.float32)
    _req(w, "rmsnorm_add.w", torch.float32, (H,))
    _req(x, "rmsnorm_add.x", torch.float32, (n, H))
    if w_next is not None:
        _req(w_next, "rmsnorm_add.w_next", torch.float32, (H,))
        if out is None:
            raise KernelError("rmsnorm_add: the norm that follows needs `out`")
        _req(out, "rmsnorm_add.out", None, (n, H))
    _check(lib().tl_rmsnorm_add(_p(z), _p(w), ctypes.c_float(eps), _p(x), _p(w_next), ctypes.c_float(eps_next),
                                _p(out) if w_next is not None else None,
                                _code(out.dtype) if w_next is not None else DT_F32, n, H, _stream()))


def stream_entry(x: torch.Tensor, extra: Optional[torch.Tensor], vec: torch.Tensor) -> None:
    """x[n, :] += extra[n, :] (None: nothing) + vec[:], all float32."""
    n, H = x.shape
    _req(x, "stream_entry.x", torch.float32)
    if extra is not None:
        _req(extra, "stream_entry.extra", torch.float32, (n, H))
    _req(vec, "stream_entry.vec", torch.float32, (H,))
    _check(lib().tl_stream_entry(_p(x), _p(extra), _p(vec), n, H, _stream()))


def scale_(x: torch.Tensor, s: float) -> None:
    """x *= s (float32, in place)."""
    _req(x, "scale.x", torch.float32)
    _check(lib().tl_scale(_p(x), ctypes.c_float(s), ctypes.c_longlong(x.numel()), _stream()))


def rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float, out: torch.Tensor) -> None:
    """out = x / sqrt(mean(x^2) + eps) * w, x float32 [n, H], w float32 [H]."""
    n, H = x.shape
    _req(x, "rmsnorm.x", torch.float32)
    _req(w, "rmsnorm.w", torch.float32, (H,))
    _req(out, "rmsnorm.out", None, (n, H))
    _check(lib().tl_rmsnorm(_p(x), _p(w), ctypes.c_float(eps), _p(out), _code(out.dtype), n, H,
                            _stream()))


class Rotation:
    """How q and k are rotated by position: the first `rotary_dim` channels of a head in pairs,
    pair i by the angle pos * inv_freq[i] (float32 [rotary_dim / 2] on the device); pairs are
    (i, i + rotary_dim/2), or (2i, 2i+1) when `interleaved`; the channels behind them pass
    through.  rotary_dim 0 (inv_freq None): nothing is rotated.  `magnitude`: a factor on both cosine
    and sine, hence on the rotated channels alone (served by `retention_scan`, `retention_prepare` and
    `latent_prepare`; the other kernels refuse one that is not 1)."""

    def __init__(self, inv_freq: Optional[torch.Tensor], rotary_dim: int, interleaved: bool = False,
                 magnitude: float = 1.0):
        self.inv_freq, self.rotary_dim, self.interleaved = inv_freq, int(rotary_dim), bool(interleaved)
        self.magnitude = float(magnitude)


NO_ROTATION = Rotation(None, 0)


def _rotation(rot, d: int, what: str, magnitude: bool = False) -> Rotation:
    """A `Rotation` checked against the head size `d`.  A bare tensor of d/2 frequencies stands
    for the rotation of the whole head in halves; None for no rotation.  `magnitude`: does the
    kernel take a factor on cosines and sines?"""
    if rot is None:
        return NO_ROTATION
    if not magnitude and isinstance(rot, Rotation) and rot.magnitude != 1.0:
        raise KernelError(f"{what}: a factor of {rot.magnitude} on the rotated channels is not served")
    if isinstance(rot, torch.Tensor):
        rot = Rotation(rot, d)
    if rot.rotary_dim % 2 or not (0 <= rot.rotary_dim <= d):
        raise KernelError(f"{what}: {rot.rotary_dim} rotated channels of a head of {d} (even, at most the head)")
    if rot.rotary_dim:
        _req(rot.inv_freq, what + ".inv_freq", torch.float32, (rot.rotary_dim // 2,))
    return rot


def rope_split(qkv: torch.Tensor, row_pos: torch.Tensor, rotation, nq: int, nkv: int,
               d: int, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, vt: Optional[torch.Tensor] = None,
               row_seq=None, tile_off=None, n_cached=None) -> None:
    """Rotate q and k of the fused projection by their rows' positions (`rotation`: a
    `Rotation`, or the d/2 frequencies of a whole head rotated in halves) and
    write q [n,nq,d], k, v [n,nkv,d] (v may be None: the values are taken by
    `v_tiles` then).  With `vt` [nkv, d, cols] the values are
    also written transposed, row n into column tile_off[b] + pos - 64 *
    (n_cached[b] // 64) of its sequence b = row_seq[n]."""
    n = qkv.shape[0]
    _req(qkv, "rope.qkv", torch.float32, (n, (nq + 2 * nkv) * d))
    _req(row_pos, "rope.row_pos", torch.int32, (n,))
    rot = _rotation(rotation, d, "rope")
    _req(q, "rope.q", None, (n, nq, d))
    if nkv:
        _req(k, "rope.k", q.dtype, (n, nkv, d))
        if v is not None:
            _req(v, "rope.v", q.dtype, (n, nkv, d))
    cols = 0
    if vt is not None:
        _req(vt, "rope.vt", q.dtype)
        if vt.dim() != 3 or tuple(vt.shape[:2]) != (nkv, d):
            raise KernelError(f"rope.vt: shape {tuple(vt.shape)}, kernel needs [{nkv}, {d}, columns]")
        cols = vt.shape[2]
        _req(row_seq, "rope.row_seq", torch.int32, (n,))
        _req(tile_off, "rope.tile_off", torch.int32)
        _req(n_cached, "rope.n_cached", torch.int32, tuple(tile_off.shape))
    _check(lib().tl_rope_split(_p(qkv), _p(row_pos), _p(rot.inv_freq), rot.rotary_dim, int(rot.interleaved),
                               n, nq, nkv, d, _p(q), _p(k), _p(v),
                               _p(vt), cols, _p(row_seq), _p(tile_off), _p(n_cached), _code(q.dtype),
                               _stream()))


def kv_commit(k: torch.Tensor, v: torch.Tensor, row_seq, row_pos, len_after, table: torch.Tensor,
              ring_pages: int, pages: torch.Tensor) -> None:
    """Write this step's keys and values into the pages of one layer.
    pages: [n_pages, 2, nkv, PAGE, d]; table: [B, stride] page ids."""
    n, nkv, d = k.shape
    _req(k, "kv_commit.k", pages.dtype)
    _req(v, "kv_commit.v", pages.dtype, (n, nkv, d))
    _req(row_seq, "kv_commit.row_seq", torch.int32, (n,))
    _req(row_pos, "kv_commit.row_pos", torch.int32, (n,))
    _req(len_after, "kv_commit.len_after", torch.int32)
    _req(table, "kv_commit.table", torch.int32)
    _req(pages, "kv_commit.pages")
    if pages.dim() != 5 or tuple(pages.shape[1:]) != (2, nkv, PAGE, d):
        raise KernelError(f"kv_commit.pages: shape {tuple(pages.shape)}, kernel needs [*, 2, {nkv}, {PAGE}, {d}]")
    if table.dim() != 2 or table.shape[0] != len_after.shape[0]:
        raise KernelError("kv_commit.table: needs one row per sequence")
    _check(lib().tl_kv_commit(_p(k), _p(v), _code(k.dtype), _p(row_seq), _p(row_pos), _p(len_after),
                              _p(table), table.shape[1], ring_pages, n, nkv, d, _p(pages), _stream()))


def _tiles_args(B, cu_seqlens, tile_off, n_cached, len_after, what):
    _req(tile_off, what + ".tile_off", torch.int32, (B,))
    _req(n_cached, what + ".n_cached", torch.int32, (B,))
    _req(len_after, what + ".len_after", torch.int32, (B,))
    if cu_seqlens is not None:
        _req(cu_seqlens, what + ".cu_seqlens", torch.int32, (B + 1,))


def v_tiles(qkv: torch.Tensor, nq: int, nkv: int, d: int, vt: torch.Tensor, cu_seqlens, tile_off, n_cached,
            len_after) -> None:
    """The values of a step transposed, from the fused projection: vt[kv head, dv, column],
    sequence b from column tile_off[b] on (`aligned_columns`), written by tiles of 64
    positions in whole lines.  Columns that hold no position of this step are left alone."""
    n = qkv.shape[0]
    _req(qkv, "v_tiles.qkv", torch.float32, (n, (nq + 2 * nkv) * d))
    _req(vt, "v_tiles.vt")
    if vt.dim() != 3 or tuple(vt.shape[:2]) != (nkv, d) or vt.shape[2] % PAGE:
        raise KernelError(f"v_tiles.vt: shape {tuple(vt.shape)}, kernel needs [{nkv}, {d}, a multiple of {PAGE}]")
    B = tile_off.shape[0]
    _tiles_args(B, cu_seqlens, tile_off, n_cached, len_after, "v_tiles")
    _check(lib().tl_v_tiles(_p(qkv), n, nq, nkv, d, _p(vt), vt.shape[2], _code(vt.dtype), B, _p(cu_seqlens),
                            _p(tile_off), _p(n_cached), _p(len_after), _stream()))


def v_tiles_rows(v: torch.Tensor, vt: torch.Tensor, cu_seqlens, tile_off, n_cached, len_after) -> None:
    """`v_tiles` from rows of values alone: v [n, nkv, d] in vt's dtype -> vt [nkv, d, columns]."""
    n, nkv, d = v.shape
    _req(v, "v_tiles_rows.v", vt.dtype)
    _req(vt, "v_tiles_rows.vt")
    if vt.dim() != 3 or tuple(vt.shape[:2]) != (nkv, d) or vt.shape[2] % PAGE:
        raise KernelError(f"v_tiles_rows.vt: shape {tuple(vt.shape)}, kernel needs [{nkv}, {d}, a multiple of {PAGE}]")
    B = tile_off.shape[0]
    _tiles_args(B, cu_seqlens, tile_off, n_cached, len_after, "v_tiles_rows")
    _check(lib().tl_v_tiles_rows(_p(v), n, nkv, d, _p(vt), vt.shape[2], _code(vt.dtype), B, _p(cu_seqlens),
                                 _p(tile_off), _p(n_cached), _p(len_after), _stream()))


def rope_v_tiles(qkv: torch.Tensor, row_pos, rotation, nq: int, nkv: int, d: int, q: torch.Tensor, k: torch.Tensor,
                 vt: torch.Tensor, cu_seqlens, tile_off, n_cached, len_after) -> None:
    """`rope_split` (q and k) and `v_tiles` in one launch: the same bits as the two."""
    n = qkv.shape[0]
    _req(qkv, "rope_v_tiles.qkv", torch.float32, (n, (nq + 2 * nkv) * d))
    _req(row_pos, "rope_v_tiles.row_pos", torch.int32, (n,))
    rot = _rotation(rotation, d, "rope_v_tiles")
    _req(q, "rope_v_tiles.q", None, (n, nq, d))
    _req(k, "rope_v_tiles.k", q.dtype, (n, nkv, d))
    _req(vt, "rope_v_tiles.vt", q.dtype)
    if vt.dim() != 3 or tuple(vt.shape[:2]) != (nkv, d) or vt.shape[2] % PAGE:
        raise KernelError(f"rope_v_tiles.vt: shape {tuple(vt.shape)}, kernel needs [{nkv}, {d}, a multiple of {PAGE}]")
    B = tile_off.shape[0]
    _tiles_args(B, cu_seqlens, tile_off, n_cached, len_after, "rope_v_tiles")
    if cu_seqlens is None:
        raise KernelError("rope_v_tiles.cu_seqlens: needed")
    _check(lib().tl_rope_v_tiles(_p(qkv), _p(row_pos), _p(rot.inv_freq), rot.rotary_dim, int(rot.interleaved), n, nq,
                                 nkv, d, _p(q), _p(k), _p(vt), vt.shape[2], B, _p(cu_seqlens), _p(tile_off),
                                 _p(n_cached), _p(len_after), _code(q.dtype), _stream()))


def kv_commit_tiles(k: torch.Tensor, vt: torch.Tensor, row_seq, row_pos, tile_off, n_cached, len_after,
                    table: torch.Tensor, ring_pages: int, pages: torch.Tensor) -> None:
    """`kv_commit` for a step whose values lie transposed by tiles (`v_tiles`): keys row by
    row, values a tile [d, 64] at a time in whole lines."""
    n, nkv, d = k.shape
    _req(k, "kv_commit.k", pages.dtype)
    _req(vt, "kv_commit.vt", pages.dtype)
    if vt.dim() != 3 or tuple(vt.shape[:2]) != (nkv, d) or vt.shape[2] % PAGE:
        raise KernelError(f"kv_commit.vt: shape {tuple(vt.shape)}, kernel needs [{nkv}, {d}, a multiple of {PAGE}]")
    _req(row_seq, "kv_commit.row_seq", torch.int32, (n,))
    _req(row_pos, "kv_commit.row_pos", torch.int32, (n,))
    B = tile_off.shape[0]
    _tiles_args(B, None, tile_off, n_cached, len_after, "kv_commit")
    _req(table, "kv_commit.table", torch.int32)
    _req(pages, "kv_commit.pages")
    if pages.dim() != 5 or tuple(pages.shape[1:]) != (2, nkv, PAGE, d):
        raise KernelError(f"kv_commit.pages: shape {tuple(pages.shape)}, kernel needs [*, 2, {nkv}, {PAGE}, {d}]")
    if table.dim() != 2 or table.shape[0] != B:
        raise KernelError("kv_commit.table: needs one row per sequence")
    _check(lib().tl_kv_commit_tiles(_p(k), _p(vt), vt.shape[2], _code(k.dtype), _p(row_seq), _p(row_pos), B,
                                    _p(tile_off), _p(n_cached), _p(len_after), _p(table), table.shape[1],
                                    ring_pages, n, nkv, d, _p(pages), _stream()))


def attn_plain(q, k_new, v_new, pages, table, ring_pages: int, row_seq, row_pos, cu_seqlens, n_cached,
               window: Optional[int], scale: float, out) -> None:
    """Attention of every row over its sequence's cached keys (j < n_cached)
    and this step's keys (k_new/v_new rows), causal, with an optional window."""
    n, nq, d = q.shape
    nkv = pages.shape[2]
    B = n_cached.shape[0]
    _req(q, "attn.q", pages.dtype)
    if k_new is not None:
        _req(k_new, "attn.k_new", pages.dtype, (n, nkv, d))
        _req(v_new, "attn.v_new", pages.dtype, (n, nkv, d))
    _req(pages, "attn.pages")
    if pages.dim() != 5 or tuple(pages.shape[1:]) != (2, nkv, PAGE, d):
        raise KernelError(f"attn.pages: shape {tuple(pages.shape)}, kernel needs [*, 2, nkv, {PAGE}, {d}]")
    _req(table, "attn.table", torch.int32)
    _req(row_seq, "attn.row_seq", torch.int32, (n,))
    _req(row_pos, "attn.row_pos", torch.int32, (n,))
    _req(cu_seqlens, "attn.cu_seqlens", torch.int32, (B + 1,))
    _req(n_cached, "attn.n_cached", torch.int32, (B,))
    _req(out, "attn.out", pages.dtype, (n, nq, d))
    if table.dim() != 2 or table.shape[0] != B:
        raise KernelError("attn.table: needs one row per sequence")
    _check(lib().tl_attn_plain(_p(q), _p(k_new), _p(v_new), _p(pages), _code(q.dtype), _p(table),
                               table.shape[1], ring_pages, _p(row_seq), _p(row_pos), _p(cu_seqlens),
                               _p(n_cached), n, nq, nkv, d, int(window or 0), ctypes.c_float(scale),
                               _p(out), _stream()))


def silu_mul(gu: torch.Tensor, out: torch.Tensor) -> None:
    """out[n, i] = silu(gu[n, i]) * gu[n, I + i]."""
    n, I2 = gu.shape
    _req(gu, "silu_mul.gu", torch.float32)
    _req(out, "silu_mul.out", None, (n, I2 // 2))
    _check(lib().tl_silu_mul(_p(gu), n, I2 // 2, _p(out), _code(out.dtype), _stream()))


def silu_mul_pairs(gu: torch.Tensor, out: torch.Tensor, activation: str = "silu", constants=None) -> None:
    """The same on bfloat16 gu whose columns come in groups of 64: 32 of gate,
    then the 32 of up that belong to them (`interleave_pairs`); `activation`: the gate's
    function (`ACTIVATIONS`)."""
    n, I2 = gu.shape
    _req(gu, "silu_mul_pairs.gu", torch.bfloat16)
    _req(out, "silu_mul_pairs.out", torch.bfloat16, (n, I2 // 2))
    if activation == "silu":
        _check(lib().tl_silu_mul_pairs(_p(gu), n, I2 // 2, _p(out), _stream()))
        return
    if activation not in ACTIVATIONS:
        raise KernelError(f"silu_mul_pairs: no function {activation!r}; there are {sorted(ACTIVATIONS)}")
    _check(lib().tl_act_mul_pairs(_p(gu), n, I2 // 2, ACTIVATIONS[activation], *_act_constants(activation, constants),
                                  _p(out), _stream()))


def layernorm(z: torch.Tensor, w: torch.Tensor, eps: float, out: Optional[torch.Tensor] = None,
              add_to: Optional[torch.Tensor] = None, bias: Optional[torch.Tensor] = None,
              beta: Optional[torch.Tensor] = None) -> None:
    """Layer norm, y = (z - mean) / sqrt(var + eps) * w + beta over z float32 [n, H] (`beta`: the norm's
    own bias, or None; `bias`: added to z first, the bias of the product that made z).  Without
    `add_to`, y goes to `out` (float32 or the compute dtype).  With it, the stream add_to += y,
    and `out`, if given, receives the new stream in its dtype."""
    n, H = z.shape
    _req(z, "layernorm.z", torch.float32)
    _req(w, "layernorm.w", torch.float32, (H,))
    if bias is not None:
        _req(bias, "layernorm.bias", torch.float32, (H,))
    if beta is not None:
        _req(beta, "layernorm.beta", torch.float32, (H,))
    if add_to is not None:
        _req(add_to, "layernorm.add_to", torch.float32, (n, H))
    elif out is None:
        raise KernelError("layernorm: needs `out` or `add_to`")
    if out is not None:
        _req(out, "layernorm.out", None, (n, H))
    _check(lib().tl_layernorm(_p(z), _p(bias), _p(w), _p(beta), ctypes.c_float(eps), _p(add_to), _p(out),
                              _code(out.dtype) if out is not None else DT_F32, n, H, _stream()))


def layernorm_rows_in_registers(H: int) -> bool:
    """Does `layernorm_add_norm` take rows of H channels?"""
    return H % 4 == 0 and H <= 8192


def layernorm_add_norm(z: torch.Tensor, w: torch.Tensor, beta, eps: float, x: torch.Tensor, bias=None,
                       w_next=None, beta_next=None, eps_next: float = 0.0, out=None, mix=None) -> None:
    """x += LN(z + bias; w, beta) and, with `w_next`, out = LN(x; w_next, beta_next) of the new row, in one
    kernel that holds the row in registers (`layernorm_rows_in_registers`).  z, x float32 [n, H]; out
    [n, H] float32 or the compute dtype.  `mix` = (kept, coef, t): between the two, what `depth_average` does:
    the new x is kept as version t and replaced by the weighted sum of versions 0 .. t."""
    n, H = z.shape
    _req(z, "layernorm_add_norm.z", torch.float32)
    _req(x, "layernorm_add_norm.x", torch.float32, (n, H))
    for t, name in ((w, "w"), (beta, "beta"), (bias, "bias"), (w_next, "w_next"), (beta_next, "beta_next")):
        if t is not None:
            _req(t, "layernorm_add_norm." + name, torch.float32, (H,))
    if w_next is not None:
        _req(out, "layernorm_add_norm.out", None, (n, H))
    kept = coef = None
    t = 0
    if mix is not None:
        kept, coef, t = mix
        _req(kept, "layernorm_add_norm.kept", torch.float32)
        _req(coef, "layernorm_add_norm.coef", torch.float32)
        if kept.dim() != 3 or tuple(kept.shape[1:]) != (n, H) or kept.shape[0] <= t or coef.numel() <= t or t < 0:
            raise KernelError(f"layernorm_add_norm: version {t} of a stream {(n, H)} in {tuple(kept.shape)} with "
                              f"{coef.numel()} weights")
    _check(lib().tl_layernorm_add_norm(_p(z), _p(bias), _p(w), _p(beta), ctypes.c_float(eps), _p(x), _p(w_next),
                                       _p(beta_next) if w_next is not None else None, ctypes.c_float(eps_next),
                                       _p(out) if w_next is not None else None,
                                       _code(out.dtype) if w_next is not None else DT_F32, n, H, _p(kept), _p(coef), int(t),
                                       _stream()))


def depth_average(x: torch.Tensor, kept: torch.Tensor, coef: torch.Tensor, t: int) -> None:
    """kept[t] = x, then x = sum over j <= t of coef[j] * kept[j]: the stream that goes on is a weighted sum
    of the stream's earlier versions and this one.  x float32 [n, H], kept float32 [>= t + 1, n, H], coef
    float32 [>= t + 1]."""
    _req(x, "depth_average.x", torch.float32)
    _req(kept, "depth_average.kept", torch.float32)
    _req(coef, "depth_average.coef", torch.float32)
    if kept.dim() != 3 or tuple(kept.shape[1:]) != tuple(x.shape) or kept.shape[0] <= t or coef.numel() <= t or t < 0:
        raise KernelError(f"depth_average: version {t} of a stream {tuple(x.shape)} in {tuple(kept.shape)} with "
                          f"{coef.numel()} weights")
    _check(lib().tl_depth_average(_p(x), _p(kept), _p(coef), int(t), ctypes.c_longlong(x.numel()), _stream()))


def gated_recurrence_chunk() -> int:
    """Rows in a run of `gated_recurrence`'s second way."""
    return int(lib().tl_gated_recurrence_chunk())


def gated_recurrence(proj: torch.Tensor, bz, bx, state: torch.Tensor, cu_seqlens, slots, out: torch.Tensor,
                     n_runs: int = 0, scratch=None) -> None:
    """A gated recurrence per channel over the rows of a step, sequence by sequence.  proj float32 [n, 3 W] =
    [a | b | g]: z = logistic(a + bz), c = cand(b + bx) (u + 1/2 for u >= 0, logistic(u) below),
    S <- (1 - z) S + z c, out = S * silu(g).  `state` float32 [slots, >= W] (rows may be strided) is read and
    left updated.  `n_runs` 0: a thread a (sequence, channel) goes through the rows in order; else the step's
    number of runs of `gated_recurrence_chunk()` rows (sum over sequences of the rounded-up quotient): a
    workgroup a run, with `scratch` float32 [>= (2 n_runs + B) W]."""
    n, W3 = proj.shape
    W = W3 // 3
    B = slots.shape[0]
    _req(proj, "gated_recurrence.proj", torch.float32)
    if W3 != 3 * W:
        raise KernelError(f"gated_recurrence: a row of {W3} is not [a | b | g]")
    for t, name in ((bz, "bz"), (bx, "bx")):
        if t is not None:
            _req(t, "gated_recurrence." + name, torch.float32, (W,))
    if state.dtype != torch.float32 or state.dim() != 2 or state.stride(1) != 1 or not state.is_cuda or state.shape[1] < W:
        raise KernelError("gated_recurrence.state: float32 [slots, >= W] on the GPU, rows may be strided")
    _req(cu_seqlens, "gated_recurrence.cu_seqlens", torch.int32, (B + 1,))
    _req(slots, "gated_recurrence.slots", torch.int32)
    _req(out, "gated_recurrence.out", None, (n, W))
    if n_runs:
        _req(scratch, "gated_recurrence.scratch", torch.float32)
        if scratch.numel() < (2 * n_runs + B) * W:
            raise KernelError(f"gated_recurrence: scratch of {scratch.numel()} for {n_runs} runs of {B} sequences")
    _check(lib().tl_gated_recurrence(_p(proj), _p(bz), _p(bx), n, W, _p(state), ctypes.c_longlong(state.stride(0)),
                                     _p(cu_seqlens), _p(slots), B, int(n_runs), _p(scratch) if n_runs else None,
                                     _p(out), _code(out.dtype), _stream()))


def cast_rows(x: torch.Tensor, out: torch.Tensor) -> None:
    """out = x rounded to bfloat16 (x float32, same shape)."""
    _req(x, "cast_rows.x", torch.float32)
    _req(out, "cast_rows.out", torch.bfloat16, tuple(x.shape))
    _check(lib().tl_cast_rows(_p(x), ctypes.c_longlong(x.numel()), _p(out), _stream()))


# The functions of a gated feed-forward.  silu: g / (1 + e^-g); gelu_tanh: the tanh form of gelu;
# swish_clamped, with the constants `alpha`, `limit` and `shift`: g' = min(g, limit),
# u' = clamp(u, -limit, limit), and the hidden value is g' / (1 + e^(-alpha g')) * (u' + shift).
ACTIVATIONS = {"silu": 0, "gelu_tanh": 1, "swish_clamped": 2, "relu": 3}
ACTIVATION_CONSTANTS = {"swish_clamped": ("alpha", "limit", "shift")}


def _act_constants(activation: str, constants):
    """(alpha, limit, shift) as the kernels take them; a function without constants ignores them."""
    names = ACTIVATION_CONSTANTS.get(activation, ())
    given = dict(constants or {})
    if set(given) != set(names):
        raise KernelError(f"activation {activation!r} takes the constants {sorted(names)}, got {sorted(given)}")
    return tuple(ctypes.c_float(float(given.get(k, 0.0))) for k in ("alpha", "limit", "shift"))


def act_mul(gu: torch.Tensor, out: torch.Tensor, activation: str = "silu", constants=None) -> None:
    """out[n, i] = act(gu[n, i]) * gu[n, I + i]; act: one of `ACTIVATIONS`, `constants` its constants."""
    n, I2 = gu.shape
    if activation not in ACTIVATIONS:
        raise KernelError(f"act_mul: no function {activation!r}; there are {sorted(ACTIVATIONS)}")
    _req(gu, "act_mul.gu", torch.float32)
    _req(out, "act_mul.out", None, (n, I2 // 2))
    _check(lib().tl_act_mul(_p(gu), n, I2 // 2, ACTIVATIONS[activation], *_act_constants(activation, constants),
                            _p(out), _code(out.dtype), _stream()))


class ScoreTerms:
    """What an attention adds to q.k * scale: `slopes` (float32 [nq] or None), a bias
    -slope[h] * (p - j) by the distance of query and key; `sinks` (float32 [nq] or None), a score
    per head with no key and no value that takes part in the softmax's sum once; `window`;
    `keep_first`: with a window, the first positions of a sequence that stay visible beside it
    (the cache must then keep every position: a ring would overwrite them); `chunk`: a key is seen
    only inside the query's run of that many positions counted from the sequence's start,
    floor(j / chunk) == floor(p / chunk); `logistic`: the weight of a key is
    1 / (1 + exp(-(score + score_bias[h]))), every key by itself, instead of a softmax over the keys
    (`score_bias` float32 [nq] or None; no sink)."""

    def __init__(self, scale: float, window: Optional[int] = None, slopes: Optional[torch.Tensor] = None,
                 sinks: Optional[torch.Tensor] = None, keep_first: int = 0, chunk: Optional[int] = None,
                 logistic: bool = False, score_bias: Optional[torch.Tensor] = None):
        self.scale, self.window, self.slopes, self.sinks = float(scale), (int(window) if window else None), slopes, sinks
        self.keep_first = int(keep_first) if self.window else 0
        self.chunk = int(chunk) if chunk else 0
        self.logistic, self.score_bias = bool(logistic), score_bias
        if self.logistic and sinks is not None:
            raise KernelError("attention: logistic weights have no sink")
        if score_bias is not None and not self.logistic:
            raise KernelError("attention: a bias on the score goes with logistic weights (a softmax does not see it)")

    @property
    def reach(self) -> Optional[int]:
        """How many positions back a query may look (None: to the first)."""
        if self.window and self.keep_first:
            return None
        both = [v for v in (self.window, self.chunk) if v]
        return min(both) if both else None


def _req_pages(pages: torch.Tensor, nkv: int, dk: int, dv: int, what: str) -> None:
    _req(pages, what + ".pages")
    per_page = pages.numel() // pages.shape[0] if pages.shape[0] else 0
    if pages.dim() < 2 or per_page != nkv * PAGE * (dk + dv):
        raise KernelError(f"{what}.pages: shape {tuple(pages.shape)}, kernel needs {nkv * PAGE * (dk + dv)} "
                          f"elements a page ({nkv} KV heads of {PAGE} keys of {dk} and values of {dv})")


def attn_scored_plain(q, k_new, v_new, pages, nkv: int, dv: int, table, ring_pages: int, row_seq, row_pos,
                      cu_seqlens, n_cached, terms: ScoreTerms, gate, out) -> None:
    """Attention of every row over its sequence's cached keys (j < n_cached) and this step's
    (k_new [n, nkv, dk], v_new [n, nkv, dv]; None when everything is in the pages), causal, with
    the terms of `ScoreTerms`; `gate` (float32 [n, nq] or None) multiplies each head's output.
    One wave per (row, head), float32 sums; `out` may be float32 whatever the operands are."""
    n, nq, dk = q.shape
    B = n_cached.shape[0]
    _req(q, "attn_scored.q", pages.dtype)
    if k_new is not None:
        _req(k_new, "attn_scored.k_new", pages.dtype, (n, nkv, dk))
        _req(v_new, "attn_scored.v_new", pages.dtype, (n, nkv, dv))
    _req_pages(pages, nkv, dk, dv, "attn_scored")
    _req(table, "attn_scored.table", torch.int32)
    _req(row_seq, "attn_scored.row_seq", torch.int32, (n,))
    _req(row_pos, "attn_scored.row_pos", torch.int32, (n,))
    _req(cu_seqlens, "attn_scored.cu_seqlens", torch.int32, (B + 1,))
    _req(n_cached, "attn_scored.n_cached", torch.int32, (B,))
    _req(out, "attn_scored.out", torch.float32 if out.dtype == torch.float32 else pages.dtype, (n, nq, dv))
    if terms.slopes is not None:
        _req(terms.slopes, "attn_scored.slopes", torch.float32, (nq,))
    if terms.sinks is not None:
        _req(terms.sinks, "attn_scored.sinks", torch.float32, (nq,))
    if gate is not None:
        _req(gate, "attn_scored.gate", torch.float32, (n, nq))
    if terms.score_bias is not None:
        _req(terms.score_bias, "attn_scored.score_bias", torch.float32, (nq,))
    if table.dim() != 2 or table.shape[0] != B:
        raise KernelError("attn_scored.table: needs one row per sequence")
    _check(lib().tl_attn_scored_plain(_p(q), _p(k_new), _p(v_new), _p(pages), _code(q.dtype), _p(table),
                                      table.shape[1], ring_pages, _p(row_seq), _p(row_pos), _p(cu_seqlens),
                                      _p(n_cached), n, nq, nkv, dk, dv, int(terms.window or 0), terms.keep_first,
                                      terms.chunk, ctypes.c_float(terms.scale), _p(terms.slopes), _p(terms.sinks),
                                      _p(gate), int(terms.logistic), _p(terms.score_bias), _p(out), _code(out.dtype),
                                      _stream()))


def scored_on_matrix_cores(dtype: torch.dtype, dk: int, dv: int) -> bool:
    """Does `attention_scored` run on the matrix cores (bfloat16, values as wide as keys, head sizes in
    steps of 16)?  Steps with several rows a sequence then take their values transposed (`vt_new`)."""
    return dtype == torch.bfloat16 and dk == dv and dk % 16 == 0 and 16 <= dk <= 256


def _terms_args(terms: ScoreTerms, gate, n: int, nq: int):
    if terms.slopes is not None:
        _req(terms.slopes, "attn_scored.slopes", torch.float32, (nq,))
    if terms.sinks is not None:
        _req(terms.sinks, "attn_scored.sinks", torch.float32, (nq,))
    if gate is not None:
        _req(gate, "attn_scored.gate", torch.float32, (n, nq))
    if terms.score_bias is not None:
        _req(terms.score_bias, "attn_scored.score_bias", torch.float32, (nq,))
    return _p(terms.slopes), _p(terms.sinks), _p(gate)


def attention_scored(q, k_new, v_new, pages, nkv: int, dv: int, table, ring_pages: int, ctx, n_cached,
                     terms: ScoreTerms, gate, out, vt_new=None) -> None:
    """Attention with the terms of `ScoreTerms` for a step's rows: keys j < n_cached[b] from the
    pages, later ones from this step's rows (`k_new`/`v_new`; None when everything is in the
    pages).  Where `scored_on_matrix_cores`, single-token steps and steps with longer rows each run
    in the TERMS variant of the kernels of `attention` (the latter takes the step's values
    transposed, `vt_new`); everything else in the plain kernel."""
    n, nq, dk = q.shape
    fast = scored_on_matrix_cores(q.dtype, dk, dv) and pages.dim() == 5
    if fast and k_new is None and ctx.all_single:
        most_pages = table.shape[1]
        if terms.window:          # (kept first positions: the table holds every page, a row reads the window's and the kept ones)
            most_pages = min(most_pages, -(-terms.window // PAGE) + 1 + -(-int(terms.keep_first or 0) // PAGE))
        if terms.chunk:
            most_pages = min(most_pages, -(-terms.chunk // PAGE) + 1)
        splits = decode_splits(n, nq, nkv, most_pages, compute_units(q.device), dk)
        part = ctx.workspace.get("attn_part", (n * nq * splits * (dk + 2),), torch.float32)
        _decode_args(q, pages, table, ctx.row_pos, part, out, splits)
        slopes, sinks, gt = _terms_args(terms, gate, n, nq)
        _check(lib().tl_attn_decode_terms_bf16(_p(q), _p(pages), _p(table), table.shape[1], ring_pages, _p(ctx.row_pos),
                                               n, nq, nkv, dk, int(terms.window or 0), int(terms.keep_first or 0),
                                               terms.chunk, ctypes.c_float(terms.scale), int(splits), _p(part), slopes, sinks,
                                               gt, int(terms.logistic), _p(terms.score_bias), _p(out), _stream()))
    elif fast and k_new is not None and vt_new is not None:
        B = n_cached.shape[0]
        n_tiles = int(sum(-(-int(x) // PREFILL_BLOCK) for x in ctx.host["n_new"]))
        _prefill_args(q, k_new, vt_new, ctx.tile_off, pages, table, ctx.row_pos, ctx.cu_seqlens, n_cached, out)
        slopes, sinks, gt = _terms_args(terms, gate, n, nq)
        _check(lib().tl_attn_prefill_terms_bf16(_p(q), _p(k_new), _p(vt_new), vt_new.shape[2], _p(ctx.tile_off), _p(pages),
                                                _p(table), table.shape[1], ring_pages, _p(ctx.row_pos),
                                                _p(ctx.cu_seqlens), _p(n_cached), B, n_tiles, nq, nkv, dk,
                                                int(terms.window or 0), int(terms.keep_first or 0), terms.chunk,
                                                ctypes.c_float(terms.scale), slopes, sinks, gt, int(terms.logistic),
                                                _p(terms.score_bias), _p(out), _stream()))
    else:
        attn_scored_plain(q, k_new, v_new, pages, nkv, dv, table, ring_pages, ctx.row_seq, ctx.row_pos,
                          ctx.cu_seqlens, n_cached, terms, gate, out)


class ProjectionTerms:
    """What happens to a row of the fused projection [q | k | v | g] before attention: `bias`
    (float32 over the whole row, or None); `q_norm`, `k_norm` (float32 weights over ALL of q and
    ALL of k, or None): division by the root mean square of the whole projection, eps inside the
    root; `temperature` (coef, every) or None: q times 1 + coef * ln(floor((p + 1) / every) + 1)."""

    def __init__(self, bias=None, q_norm=None, k_norm=None, eps: float = 0.0, temperature=None):
        self.bias, self.q_norm, self.k_norm, self.eps = bias, q_norm, k_norm, float(eps)
        self.coef, self.every = (float(temperature[0]), float(temperature[1])) if temperature else (0.0, 1.0)


def split_projection(proj: torch.Tensor, row_pos, terms: ProjectionTerms, nq: int, nkv: int, dk: int, dv: int,
                     ng: int, q: torch.Tensor, k, v, gate, table=None, ring_pages: int = 0, pages=None) -> None:
    """proj float32 [n, nq*dk + nkv*(dk+dv) + ng] (rows may be strided: columns of a wider product) -> q [n, nq, dk], gate float32 [n, ng] (after the
    logistic function) and, with nkv > 0, k [n, nkv, dk] and v [n, nkv, dv], or, with `pages`
    (one token a sequence, row n belongs to sequence n), k and v straight into the page of the
    row's position."""
    n = proj.shape[0]
    width = nq * dk + nkv * (dk + dv) + ng
    _req(proj, "split_projection.proj", torch.float32, (n, width))
    _req(row_pos, "split_projection.row_pos", torch.int32, (n,))
    _req(q, "split_projection.q", None, (n, nq, dk))
    for t, name, size in ((terms.bias, "bias", width), (terms.q_norm, "q_norm", nq * dk), (terms.k_norm, "k_norm", nkv * dk)):
        if t is not None:
            _req(t, "split_projection." + name, torch.float32, (size,))
    if ng:
        _req(gate, "split_projection.gate", torch.float32, (n, ng))
    if nkv and pages is None:
        _req(k, "split_projection.k", q.dtype, (n, nkv, dk))
        _req(v, "split_projection.v", q.dtype, (n, nkv, dv))
    stride = 0
    if pages is not None:
        _req_pages(pages, nkv, dk, dv, "split_projection")
        _req(table, "split_projection.table", torch.int32)
        if pages.dtype != q.dtype or table.dim() != 2 or table.shape[0] != n:
            raise KernelError("split_projection: pages of q's dtype and a page table with one row per row")
        stride = table.shape[1]
    _check(lib().tl_split_projection(_p(proj), _p(row_pos), _p(terms.bias), _p(terms.q_norm), _p(terms.k_norm),
                                     ctypes.c_float(terms.eps), ctypes.c_float(terms.coef), ctypes.c_float(terms.every),
                                     n, nq, nkv, dk, dv, ng, _p(q), _p(k), _p(v), _p(gate), _code(q.dtype),
                                     _p(table), stride, int(ring_pages), _p(pages), _stream()))


def kv_commit_wide(k: torch.Tensor, v: torch.Tensor, row_seq, row_pos, len_after, table: torch.Tensor,
                   ring_pages: int, pages: torch.Tensor) -> None:
    """Rows of keys [n, nkv, dk] and values [n, nkv, dv] into the pages of their positions (values
    transposed, as the pages keep them); dk and dv need not be equal."""
    n, nkv, dk = k.shape
    dv = v.shape[2]
    _req(k, "kv_commit_wide.k", pages.dtype)
    _req(v, "kv_commit_wide.v", pages.dtype, (n, nkv, dv))
    _req_pages(pages, nkv, dk, dv, "kv_commit_wide")
    _req(row_seq, "kv_commit_wide.row_seq", torch.int32, (n,))
    _req(row_pos, "kv_commit_wide.row_pos", torch.int32, (n,))
    _req(table, "kv_commit_wide.table", torch.int32)
    _req(len_after, "kv_commit_wide.len_after", torch.int32, (table.shape[0],))
    _check(lib().tl_kv_commit_wide(_p(k), _p(v), _code(k.dtype), _p(row_seq), _p(row_pos), _p(len_after), _p(table),
                                   table.shape[1], ring_pages, n, nkv, dk, dv, _p(pages), _stream()))


def latent_norms(proj: torch.Tensor, na: int, nb: int, wa: torch.Tensor, wb: torch.Tensor, eps: float, a: torch.Tensor,
                 b: torch.Tensor, gate: Optional[torch.Tensor]) -> None:
    """proj float32 [n, na + nb + ng] = [a | b | g]: a and b each divided by their root mean square
    (eps inside the root) and multiplied by their weights (float32 [na], [nb]) into the compute dtype;
    `gate` (float32 [n, ng], or None when ng = 0) = the logistic function of g."""
    n, width = proj.shape
    ng = width - na - nb
    _req(proj, "latent_norms.proj", torch.float32)
    _req(wa, "latent_norms.wa", torch.float32, (na,))
    _req(wb, "latent_norms.wb", torch.float32, (nb,))
    _req(a, "latent_norms.a", None, (n, na))
    _req(b, "latent_norms.b", a.dtype, (n, nb))
    if ng < 0 or (ng > 0) != (gate is not None):
        raise KernelError(f"latent_norms: a row of {width} holds {na} + {nb} and {ng} gate channels; gate buffer "
                          f"{'given' if gate is not None else 'missing'}")
    if gate is not None:
        _req(gate, "latent_norms.gate", torch.float32, (n, ng))
    _check(lib().tl_latent_norms(_p(proj), n, na, nb, ng, _p(wa), _p(wb), ctypes.c_float(eps), _p(a), _p(b), _p(gate),
                                 _code(a.dtype), _stream()))


def split_heads(qf: torch.Tensor, kvf: torch.Tensor, row_pos, nq: int, nkv: int, dk: int, dv: int, q: torch.Tensor,
                k, v, table=None, ring_pages: int = 0, pages=None) -> None:
    """qf float32 [n, nq*dk] and kvf float32 [n, nkv*dk + nkv*dv] (keys of all heads, then values of all
    heads) -> q [n, nq, dk], k [n, nkv, dk] and v [n, nkv, dv] in the compute dtype; or, with `pages`
    (one token a sequence, row n belongs to sequence n), k and v straight into the page of the row's
    position."""
    n = qf.shape[0]
    _req(qf, "split_heads.qf", torch.float32, (n, nq * dk))
    _req(kvf, "split_heads.kvf", torch.float32, (n, nkv * (dk + dv)))
    _req(row_pos, "split_heads.row_pos", torch.int32, (n,))
    _req(q, "split_heads.q", None, (n, nq, dk))
    stride = 0
    if pages is None:
        _req(k, "split_heads.k", q.dtype, (n, nkv, dk))
        _req(v, "split_heads.v", q.dtype, (n, nkv, dv))
    else:
        _req_pages(pages, nkv, dk, dv, "split_heads")
        _req(table, "split_heads.table", torch.int32)
        if pages.dtype != q.dtype or table.dim() != 2 or table.shape[0] != n:
            raise KernelError("split_heads: pages of q's dtype and a page table with one row per row")
        stride = table.shape[1]
    kv = kvf.data_ptr()
    _check(lib().tl_split_heads(_p(qf), nq * dk, ctypes.c_void_p(kv), ctypes.c_void_p(kv + 4 * nkv * dk),
                                nkv * (dk + dv), _p(row_pos), n, nq, nkv, dk, dv, _p(q),
                                _p(k) if pages is None else None, _p(v) if pages is None else None, _code(q.dtype),
                                _p(table), stride, int(ring_pages), _p(pages), _stream()))


def mul_gate(x: torch.Tensor, gate: torch.Tensor) -> None:
    """x *= gate, element by element (x in the compute dtype, gate float32 of as many elements)."""
    _req(x, "mul_gate.x")
    _req(gate, "mul_gate.gate", torch.float32)
    if gate.numel() != x.numel():
        raise KernelError(f"mul_gate: {x.numel()} values and {gate.numel()} gates")
    _check(lib().tl_mul_gate(_p(x), _p(gate), ctypes.c_longlong(x.numel()), _code(x.dtype), _stream()))


def diff_split(proj: torch.Tensor, bias, row_pos, rotation, H: int, G: int, d: int, dv: int, q: torch.Tensor, k, v,
               table=None, ring_pages: int = 0, pages=None) -> None:
    """A row of the fused projection of a differential attention, float32 [n, 2*H*d + 2*G*d + G*dv] =
    [q | k | v] with two maps of d channels per head, plus `bias` (float32 over the row, or None);
    each map of q and k rotated (`rotation`: the first channels of every MAP); q laid out as 2*H heads
    of 2*d channels, map m of head h as head 2h + m with its channels in half m and zeros in the
    other; k [n, G, 2*d] and v [n, G, dv] as rows, or, with `pages` (one token a sequence), straight
    into the page of the row's position."""
    n = proj.shape[0]
    rot = _rotation(rotation, d, "diff_split")
    _req(proj, "diff_split.proj", torch.float32, (n, 2 * H * d + 2 * G * d + G * dv))
    if bias is not None:
        _req(bias, "diff_split.bias", torch.float32, (proj.shape[1],))
    _req(row_pos, "diff_split.row_pos", torch.int32, (n,))
    _req(q, "diff_split.q", None, (n, 2 * H, 2 * d))
    stride = 0
    if pages is None:
        _req(k, "diff_split.k", q.dtype, (n, G, 2 * d))
        _req(v, "diff_split.v", q.dtype, (n, G, dv))
    else:
        _req_pages(pages, G, 2 * d, dv, "diff_split")
        _req(table, "diff_split.table", torch.int32)
        if pages.dtype != q.dtype or table.dim() != 2 or table.shape[0] != n:
            raise KernelError("diff_split: pages of q's dtype and a page table with one row per row")
        stride = table.shape[1]
    if rot.interleaved:
        raise KernelError("diff_split: pairs (2i, 2i + 1) are not served, only (i, i + rotary_dim / 2)")
    _check(lib().tl_diff_split(_p(proj), _p(bias), _p(row_pos), _p(rot.inv_freq), rot.rotary_dim, n, H, G, d, dv, _p(q),
                               _p(k) if pages is None else None, _p(v) if pages is None else None, _code(q.dtype),
                               _p(table), stride, int(ring_pages), _p(pages), _stream()))


def diff_combine(att: torch.Tensor, lam: float, eps: float, post: float, out: torch.Tensor) -> None:
    """att [n, 2*H, dv] (heads 2h and 2h + 1: the two maps of head h; of out's dtype, or float32) ->
    out [n, H, dv]: o = a1 - lam * a2, then o / sqrt(mean(o^2) + eps) * post, in float32."""
    n, H2, dv = att.shape
    _req(att, "diff_combine.att")
    if H2 % 2:
        raise KernelError(f"diff_combine: {H2} maps are not pairs")
    _req(out, "diff_combine.out", None, (n, H2 // 2, dv))
    _check(lib().tl_diff_combine(_p(att), _code(att.dtype), n, H2 // 2, dv, ctypes.c_float(lam), ctypes.c_float(eps),
                                 ctypes.c_float(post), _p(out), _code(out.dtype), _stream()))


class HeadTerms:
    """What happens to a row of the fused projection [q | k | v | g] of an attention before the
    attention itself, head by head (`head_prepare`): `bias` (float32 over the whole row, or None);
    `q_norm`, `k_norm` (float32 [dk] each, or None): every head divided by its own root mean
    square (eps inside the root) times a weight that all heads share; `mix`: 0, or 1 (the values
    are left, unrounded, for later layers) or 2 (v <- (1 - lam) v + lam * the values that were left);
    `unit_norm`: instead of the weighted norm, every head of q and of k is divided by its root mean
    square (the same eps) AFTER the rotation, with no weight; `v_factor` multiplies the (biased) values."""

    def __init__(self, bias=None, q_norm=None, k_norm=None, eps: float = 0.0, mix: int = 0, lam: float = 0.0,
                 unit_norm: bool = False, v_factor: float = 1.0):
        self.bias, self.q_norm, self.k_norm, self.eps = bias, q_norm, k_norm, float(eps)
        self.mix, self.lam = int(mix), float(lam)
        self.unit_norm = bool(unit_norm)
        self.v_factor = float(v_factor)


def head_prepare(proj: torch.Tensor, row_pos, rotation, terms: HeadTerms, nq: int, nkv: int, dk: int, dv: int, ng: int,
                 q: torch.Tensor, k, v, gate, v_first=None, table=None, ring_pages: int = 0, pages=None) -> None:
    """proj float32 [n, nq*dk + nkv*(dk+dv) + ng] (rows may be strided: columns of a wider product) -> q [n, nq, dk] (biased, normed per head, rotated),
    `gate` float32 [n, ng] (after the logistic function) and k [n, nkv, dk] and v [n, nkv, dv], or,
    with `pages` (one token a sequence, row n belongs to sequence n), k and v straight into the
    page of the row's position.  `v_first` (float32 [n, nkv*dv]): where a layer that mixes values
    leaves or finds the first such layer's.  nkv 0: the row holds [q | g] alone (a mixer that reads
    another's keys and values)."""
    n = proj.shape[0]
    width = nq * dk + nkv * (dk + dv) + ng
    rot = _rotation(rotation, dk, "head_prepare")
    if rot.interleaved:
        raise KernelError("head_prepare: pairs (2i, 2i + 1) are not served, only (i, i + rotary_dim / 2)")
    _req_columns(proj, (n, width), "head_prepare.proj")
    _req(row_pos, "head_prepare.row_pos", torch.int32, (n,))
    _req(q, "head_prepare.q", None, (n, nq, dk))
    for t, name, size in ((terms.bias, "bias", width), (terms.q_norm, "q_norm", dk), (terms.k_norm, "k_norm", dk)):
        if t is not None:
            _req(t, "head_prepare." + name, torch.float32, (size,))
    if ng:
        _req(gate, "head_prepare.gate", torch.float32, (n, ng))
    if terms.mix:
        if v_first is None:
            raise KernelError("head_prepare: mixing values needs the buffer they are left in")
        _req(v_first, "head_prepare.v_first", torch.float32, (n, nkv * dv))
    stride = 0
    if nkv == 0:
        pages = k = v = None
    elif pages is None:
        _req(k, "head_prepare.k", q.dtype, (n, nkv, dk))
        _req(v, "head_prepare.v", q.dtype, (n, nkv, dv))
    else:
        _req_pages(pages, nkv, dk, dv, "head_prepare")
        _req(table, "head_prepare.table", torch.int32)
        if pages.dtype != q.dtype or table.dim() != 2 or table.shape[0] != n:
            raise KernelError("head_prepare: pages of q's dtype and a page table with one row per row")
        stride = table.shape[1]
    _check(lib().tl_head_prepare(_p(proj), proj.stride(0), _p(row_pos), _p(rot.inv_freq), rot.rotary_dim, _p(terms.bias), _p(terms.q_norm),
                                 _p(terms.k_norm), ctypes.c_float(terms.eps), int(terms.unit_norm), terms.mix,
                                 ctypes.c_float(terms.lam), ctypes.c_float(terms.v_factor),
                                 _p(v_first) if terms.mix else None, n, nq, nkv, dk, dv, ng, _p(q),
                                 _p(k) if pages is None else None, _p(v) if pages is None else None, _p(gate),
                                 _code(q.dtype), _p(table), stride, int(ring_pages), _p(pages), _stream()))


# ---- the state-space mixer ---------------------------------------------------------------------------
def ssm_conv(proj: torch.Tensor, off: int, C: int, w: torch.Tensor, bias, conv_state: torch.Tensor, row_seq, cu_seqlens,
             slots, out: torch.Tensor, single: bool = False) -> None:
    """The short causal convolution of a state-space mixer over the columns off .. off + C - 1 of proj
    (float32 [n, width]) and silu: out[n, c] = silu(bias[c] + sum_j w[c, j] * u[row - (taps - 1 - j), c]).  Rows
    before the step come from the sequence's block `conv_state` [slots, >= (taps - 1) * C] (float32, the
    oldest row first, zeros before the start), which afterwards holds the step's last taps - 1 inputs.  `single`: every
    sequence brings one row (row b is sequence b's): one pass does both."""
    n, width = proj.shape
    taps = w.shape[1]
    B = slots.shape[0]
    _req(proj, "ssm_conv.proj", torch.float32)
    _req(w, "ssm_conv.w", torch.float32, (C, taps))
    if bias is not None:
        _req(bias, "ssm_conv.bias", torch.float32, (C,))
    if conv_state.dtype != torch.float32 or conv_state.dim() != 2 or conv_state.stride(1) != 1 or not conv_state.is_cuda:
        raise KernelError("ssm_conv.conv_state: float32 [slots, block] on the GPU, rows may be strided")
    _req(row_seq, "ssm_conv.row_seq", torch.int32, (n,))
    _req(cu_seqlens, "ssm_conv.cu_seqlens", torch.int32, (B + 1,))
    _req(slots, "ssm_conv.slots", torch.int32)
    _req(out, "ssm_conv.out", None, (n, C))
    if conv_state.shape[1] < (taps - 1) * C:
        raise KernelError(f"ssm_conv: a block of {conv_state.shape[1]} for {taps - 1} rows of {C}")
    _check(lib().tl_ssm_conv(_p(proj), width, int(off), int(C), _p(w), _p(bias), taps, _p(conv_state),
                             ctypes.c_longlong(conv_state.stride(0)), _p(row_seq), _p(cu_seqlens), _p(slots), n, B, int(bool(single)),
                             _p(out), _code(out.dtype), _stream()))


def ssm_scan(u: torch.Tensor, proj: torch.Tensor, dt_off: int, G: int, N: int, heads: int, dv: int, dt_bias, A_log, D,
             state: torch.Tensor, cu_seqlens, slots, y: torch.Tensor) -> None:
    """The recurrence of a state-space mixer over the rows of a step, sequence by sequence: u [n, heads*dv + 2*G*N]
    = [x | B | C] (after the convolution), dt at the columns dt_off .. of proj (float32 [n, width]);
    dt' = softplus(dt + dt_bias[h]), S <- exp(-exp(A_log[h]) dt') S + dt' B x^T, y = S^T C + D[h] x; `state`
    float32 [slots, >= heads*N*dv] is read and left updated; y float32 [n, heads*dv]."""
    n, C = u.shape
    B = slots.shape[0]
    _req(u, "ssm_scan.u")
    _req(proj, "ssm_scan.proj", torch.float32)
    for t, name in ((dt_bias, "dt_bias"), (A_log, "A_log"), (D, "D")):
        _req(t, "ssm_scan." + name, torch.float32, (heads,))
    if state.dtype != torch.float32 or state.dim() != 2 or state.stride(1) != 1 or not state.is_cuda:
        raise KernelError("ssm_scan.state: float32 [slots, block] on the GPU, rows may be strided")
    if state.shape[1] < heads * N * dv or proj.shape[0] != n:
        raise KernelError(f"ssm_scan: a block of {state.shape[1]} for a state of {heads} x {N} x {dv}")
    _req(cu_seqlens, "ssm_scan.cu_seqlens", torch.int32, (B + 1,))
    _req(slots, "ssm_scan.slots", torch.int32)
    _req(y, "ssm_scan.y", torch.float32, (n, heads * dv))
    _check(lib().tl_ssm_scan(_p(u), _code(u.dtype), C, G, N, heads, dv, _p(proj), proj.shape[1], int(dt_off), _p(dt_bias),
                             _p(A_log), _p(D), _p(state), ctypes.c_longlong(state.stride(0)), _p(cu_seqlens), _p(slots), n, B,
                             _p(y), _stream()))


def ssm_gate_norm(y: torch.Tensor, proj: torch.Tensor, parts: int, w: torch.Tensor, eps: float, out: torch.Tensor) -> None:
    """out = rms(y * silu(z)) * w over each of `parts` equal parts of a row; y float32 [n, inner], z the first
    `inner` columns of proj (float32 [n, width]), w float32 [inner]."""
    n, inner = y.shape
    _req(y, "ssm_gate_norm.y", torch.float32)
    _req(proj, "ssm_gate_norm.proj", torch.float32)
    _req(w, "ssm_gate_norm.w", torch.float32, (inner,))
    _req(out, "ssm_gate_norm.out", None, (n, inner))
    if proj.shape[0] != n:
        raise KernelError("ssm_gate_norm: y and proj differ in rows")
    _check(lib().tl_ssm_gate_norm(_p(y), _p(proj), proj.shape[1], inner, int(parts), _p(w), ctypes.c_float(eps), n, _p(out),
                                  _code(out.dtype), _stream()))


# ---- routed experts ----------------------------------------------------------------------------------
EXPERT_ACTIVATIONS = {"relu2": 0, "relu": 1, "xielu": 2}
UNARY_CONSTANTS = {"xielu": ("a", "b")}      # activations with numbers of their own, in the kernels' order


def _unary_args(activation: str, constants):
    """Code and constants of an activation of one argument, as the kernels take them."""
    if activation not in EXPERT_ACTIVATIONS:
        raise KernelError(f"no function {activation!r}; there are {sorted(EXPERT_ACTIVATIONS)}")
    need = UNARY_CONSTANTS.get(activation, ())
    if set(constants or {}) != set(need):
        raise KernelError(f"{activation!r} takes the constants {sorted(need)}, got {sorted(constants or {})}")
    k = [float(constants[n]) for n in need] + [0.0] * (2 - len(need))
    return EXPERT_ACTIVATIONS[activation], ctypes.c_float(k[0]), ctypes.c_float(k[1])


def _shared_weight(w: Optional[torch.Tensor], n: int, what: str):
    if w is not None:
        _req(w, what + ".shared_weight", torch.float32, (n,))
    return _p(w)


def route(h: torch.Tensor, router: torch.Tensor, groups: int, keep: int, top: int, weights: torch.Tensor,
          chosen: Optional[torch.Tensor] = None, logistic: bool = False, correction: Optional[torch.Tensor] = None,
          two_largest: bool = False, normalise_eps: Optional[float] = None,
          shared_weight: Optional[torch.Tensor] = None, bias: Optional[torch.Tensor] = None) -> None:
    """The router of a mixture of experts, in float32: s = softmax(router h (+ `bias`, float32 [E])) over the E experts (`logistic`:
    every expert's own 1 / (1 + exp(-router h)) instead).  The choice goes by c = s (+ `correction`, float32 [E]):
    of the `keep` groups (of `groups` equal groups of neighbours; 0: no groups) whose best c is largest
    (`two_largest`: the sum of whose two best is), the `top` experts with the largest c; `weights` float32
    [n, E] receives s for those (with `normalise_eps`: divided by (their sum + normalise_eps)) and 0 for the
    others, `chosen` (int32 [n, top], or None) their indices, the best first.  With `shared_weight` (float32
    [n]) the router has one row more, whose product's logistic function goes there."""
    n, W = h.shape
    E = weights.shape[1]
    _req(h, "route.h")
    _req(router, "route.router", torch.float32, (E + (1 if shared_weight is not None else 0), W))
    _req(weights, "route.weights", torch.float32, (n, E))
    if chosen is not None:
        _req(chosen, "route.chosen", torch.int32, (n, top))
    if correction is not None:
        _req(correction, "route.correction", torch.float32, (E,))
    if bias is not None:
        _req(bias, "route.bias", torch.float32, (E,))
    _check(lib().tl_route(_p(h), _code(h.dtype), n, W, _p(router), E, int(groups), int(keep), int(top), int(bool(logistic)),
                          _p(correction), int(bool(two_largest)), int(normalise_eps is not None),
                          ctypes.c_float(normalise_eps or 0.0), _shared_weight(shared_weight, n, "route"), _p(bias),
                          _p(weights), _p(chosen), _stream()))


class GateTerms:
    """The constants of a gated expert, act(g, u) = g' logistic(alpha g') (u' + shift) with g' = min(g, limit) and
    u' = clamp(u, -limit, limit); the shared expert has a limit of its own (`limit_shared`; None: the same).
    `on_input`: the router's weight multiplies the expert's input (g and u before the clamps) instead of its output.
    Limits of infinity, alpha 1 and shift 0 make it silu(g) u."""

    def __init__(self, limit: float, alpha: float, shift: float, limit_shared: Optional[float] = None, on_input: bool = False):
        self.limit, self.alpha, self.shift = float(limit), float(alpha), float(shift)
        self.limit_shared = self.limit if limit_shared is None else float(limit_shared)
        self.on_input = bool(on_input)

    def args(self):
        return (ctypes.c_float(self.limit), ctypes.c_float(self.limit_shared), ctypes.c_float(self.alpha),
                ctypes.c_float(self.shift), int(self.on_input))


def expert_gated_act(gu: torch.Tensor, weights: Optional[torch.Tensor], E: int, ff: int, shared: int, terms: GateTerms,
                     out: torch.Tensor, shared_weight: Optional[torch.Tensor] = None) -> None:
    """The activations of gated experts laid side by side: gu float32 [n, 2 (E ff + shared)] holds, expert after
    expert, [gate (ff) | up (ff)] and behind them the shared expert's [gate (shared) | up (shared)]; out
    [n, E ff + shared] = act(g, u) with the row's weight of the column's expert (`weights` float32 [n, E]; the
    shared part has weight 1, or `shared_weight` float32 [n] on its output; E 0: no weights)."""
    n = gu.shape[0]
    total = E * ff + shared
    _req(gu, "expert_gated_act.gu", torch.float32, (n, 2 * total))
    if E:
        _req(weights, "expert_gated_act.weights", torch.float32, (n, E))
    _req(out, "expert_gated_act.out", None, (n, total))
    _check(lib().tl_expert_gated_act(_p(gu), _p(weights) if E else None, _shared_weight(shared_weight, n, "expert_gated_act"), n, int(E), int(ff), int(shared), *terms.args(),
                                     _p(out), _code(out.dtype), _stream()))


def expert_rows_gated_up(y: torch.Tensor, up: torch.Tensor, chosen: torch.Tensor, weights: torch.Tensor, ff: int, shared: int,
                         terms: GateTerms, hs: torch.Tensor, shared_weight: Optional[torch.Tensor] = None) -> None:
    """The chosen gated experts' first halves, row by row (see `expert_rows_up`): up [2 (E ff + shared), H] is the
    stacked matrix of `expert_gated_act`'s layout."""
    n, H = y.shape
    top, E = chosen.shape[1], weights.shape[1]
    _req(y, "expert_rows_gated_up.y")
    _req(up, "expert_rows_gated_up.up", y.dtype, (2 * (E * ff + shared), H))
    _req(chosen, "expert_rows_gated_up.chosen", torch.int32, (n, top))
    _req(weights, "expert_rows_gated_up.weights", torch.float32, (n, E))
    _req(hs, "expert_rows_gated_up.hs", y.dtype, (n, top * ff + shared))
    _check(lib().tl_expert_rows_gated_up(_p(y), H, _p(up), _p(chosen), _p(weights),
                                         _shared_weight(shared_weight, n, "expert_rows_gated_up"), n, E, top, int(ff), int(shared),
                                         *terms.args(), _p(hs), _code(y.dtype), _stream()))


def expert_act(u: torch.Tensor, weights: Optional[torch.Tensor], E: int, ff: int, activation: str, out: torch.Tensor,
               constants=None, shared_weight: Optional[torch.Tensor] = None) -> None:
    """out[n, j] = act(u[n, j]) * (weights[n, j // ff] for the first E * ff columns, 1 or `shared_weight[n]` for the
    rest); u float32; `constants` by name for an activation of `UNARY_CONSTANTS`."""
    n, total = u.shape
    code = _unary_args(activation, constants)
    _req(u, "expert_act.u", torch.float32)
    if E:
        _req(weights, "expert_act.weights", torch.float32, (n, E))
    _req(out, "expert_act.out", None, (n, total))
    _check(lib().tl_expert_act(_p(u), _p(weights) if E else None, _shared_weight(shared_weight, n, "expert_act"), n, int(E),
                               int(ff), total, *code,
                               _p(out), _code(out.dtype), _stream()))


def unary_act(u: torch.Tensor, activation: str, out: torch.Tensor, constants=None) -> None:
    """out = act(u) element by element (u float32, or bfloat16 like out; any number of elements that is a multiple of 8)."""
    code = _unary_args(activation, constants)
    _req(u, "unary_act.u", u.dtype if u.dtype == torch.float32 else out.dtype)
    _req(out, "unary_act.out", None, u.shape)
    _check(lib().tl_unary_act(_p(u), _code(u.dtype), ctypes.c_longlong(u.numel()), *code, _p(out), _code(out.dtype), _stream()))


def expert_rows_up(y: torch.Tensor, up: torch.Tensor, chosen: torch.Tensor, weights: torch.Tensor, ff: int, shared: int,
                   activation: str, hs: torch.Tensor, constants=None, shared_weight: Optional[torch.Tensor] = None) -> None:
    """The chosen experts' first halves, row by row: hs[n, k*ff + j] = act(up[chosen[n,k]*ff + j] . y[n]) * weights[n, chosen[n,k]]
    and, behind them, the shared expert's `shared` rows with weight 1 (or `shared_weight[n]`).  up [E*ff + shared, H] and y [n, H] of one dtype."""
    n, H = y.shape
    top, E = chosen.shape[1], weights.shape[1]
    code = _unary_args(activation, constants)
    _req(y, "expert_rows_up.y")
    _req(up, "expert_rows_up.up", y.dtype, (E * ff + shared, H))
    _req(chosen, "expert_rows_up.chosen", torch.int32, (n, top))
    _req(weights, "expert_rows_up.weights", torch.float32, (n, E))
    _req(hs, "expert_rows_up.hs", y.dtype, (n, top * ff + shared))
    _check(lib().tl_expert_rows_up(_p(y), H, _p(up), _p(chosen), _p(weights), _shared_weight(shared_weight, n, "expert_rows_up"),
                                   n, E, top, int(ff), int(shared), *code, _p(hs), _code(y.dtype), _stream()))


def expert_rows_down(hs: torch.Tensor, down: torch.Tensor, chosen: torch.Tensor, E: int, ff: int, shared: int, out: torch.Tensor,
                     accumulate: bool = False) -> None:
    """out[n] (+)= sum over the row's chosen experts (and the shared one) of their down projections of their part of
    hs [n, top*ff + shared]; down [H, E*ff + shared] of hs's dtype, out float32 [n, H]."""
    n = hs.shape[0]
    top = chosen.shape[1]
    H = down.shape[0]
    _req(hs, "expert_rows_down.hs", None, (n, top * ff + shared))
    _req(down, "expert_rows_down.down", hs.dtype, (H, E * ff + shared))
    _req(chosen, "expert_rows_down.chosen", torch.int32, (n, top))
    _req(out, "expert_rows_down.out", torch.float32, (n, H))
    _check(lib().tl_expert_rows_down(_p(hs), _p(down), _p(chosen), n, int(E), top, int(ff), int(shared), H, int(bool(accumulate)),
                                     _p(out), _code(hs.dtype), _stream()))


# ---- attention over cached latents ---------------------------------------------------------------------
LATENT_MAX_R, LATENT_MAX_ROT = 1024, 256


def _req_latent_pages(pages: torch.Tensor, D: int, dtype, what: str) -> None:
    _req(pages, what + ".pages", dtype)
    if pages.dim() < 2 or pages.numel() != pages.shape[0] * PAGE * D:
        raise KernelError(f"{what}.pages: shape {tuple(pages.shape)}, kernel needs {PAGE} rows of {D} a page")


def _req_table(table: torch.Tensor, B: int, what: str) -> int:
    _req(table, what + ".table", torch.int32)
    if table.dim() != 2 or table.shape[0] != B:
        raise KernelError(f"{what}.table: needs one row per sequence")
    return table.shape[1]


def latent_prepare(qf: torch.Tensor, cf: torch.Tensor, row_pos, rotation, H: int, dn: int, dr: int, w: torch.Tensor, eps: float,
                   qn: torch.Tensor, qr: Optional[torch.Tensor], c: Optional[torch.Tensor], rows: Optional[torch.Tensor],
                   table=None, ring_pages: int = 0, pages=None) -> None:
    """One pass over the products of an attention out of latents.  qf float32 [n, H * (dn + dr)] and cf float32
    [n, R + dr] (both may be columns of wider rows: stride(1) 1) -> qn [n, H, dn], qr [n, H, dr] (rotated;
    both may be strided views with stride(2) 1), c [n, R] = the normed latent (or None) and rows [n, R + dr] = [c | rotated
    key part] (or None), or with `pages` (one token a sequence, row n belongs to sequence n) that row straight into
    the page of its position."""
    n, R = qf.shape[0], w.shape[0]
    rot = _rotation(rotation, dr, "latent_prepare", magnitude=True)
    for t, width, name in ((qf, H * (dn + dr), "qf"), (cf, R + dr, "cf")):
        if not t.is_cuda or t.dtype != torch.float32 or t.dim() != 2 or tuple(t.shape) != (n, width) or t.stride(1) != 1:
            raise KernelError(f"latent_prepare.{name}: float32 [{n}, {width}] on the GPU, rows may be strided")
    _req(w, "latent_prepare.w", torch.float32, (R,))
    _req(row_pos, "latent_prepare.row_pos", torch.int32, (n,))
    dt = qn.dtype
    for t, width, name in ((qn, dn, "qn"),) + (((qr, dr, "qr"),) if dr else ()):
        if t is None or not t.is_cuda or t.dtype != dt or tuple(t.shape) != (n, H, width) or t.stride(2) != 1:
            raise KernelError(f"latent_prepare.{name}: [{n}, {H}, {width}] on the GPU, heads may be strided")
    if c is not None:
        _req(c, "latent_prepare.c", dt, (n, R))
    if rows is not None:
        _req(rows, "latent_prepare.rows", dt, (n, R + dr))
    stride = 0
    if pages is not None:
        _req_latent_pages(pages, R + dr, dt, "latent_prepare")
        stride = _req_table(table, n, "latent_prepare")
    L = ctypes.c_longlong
    _check(lib().tl_latent_prepare(_p(qf), qf.stride(0), _p(cf), cf.stride(0), n, H, dn, dr, R, _p(w), ctypes.c_float(eps),
                                   _p(row_pos), _p(rot.inv_freq), rot.rotary_dim, int(rot.interleaved),
                                   ctypes.c_float(rot.magnitude), _p(qn), L(qn.stride(0)), L(qn.stride(1)),
                                   _p(qr) if dr else None, L(qr.stride(0) if dr else 0), L(qr.stride(1) if dr else 0), _p(c),
                                   _p(rows), _p(pages), _p(table) if pages is not None else None, stride, int(ring_pages),
                                   _code(dt), _stream()))


def latent_commit(rows: torch.Tensor, row_seq, row_pos, len_after, table: torch.Tensor, ring_pages: int, pages: torch.Tensor) -> None:
    """Rows [n, D] into the pages of their positions."""
    n, D = rows.shape
    _req(rows, "latent_commit.rows")
    _req_latent_pages(pages, D, rows.dtype, "latent_commit")
    _req(row_seq, "latent_commit.row_seq", torch.int32, (n,))
    _req(row_pos, "latent_commit.row_pos", torch.int32, (n,))
    B = len_after.shape[0]
    _req(len_after, "latent_commit.len_after", torch.int32, (B,))
    stride = _req_table(table, B, "latent_commit")
    _check(lib().tl_latent_commit(_p(rows), _code(rows.dtype), _p(row_seq), _p(row_pos), _p(len_after), _p(table), stride,
                                  int(ring_pages), n, D, _p(pages), _stream()))


def latent_gather(pages: torch.Tensor, table: torch.Tensor, off: torch.Tensor, n_pages: int, c: torch.Tensor,
                  kr: Optional[torch.Tensor]) -> None:
    """The pages of a step's sequences one behind the other: off int32 [B + 1] is the running number of pages, of
    sequence b's the first off[b + 1] - off[b] entries of its row of `table`; c [n_pages * 64, R], kr [n_pages * 64, dr]."""
    R, dr = c.shape[1], 0 if kr is None else kr.shape[1]
    B = table.shape[0]
    _req_latent_pages(pages, R + dr, c.dtype, "latent_gather")
    stride = _req_table(table, B, "latent_gather")
    _req(off, "latent_gather.off", torch.int32, (B + 1,))
    _req(c, "latent_gather.c", None, (n_pages * PAGE, R))
    if dr:
        _req(kr, "latent_gather.kr", c.dtype, (n_pages * PAGE, dr))
    _check(lib().tl_latent_gather(_p(pages), _code(c.dtype), _p(table), stride, _p(off), B, int(n_pages), R, dr, _p(c), _p(kr),
                                  _stream()))


def latent_heads(kvf: torch.Tensor, kr: Optional[torch.Tensor], H: int, dn: int, dr: int, dv: int, k: torch.Tensor,
                 v: torch.Tensor) -> None:
    """kvf float32 [n, H * (dn + dv)] = [keys of all heads | values of all heads] and kr [n, dr] (rows may be strided) ->
    k [n, H, dn + dr] with the shared part behind every head's own, v [n, H, dv]."""
    n = kvf.shape[0]
    _req(kvf, "latent_heads.kvf", torch.float32, (n, H * (dn + dv)))
    _req(k, "latent_heads.k", None, (n, H, dn + dr))
    _req(v, "latent_heads.v", k.dtype, (n, H, dv))
    if dr and (kr.dtype != k.dtype or tuple(kr.shape) != (n, dr) or kr.stride(1) != 1 or not kr.is_cuda):
        raise KernelError(f"latent_heads.kr: [{n}, {dr}] of k's dtype on the GPU, rows may be strided")
    _check(lib().tl_latent_heads(_p(kvf), _p(kr) if dr else None, kr.stride(0) if dr else 0, n, H, dn, dr, dv, _p(k), _p(v),
                                 _code(k.dtype), _stream()))


def latent_heads_pages(kvf: torch.Tensor, kr: Optional[torch.Tensor], H: int, dn: int, dr: int, dv: int, pages: torch.Tensor) -> None:
    """`latent_heads` of gathered pages: kvf float32 [n_pages * 64, H * (dn + dv)], kr [n_pages * 64, dr] -> pages as
    `KVGroup` keeps keys and values per head."""
    n = pages.shape[0]
    _req(kvf, "latent_heads_pages.kvf", torch.float32, (n * PAGE, H * (dn + dv)))
    if dr:
        _req(kr, "latent_heads_pages.kr", pages.dtype, (n * PAGE, dr))
    _req_pages(pages, H, dn + dr, dv, "latent_heads_pages")
    _check(lib().tl_latent_heads_pages(_p(kvf), _p(kr) if dr else None, n, H, dn, dr, dv, _p(pages), _code(pages.dtype), _stream()))


def head_products(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor) -> None:
    """out[n, h] = w[h] x[n, h] for every head: x [n, H, K], w [H, N, K] and out [n, H, N] (heads may be strided) of one
    dtype, float32 sums."""
    n, H, K = x.shape
    N = w.shape[1]
    _req(x, "head_products.x")
    _req(w, "head_products.w", x.dtype, (H, N, K))
    if out.dtype != x.dtype or tuple(out.shape) != (n, H, N) or out.stride(2) != 1 or not out.is_cuda:
        raise KernelError(f"head_products.out: [{n}, {H}, {N}] of x's dtype on the GPU, heads may be strided")
    rest = (_p(x), _p(w), n, H, N, K, _p(out), ctypes.c_longlong(out.stride(0)), ctypes.c_longlong(out.stride(1)))
    if x.dtype == torch.bfloat16 and K % 8 == 0:
        _check(lib().tl_head_products_bf16(*rest, compute_units(x.device), _stream()))
    else:
        _check(lib().tl_head_products(*rest, _code(x.dtype), _stream()))


def latents_on_matrix_cores(dtype: torch.dtype, R: int, dr: int) -> bool:
    """Does `latent_attention` run on the matrix cores (bfloat16, latents up to 512 channels, rows up to 576 in steps of 8)?"""
    return dtype == torch.bfloat16 and R <= 512 and R + dr <= 576 and (R + dr) % 8 == 0


@functools.lru_cache(maxsize=4096)
def latent_splits(B: int, H: int, R: int, D: int, max_pages: int, units: int):
    """(blocks of 16 heads a workgroup, parts that the cached rows are cut into) of a single-token step, by what was
    measured (us, rows of 576 channels): 8 to start and 2.2 a page for a workgroup of one block that has a compute unit to
    itself, 4 where two share it; 11 to start and 3.3 a page with two blocks; the parts' sums 3 and what they take to be
    written and read back at 3 TB/s."""
    def cost(blocks, s):
        groups = B * -(-H // (16 * blocks)) * s
        if blocks == 2:
            start, page, at_once = 11.0, 3.3, units
        else:
            start, page, at_once = 8.0, 2.2 if groups <= units else 4.0, 2 * units
        return (start + -(-groups // at_once) * -(-max_pages // s) * page * max(D, 128) / 576.0
                + (3.0 + B * H * s * R * 8 / 3e6 if s > 1 else 0.0))

    most = max(1, min(max_pages, 4 * units // (B * -(-H // 16)) + 1, 1024))
    kinds = (1, 2) if R > 256 and D == 576 and H > 16 else (1,)
    return min(((k, s) for s in range(1, most + 1) for k in kinds), key=lambda ks: (cost(*ks), ks[1]))


def latent_attention(q: torch.Tensor, pages: torch.Tensor, table: torch.Tensor, ring_pages: int, ctx, dr: int,
                     window: Optional[int], scale: float, out: torch.Tensor) -> None:
    """Attention of one token a sequence over its cached rows [c | k_r] (its own is committed): q [B, H, R + dr] in the
    rows' channels, out [B, H, R] = the softmax-weighted sum of c."""
    B, H, D = q.shape
    R = D - dr
    _req(q, "latent_attention.q")
    _req_latent_pages(pages, D, q.dtype, "latent_attention")
    stride = _req_table(table, B, "latent_attention")
    _req(ctx.row_pos, "latent_attention.row_pos", torch.int32, (B,))
    _req(out, "latent_attention.out", q.dtype, (B, H, R))
    if latents_on_matrix_cores(q.dtype, R, dr):
        most = stride if not window else min(stride, -(-window // PAGE) + 1)
        blocks, splits = latent_splits(B, H, R, D, most, compute_units(q.device))      # by the table's width: fixed while a graph lives
        line = int(lib().tl_latent_part_line(R))
        part = ctx.workspace.get("latent_part", (B * H * splits * line,), torch.float32) if splits > 1 else None
        _check(lib().tl_latent_decode_bf16(_p(q), _p(pages), _p(table), stride, int(ring_pages), _p(ctx.row_pos), B, H, R, dr,
                                           int(window or 0), ctypes.c_float(scale), splits, blocks, _p(part), _p(out), _stream()))
        return
    _check(lib().tl_latent_attn_plain(_p(q), _p(pages), _code(q.dtype), _p(table), stride, int(ring_pages), _p(ctx.row_pos), B, H, R,
                                      dr, int(window or 0), ctypes.c_float(scale), _p(out), _stream()))


def wide_on_matrix_cores(dtype: torch.dtype, dk: int, dv: int) -> bool:
    """Does `attend_heads` run on the matrix cores (bfloat16; keys in steps of 8, values in steps of 4, up to 256)?"""
    return dtype == torch.bfloat16 and dk % 8 == 0 and 8 <= dk <= 256 and dv % 4 == 0 and 4 <= dv <= 256


def attend_heads(ctx, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, pages: torch.Tensor, table: torch.Tensor,
                 ring_pages: int, window: Optional[int], scale: float, out: torch.Tensor) -> None:
    """Attention of a step's rows over their own keys and values (k [n, H, dk], v [n, H, dv], a KV head for every query
    head) and, for cached positions, those of `pages` (flat, of the kind that `KVGroup` keeps); nothing is committed.  On
    the matrix cores where `wide_on_matrix_cores`, else in the plain kernel."""
    n, H, dk = q.shape
    dv = v.shape[2]
    if not wide_on_matrix_cores(q.dtype, dk, dv) or not scale > 0.0:
        attn_scored_plain(q, k, v, pages, H, dv, table, ring_pages, ctx.row_seq, ctx.row_pos, ctx.cu_seqlens, ctx.len_before,
                          ScoreTerms(scale, window), None, out)
        return
    B = ctx.len_before.shape[0]
    _req(q, "attend_heads.q", torch.bfloat16)
    _req(k, "attend_heads.k", torch.bfloat16, (n, H, dk))
    _req(v, "attend_heads.v", torch.bfloat16, (n, H, dv))
    _req_pages(pages, H, dk, dv, "attend_heads")
    stride = _req_table(table, B, "attend_heads")
    _req(ctx.row_pos, "attend_heads.row_pos", torch.int32, (n,))
    _req(ctx.cu_seqlens, "attend_heads.cu_seqlens", torch.int32, (B + 1,))
    _req(ctx.tile_off, "attend_heads.tile_off", torch.int32, (B,))
    _req(out, "attend_heads.out", torch.bfloat16, (n, H, dv))
    vt = ctx.workspace.get("attend_heads_vt", (H, dv, ctx.host["aligned_cols"]), q.dtype)
    v_tiles_rows(v, vt, ctx.cu_seqlens, ctx.tile_off, ctx.len_before, ctx.len_after)
    n_tiles = int(sum(-(-int(x) // PREFILL_BLOCK) for x in ctx.host["n_new"]))
    cuts = part = None
    if not ctx.host.get("fixed_launches"):       # (a captured graph's launches must not be shaped by lengths)
        at = ("prefill_cuts", window, H)
        if at not in ctx.host:                   # the same for every layer of the step
            ctx.host[at] = prefill_cuts(ctx.host["n_new"], ctx.host["len_before"], window, H, compute_units(q.device), q.device)
        cuts = ctx.host[at]
        if cuts is not None:
            part = ctx.workspace.get("attn_prefill_part", (n * H * cuts.ways * (dv + 4),), torch.float32)
    _check(lib().tl_attn_prefill_wide_bf16(_p(q), _p(k), _p(vt), vt.shape[2], _p(ctx.tile_off), _p(pages), _p(table), stride,
                                           int(ring_pages), _p(ctx.row_pos), _p(ctx.cu_seqlens), _p(ctx.len_before), B,
                                           cuts.n_items if cuts else n_tiles, H, H, dk, dv, int(window or 0),
                                           ctypes.c_float(scale), _p(out), _p(cuts.items) if cuts else None,
                                           _p(cuts.blocks) if cuts else None, cuts.n_cut if cuts else 0, _p(part),
                                           cuts.ways if cuts else 0, ctypes.c_longlong(part.numel() if cuts else 0), n, _stream()))


# ---- retention -----------------------------------------------------------------------------------------
def _req_state(state: torch.Tensor, elems: int, what: str) -> None:
    if state.dtype != torch.float32 or state.dim() != 2 or state.stride(1) != 1 or not state.is_cuda or state.shape[1] < elems:
        raise KernelError(f"{what}.state: float32 [slots, {elems} or more] on the GPU, rows may be strided")


def retention_scan(proj: torch.Tensor, row_pos, rotation, H: int, dk: int, dv: int, kscale: float, decay: torch.Tensor,
                   state: torch.Tensor, cu_seqlens, slots, o: torch.Tensor) -> None:
    """Row after row, sequence by sequence, all in float32: proj [n, width] starts with [q | k | v] (H heads of dk, dk,
    dv); q and k rotated, k times kscale; S <- decay[h] S + k v^T, o = S^T q; `state` float32 [slots, >= H*dk*dv] is read
    and left updated; o float32 [n, H*dv]."""
    n, width = proj.shape
    B = slots.shape[0]
    rot = _rotation(rotation, dk, "retention", magnitude=True)
    _req(proj, "retention.proj", torch.float32)
    _req(row_pos, "retention.row_pos", torch.int32, (n,))
    _req(decay, "retention.decay", torch.float32, (H,))
    _req_state(state, H * dk * dv, "retention")
    _req(cu_seqlens, "retention.cu_seqlens", torch.int32, (B + 1,))
    _req(slots, "retention.slots", torch.int32)
    _req(o, "retention.o", torch.float32, (n, H * dv))
    _check(lib().tl_retention_scan(_p(proj), width, H, dk, dv, _p(row_pos), _p(rot.inv_freq), rot.rotary_dim,
                                   int(rot.interleaved), ctypes.c_float(rot.magnitude), ctypes.c_float(kscale), _p(decay),
                                   _p(state), ctypes.c_longlong(state.stride(0)), _p(cu_seqlens), _p(slots), n, B, _p(o),
                                   _stream()))


def _req_columns(t: torch.Tensor, shape, what: str, dtype=torch.float32) -> None:
    """Columns of a wider matrix: rows may be strided."""
    if not t.is_cuda or t.dtype != dtype or tuple(t.shape) != tuple(shape) or t.stride(1) != 1:
        raise KernelError(f"{what}: {dtype} {list(shape)} on the GPU, rows may be strided")


def heads_norm_gate(o: torch.Tensor, gate: torch.Tensor, H: int, eps: float, out: torch.Tensor, weight: Optional[torch.Tensor] = None,
                    silu: bool = True, factor: float = 1.0) -> None:
    """out[n, h] = factor * o / sqrt(mean(o^2) + eps) * weight * silu(gate) (`silu` False: its logistic function) per head: o
    float32 [n, H*dv], gate float32 [n, H*dv] (rows may be strided: columns of the projection), weight float32 [dv] that all
    heads share (None: none), out [n, H*dv] in the compute dtype (rows may be strided)."""
    n, inner = o.shape
    _req(o, "heads_norm_gate.o", torch.float32)
    _req_columns(gate, (n, inner), "heads_norm_gate.gate")
    if weight is not None:
        _req(weight, "heads_norm_gate.weight", torch.float32, (inner // H,))
    _req_columns(out, (n, inner), "heads_norm_gate.out", out.dtype)
    _check(lib().tl_heads_norm_gate(_p(o), _p(weight), _p(gate), gate.stride(0), int(bool(silu)), n, H, inner // H, ctypes.c_float(eps),
                                    ctypes.c_float(factor), _p(out), out.stride(0), _code(out.dtype), _stream()))


def retention_norm_gate(o: torch.Tensor, gate: torch.Tensor, H: int, eps: float, out: torch.Tensor) -> None:
    """`heads_norm_gate` as retention has it: no weight, silu."""
    heads_norm_gate(o, gate, H, eps, out)


def retention_chunk() -> int:
    """Rows of a chunk of `retention_chunks`."""
    return int(lib().tl_retention_chunk())


def retention_chunks_serve(dtype: torch.dtype, dk: int, dv: int) -> bool:
    """Does `retention_chunks` take this dtype and these heads?"""
    return dtype == torch.bfloat16 and dk % 8 == 0 and 8 <= dk <= 256 and dv % 4 == 0 and 4 <= dv <= 256


def retention_chunks(proj: torch.Tensor, row_pos, rotation, H: int, dk: int, dv: int, kscale: float, log2_decay: torch.Tensor,
                     eps: float, state: torch.Tensor, cu_seqlens, slots, chunks: int, workspace, out: torch.Tensor) -> None:
    """`retention_scan` and `retention_norm_gate` of a step with many rows, by chunks of `retention_chunk()` rows on the
    matrix cores: proj float32 [n, 2 H (dk + dv)] = [q | k | v | g]; log2_decay float32 [H] (a decay of 0: a large negative
    number); `chunks`: the sequences' new rows in chunks, every sequence's rounded up, added up; `workspace` gives the
    scratch; out bfloat16 [n, H*dv]."""
    n, width = proj.shape
    B = slots.shape[0]
    rot = _rotation(rotation, dk, "retention_chunks", magnitude=True)
    _req(proj, "retention_chunks.proj", torch.float32, (n, 2 * H * (dk + dv)))
    _req(row_pos, "retention_chunks.row_pos", torch.int32, (n,))
    _req(log2_decay, "retention_chunks.log2_decay", torch.float32, (H,))
    _req_state(state, H * dk * dv, "retention_chunks")
    _req(cu_seqlens, "retention_chunks.cu_seqlens", torch.int32, (B + 1,))
    _req(slots, "retention_chunks.slots", torch.int32)
    _req(out, "retention_chunks.out", torch.bfloat16, (n, H * dv))
    if not retention_chunks_serve(out.dtype, dk, dv):
        raise KernelError(f"retention_chunks: heads of {dk} and {dv} are not served")
    C, bf, get = retention_chunk(), torch.bfloat16, workspace.get
    scratch = (get("retc_q", (n * H * dk,), bf), get("retc_k", (n * H * dk,), bf), get("retc_kt_hi", (chunks * H * dk * C,), bf),
               get("retc_kt_lo", (chunks * H * dk * C,), bf), get("retc_vt", (chunks * H * dv * C,), bf),
               get("retc_kv", (chunks * H * dk * dv,), torch.float32), get("retc_st_hi", (chunks * H * dk * dv,), bf),
               get("retc_st_lo", (chunks * H * dk * dv,), bf))
    _check(lib().tl_retention_chunks(_p(proj), width, H, dk, dv, _p(row_pos), _p(rot.inv_freq), rot.rotary_dim,
                                     int(rot.interleaved), ctypes.c_float(rot.magnitude), ctypes.c_float(kscale), _p(log2_decay),
                                     ctypes.c_float(eps), _p(state), ctypes.c_longlong(state.stride(0)), _p(cu_seqlens), _p(slots), n,
                                     B, int(chunks), *[_p(t) for t in scratch], _p(out), _stream()))


# ---- linear attention with a decay per key channel -----------------------------------------------------
class ChannelTerms:
    """How a row of a product becomes the rows of a linear attention with a decay per head and key channel: `G` heads of q and
    k, `H` of v and of the decays, sizes dk and dv; columns of beta (`b_off`, None: the plain recurrence, no delta rule), of the
    decays' inner row (`a_off`, `a_rank` channels; second matrix `a2` [H*dk, a_rank], `bias` float32 [H*dk] or None) and of the
    gate's (`g_off`, `g_rank`, `g2` [H*dv, g_rank]; None: the gate is none of this); `conv` (float32 [2*G*dk + H*dv, taps], None:
    no convolution); `rate` (float32 [H]: decays exp(-exp(rate) softplus(z)); None: logistic(z)^(1 / tau)); `qscale`; `unit_eps`
    (None: q and k are not made unit vectors)."""

    def __init__(self, G: int, H: int, dk: int, dv: int, a_off: int, a2: torch.Tensor, bias=None, b_off: Optional[int] = None,
                 g_off: Optional[int] = None, g2: Optional[torch.Tensor] = None, conv: Optional[torch.Tensor] = None,
                 rate: Optional[torch.Tensor] = None, tau: float = 1.0, qscale: float = 1.0, unit_eps: Optional[float] = None):
        self.G, self.H, self.dk, self.dv = int(G), int(H), int(dk), int(dv)
        self.a_off, self.a2, self.bias, self.b_off, self.g_off, self.g2 = int(a_off), a2, bias, b_off, g_off, g2
        self.conv, self.rate, self.inv_tau, self.qscale, self.unit_eps = conv, rate, 1.0 / float(tau), float(qscale), unit_eps

    @property
    def channels(self) -> int:
        """The columns [q | k | v] that a convolution covers."""
        return 2 * self.G * self.dk + self.H * self.dv

    @property
    def taps(self) -> int:
        return 0 if self.conv is None else int(self.conv.shape[1])

    def check(self, what: str) -> None:
        _req(self.a2, what + ".a2", None, (self.H * self.dk, self.a2.shape[1]))
        if self.g2 is not None:
            _req(self.g2, what + ".g2", self.a2.dtype, (self.H * self.dv, self.g2.shape[1]))
        if self.bias is not None:
            _req(self.bias, what + ".bias", torch.float32, (self.H * self.dk,))
        if self.rate is not None:
            _req(self.rate, what + ".rate", torch.float32, (self.H,))
        if self.conv is not None:
            _req(self.conv, what + ".conv", torch.float32, (self.channels, self.taps))


def channel_rows(proj: torch.Tensor, t: ChannelTerms, conv_state, row_seq, cu_seqlens, slots, single: bool, q, k, v, decay, beta,
                 gate) -> None:
    """proj float32 [n, width] (rows may be strided) = [q | k | v | ...] -> q, k float32 [n, G*dk], v [n, H*dv], decay [n, H*dk]
    (factors between 0 and 1), beta [n, H] (with the delta rule) and gate [n, H*dv] (second step of its projection, where the
    terms have one): see `ChannelTerms`.  `conv_state` (float32 [slots, >= (taps - 1) * channels]): the convolution's last
    inputs, read and left updated."""
    n, width = proj.shape
    B = slots.shape[0]
    _req_columns(proj, (n, width), "channel_rows.proj")
    t.check("channel_rows")
    for x, name, size in ((q, "q", t.G * t.dk), (k, "k", t.G * t.dk), (v, "v", t.H * t.dv), (decay, "decay", t.H * t.dk),
                          (beta, "beta", t.H), (gate, "gate", t.H * t.dv)):
        if (name == "beta" and t.b_off is None) or (name == "gate" and t.g2 is None):
            continue
        _req(x, "channel_rows." + name, torch.float32, (n, size))
    if t.taps:
        _req_state(conv_state, (t.taps - 1) * t.channels, "channel_rows")
        _req(row_seq, "channel_rows.row_seq", torch.int32, (n,))
    _req(cu_seqlens, "channel_rows.cu_seqlens", torch.int32, (B + 1,))
    _req(slots, "channel_rows.slots", torch.int32)
    if proj.shape[1] < t.channels:
        raise KernelError(f"channel_rows: rows of {width} for {t.channels} channels")
    _check(lib().tl_channel_rows(_p(proj), proj.stride(0), t.G, t.H, t.dk, t.dv, -1 if t.b_off is None else int(t.b_off), t.a_off,
                                 t.a2.shape[1], 0 if t.g2 is None else int(t.g_off), 0 if t.g2 is None else t.g2.shape[1], t.taps,
                                 _p(t.conv), _p(t.bias), _p(t.rate), ctypes.c_float(t.inv_tau), ctypes.c_float(t.qscale),
                                 ctypes.c_float(-1.0 if t.unit_eps is None else t.unit_eps), _p(t.a2), _p(t.g2), _code(t.a2.dtype),
                                 _p(conv_state), ctypes.c_longlong(conv_state.stride(0) if t.taps else 0), _p(row_seq),
                                 _p(cu_seqlens), _p(slots), n, B, int(bool(single)), _p(q), _p(k), _p(v), _p(decay), _p(beta),
                                 _p(gate), _stream()))
    if t.taps > 1 and not single:
        conv_carry(proj, 0, t.channels, t.taps, conv_state, cu_seqlens, slots)


def conv_carry(proj: torch.Tensor, off: int, C: int, taps: int, conv_state: torch.Tensor, cu_seqlens, slots) -> None:
    """Keep the last taps - 1 rows of the columns off .. off + C - 1 of every sequence's rows in its block (older ones shifted
    down where a step brings fewer)."""
    _check(lib().tl_conv_carry(_p(proj), proj.stride(0), int(off), int(C), int(taps), _p(conv_state),
                               ctypes.c_longlong(conv_state.stride(0)), _p(cu_seqlens), _p(slots), slots.shape[0], _stream()))


def _channel_scan(q, k, v, decay, beta, t: ChannelTerms, state, cu_seqlens, slots, o, weight, gate, silu, eps, factor, out) -> None:
    n, B = q.shape[0], slots.shape[0]
    for x, name, size in ((q, "q", t.G * t.dk), (k, "k", t.G * t.dk), (v, "v", t.H * t.dv), (decay, "decay", t.H * t.dk)):
        _req(x, "channel_scan." + name, torch.float32, (n, size))
    if t.b_off is not None:
        _req(beta, "channel_scan.beta", torch.float32, (n, t.H))
    _req_state(state, t.H * t.dk * t.dv, "channel_scan")
    _req(cu_seqlens, "channel_scan.cu_seqlens", torch.int32, (B + 1,))
    _req(slots, "channel_scan.slots", torch.int32)
    _check(lib().tl_channel_scan(_p(q), _p(k), _p(v), _p(decay), _p(beta) if t.b_off is not None else None, t.G, t.H, t.dk, t.dv,
                                 _p(state), ctypes.c_longlong(state.stride(0)), _p(cu_seqlens), _p(slots), n, B, _p(o), _p(weight),
                                 _p(gate), gate.stride(0) if gate is not None else 0, int(bool(silu)), ctypes.c_float(eps),
                                 ctypes.c_float(factor), _p(out), out.stride(0) if out is not None else 0,
                                 _code(out.dtype) if out is not None else DT_F32, _stream()))


def channel_scan(q, k, v, decay, beta, t: ChannelTerms, state: torch.Tensor, cu_seqlens, slots, o: torch.Tensor) -> None:
    """The recurrence row after row, sequence by sequence, all in float32, over what `channel_rows` made: `state` float32
    [slots, >= H*dv*dk] (a head's state column by column) is read and left updated; o float32 [n, H*dv]."""
    _req(o, "channel_scan.o", torch.float32, (q.shape[0], t.H * t.dv))
    _channel_scan(q, k, v, decay, beta, t, state, cu_seqlens, slots, o, None, None, True, 0.0, 1.0, None)


def channel_scan_gated(q, k, v, decay, beta, t: ChannelTerms, state: torch.Tensor, cu_seqlens, slots, gate: torch.Tensor, eps: float,
                       out: torch.Tensor, weight=None, silu: bool = True, factor: float = 1.0) -> None:
    """`channel_scan` and `heads_norm_gate` of a step in which every sequence brings one row (row b is sequence b's), in one
    kernel."""
    n, inner = q.shape[0], t.H * t.dv
    _req_columns(gate, (n, inner), "channel_scan.gate")
    _req_columns(out, (n, inner), "channel_scan.out", out.dtype)
    if weight is not None:
        _req(weight, "channel_scan.weight", torch.float32, (t.dv,))
    _channel_scan(q, k, v, decay, beta, t, state, cu_seqlens, slots, None, weight, gate, silu, eps, factor, out)


def channel_chunk() -> int:
    """Rows of a chunk of `channel_chunks`."""
    return int(lib().tl_channel_chunk())


def channel_chunks_serve(dtype: torch.dtype, dk: int, dv: int) -> bool:
    """Does `channel_chunks` take this dtype and these heads?"""
    return dtype == torch.bfloat16 and 1 <= dk <= 128 and 1 <= dv <= 256


def channel_chunks(proj: torch.Tensor, t: ChannelTerms, z: torch.Tensor, conv_state, state: torch.Tensor, cu_seqlens, slots, chunks: int,
                   workspace, gate: torch.Tensor, eps: float, out: torch.Tensor, weight=None, silu: bool = True, factor: float = 1.0) -> None:
    """`channel_rows`, `channel_scan` and `heads_norm_gate` of a step with many rows, by chunks of `channel_chunk()` rows on the
    matrix cores: proj as there; z float32 [n, H*dk] = the second step of the decays' projection without its bias; gate float32
    [n, H*dv] (rows may be strided); `chunks`: the sequences' new rows in chunks, every sequence's rounded up, added up;
    `workspace` gives the scratch; out bfloat16 [n, H*dv] (rows may be strided)."""
    n, width = proj.shape
    B = slots.shape[0]
    _req_columns(proj, (n, width), "channel_chunks.proj")
    t.check("channel_chunks")
    _req(z, "channel_chunks.z", torch.float32, (n, t.H * t.dk))
    _req_state(state, t.H * t.dk * t.dv, "channel_chunks")
    if t.taps:
        _req_state(conv_state, (t.taps - 1) * t.channels, "channel_chunks")
    _req(cu_seqlens, "channel_chunks.cu_seqlens", torch.int32, (B + 1,))
    _req(slots, "channel_chunks.slots", torch.int32)
    _req_columns(gate, (n, t.H * t.dv), "channel_chunks.gate")
    _req_columns(out, (n, t.H * t.dv), "channel_chunks.out", torch.bfloat16)
    if weight is not None:
        _req(weight, "channel_chunks.weight", torch.float32, (t.dv,))
    if width < t.channels or not channel_chunks_serve(torch.bfloat16, t.dk, t.dv):
        raise KernelError(f"channel_chunks: heads of {t.dk} and {t.dv} in rows of {width} are not served")
    delta = t.b_off is not None
    rec = workspace.get("chunk_rec", (chunks * t.H * int(lib().tl_channel_record(t.dk, int(delta))),), torch.bfloat16)
    gam = workspace.get("chunk_gam", (chunks * t.H * int(lib().tl_channel_padded(t.dk)),), torch.float32)
    uf = workspace.get("chunk_u", (chunks * t.H * -(-t.dv // 16) * 1024,), torch.float32)
    su = workspace.get("chunk_su", (chunks * t.H * -(-t.dv // 16) * int(lib().tl_channel_carried(t.dk)),), torch.bfloat16)
    _check(lib().tl_channel_chunks(_p(proj), proj.stride(0), t.G, t.H, t.dk, t.dv, int(t.b_off) if delta else -1, t.taps, _p(t.conv),
                                   _p(t.bias), _p(t.rate), ctypes.c_float(t.inv_tau), ctypes.c_float(t.qscale),
                                   ctypes.c_float(-1.0 if t.unit_eps is None else t.unit_eps), _p(z), _p(conv_state),
                                   ctypes.c_longlong(conv_state.stride(0) if t.taps else 0), _p(state),
                                   ctypes.c_longlong(state.stride(0)), _p(cu_seqlens), _p(slots), n, B, int(chunks), _p(rec), _p(gam),
                                   _p(uf), _p(su), _p(weight), _p(gate), gate.stride(0), int(bool(silu)), ctypes.c_float(eps),
                                   ctypes.c_float(factor), _p(out), out.stride(0), _stream()))
    if t.taps > 1:
        conv_carry(proj, 0, t.channels, t.taps, conv_state, cu_seqlens, slots)


def split_columns(x: torch.Tensor, pad: int, out: torch.Tensor) -> None:
    """x float32 [n, cols] (rows may be strided) as two bfloat16 terms, x = hi + lo, side by side: out bfloat16 [n, 2 * pad] =
    [hi | zeros | lo | zeros].  Times [W | W] it gives the product of 16 bits of x's mantissa."""
    n, cols = x.shape
    _req_columns(x, (n, cols), "split_columns.x")
    _req(out, "split_columns.out", torch.bfloat16, (n, 2 * pad))
    _check(lib().tl_split_columns(_p(x), x.stride(0), cols, int(pad), n, _p(out), _stream()))


def take_tokens(src: torch.Tensor, idx: torch.Tensor, vocab: int, tokens: torch.Tensor) -> None:
    """tokens[j] = src[idx[j]] (int32, on the device); ids outside [0, vocab) become 0."""
    n = tokens.shape[0]
    _req(src, "take_tokens.src", torch.int32)
    _req(idx, "take_tokens.idx", torch.int32, (n,))
    _req(tokens, "take_tokens.tokens", torch.int32, (n,))
    _check(lib().tl_take_tokens(_p(src), _p(idx), n, src.numel(), int(vocab), _p(tokens), _stream()))


def gather_rows(x: torch.Tensor, idx: torch.Tensor, out: torch.Tensor) -> None:
    m, H = idx.shape[0], x.shape[1]
    _req(x, "gather.x", torch.float32)
    _req(idx, "gather.idx", torch.int32, (m,))
    _req(out, "gather.out", torch.float32, (m, H))
    _check(lib().tl_gather_rows(_p(x), _p(idx), m, H, _p(out), _stream()))


def gemm_plain(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor, accumulate: bool = False) -> None:
    """out[M,N] (+)= a[M,K] @ w[N,K]^T, float32 accumulation in plain FMA."""
    M, K = a.shape
    N = w.shape[0]
    _req(a, "gemm.a")
    _req(w, "gemm.w", None, (N, K))
    _req(out, "gemm.out", torch.float32, (M, N))
    _check(lib().tl_gemm_plain(_p(a), _code(a.dtype), _p(w), _code(w.dtype), _p(out), M, N, K, K, K, N,
                               int(accumulate), _stream()))


def sample(logits: torch.Tensor, temperature: float, top_k: int, top_p: float, seed: int,
           counters: torch.Tensor, probs: torch.Tensor, out: torch.Tensor) -> None:
    """One token per row.  counters[b] = (sequence, step) feeds the generator;
    probs receives the distribution the draw was made from (when T > 0)."""
    B, V = logits.shape
    _req(logits, "sample.logits", torch.float32)
    _req(counters, "sample.counters", torch.int32, (B, 2))
    _req(probs, "sample.probs", torch.float32, (B, V))
    _req(out, "sample.out", torch.int32, (B,))
    _check(lib().tl_sample(_p(logits), B, V, ctypes.c_float(temperature), int(top_k),
                           ctypes.c_float(top_p), ctypes.c_ulonglong(seed & (2 ** 64 - 1)),
                           _p(counters), _p(probs), _p(out), _stream()))


EPI_STORE, EPI_ACCUMULATE, EPI_SILU_PAIR, EPI_GELU_PAIR = 0, 1, 2, 3


EPI_SWISH_CLAMPED_PAIR = 4
EPI_RELU_PAIR = 5
PAIR_EPILOGUES = {"silu": EPI_SILU_PAIR, "gelu_tanh": EPI_GELU_PAIR, "swish_clamped": EPI_SWISH_CLAMPED_PAIR,
                  "relu": EPI_RELU_PAIR}


def _pair_epilogue(pair_act, constants=None) -> int:
    """The code of the paired epilogue act(gate) * up for the gate's function `pair_act`: a name of
    `PAIR_EPILOGUES`, or (name, constants) for a function that has some.  The constants are handed to the
    library for the launches that follow on this thread (each launch carries them by value)."""
    if isinstance(pair_act, tuple):
        pair_act, constants = pair_act
    if pair_act not in PAIR_EPILOGUES:
        raise KernelError(f"paired epilogue: no function {pair_act!r}; there are {sorted(PAIR_EPILOGUES)}")
    k = _act_constants(pair_act, constants)
    if pair_act in ACTIVATION_CONSTANTS:
        _check(lib().tl_pair_constants(*k))
    return PAIR_EPILOGUES[pair_act]


def tiles_fit(N: int, K: int) -> bool:
    """Can a weight [N, K] have a tiled copy?"""
    return N % 16 == 0 and K % 64 == 0


def tile_height(N: int) -> int:
    """Rows of a tile of the tiled copy of a weight with N rows: the channels that a workgroup of the
    products for at most 16 rows owns (16; more where the device has fewer compute units than the
    weight has tiles of 16, so that the units get equal shares)."""
    return int(lib().tl_tile_height(int(N)))


def tile_weights(w: torch.Tensor, rows: Optional[torch.Tensor] = None, height: Optional[int] = None) -> torch.Tensor:
    """The copy of w [N, K] (bfloat16, N % 16 == 0, K % 64 == 0) that the products for at most
    16 rows stream from: [ceil(N / R), K/64, 2, 4, R, 8] with element (T, s, c, g, r, e) =
    w[rows[R T + r], 64 s + 16 g + 8 c + e], so that what a workgroup reads is one run of memory (and
    with R = 16 what a wave loads at a time, lane after lane).  `rows` (int32 [N], on the device): a
    permutation of the rows; None: none.  `height`: R; None: `tile_height(N)`, or 16 with `rows`
    (the kernel that wants its own order reads tiles of 16).  Places of the last tile behind row N are
    zero."""
    N, K = w.shape
    _req(w, "tile_weights.w", torch.bfloat16)
    if not tiles_fit(N, K):
        raise KernelError(f"tile_weights: N={N} must be a multiple of 16 and K={K} of 64")
    if rows is not None:
        _req(rows, "tile_weights.rows", torch.int32, (N,))
    R = int(height) if height is not None else (16 if rows is not None else tile_height(N))
    if not 16 <= R <= 32:
        raise KernelError(f"tile_weights: tiles of {R} rows (16 to 32)")
    n_tiles = -(-N // R)
    make = torch.empty if n_tiles * R == N else torch.zeros
    out = make((n_tiles, K // 64, 2, 4, R, 8), dtype=torch.bfloat16, device=w.device)
    _check(lib().tl_tile_weights(_p(w), _p(rows), N, K, R, _p(out), _stream()))
    return out


def qkv_tile_rows(nq: int, nkv: int, d: int, device, rotation=None) -> torch.Tensor:
    """The order of the rows of w = q|k|v in the tiled copy that `qkv_rope_commit` reads
    (a tile of a q or k head holds both channels of 8 pairs of `rotation`; None: the whole
    head rotated in halves)."""
    n = (nq + 2 * nkv) * d
    buf = (ctypes.c_int * n)()
    rotary_dim, interleaved = (d, False) if rotation is None else (rotation.rotary_dim, rotation.interleaved)
    _check(lib().tl_qkv_tile_rows(int(nq), int(nkv), int(d), int(rotary_dim), int(interleaved), buf))
    return torch.tensor(list(buf), dtype=torch.int32, device=device)


def _req_tiles(tiles: Optional[torch.Tensor], N: int, K: int, height: Optional[int] = None) -> int:
    """Check a tiled copy of a weight [N, K] (`height`: the only tile height the caller reads) and
    return its tile height (16 where there is no copy)."""
    if tiles is None:
        return 16
    if not tiles_fit(N, K):
        raise KernelError(f"gemm.tiles: a weight [{N}, {K}] has no tiled copy")
    R = int(tiles.shape[4]) if tiles.dim() == 6 else 0
    if R < 16 or (height is not None and R != height):
        raise KernelError(f"gemm.tiles: shape {tuple(tiles.shape)} is no tiled copy"
                          + (f" with tiles of {height} rows" if height is not None else ""))
    _req(tiles, "gemm.tiles", torch.bfloat16, (-(-N // R), K // 64, 2, 4, R, 8))
    return R


def gemm_bf16(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor, accumulate: bool = False,
              variant: Optional[int] = None, silu_pair: bool = False,
              tiles: Optional[torch.Tensor] = None, pair_act: str = "silu") -> None:
    """out[M,N] (+)= a[M,K] @ w[N,K]^T on the matrix cores: bfloat16 operands,
    float32 accumulation.  K must be a multiple of 8.  With `silu_pair`, w's
    rows come in groups of 64 (32 gate rows and the 32 up rows that belong to
    them) and out is bfloat16 [M, N/2] = silu(gate) * up.  `variant` (tests
    and tuning) forces one kernel.  `tiles`: `tile_weights(w)`, read instead of
    w by the kernel for at most 16 rows and 16 to 32 channels a workgroup."""
    M, K = a.shape
    N = w.shape[0]
    _req(a, "gemm.a", torch.bfloat16)
    _req(w, "gemm.w", torch.bfloat16, (N, K))
    th = _req_tiles(tiles, N, K)
    if silu_pair:
        if accumulate or N % 64:
            raise KernelError("gemm: the paired epilogue stores, and needs N to be a multiple of 64")
        _req(out, "gemm.out", torch.bfloat16, (M, N // 2))
        epi = _pair_epilogue(pair_act)
    else:
        _req(out, "gemm.out", torch.float32, (M, N))
        epi = EPI_ACCUMULATE if accumulate else EPI_STORE
    if variant is None:
        _check(lib().tl_gemm_bf16(_p(a), _p(w), _p(tiles), th, _p(out), M, N, K, epi, _stream()))
    else:
        _check(lib().tl_gemm_bf16_variant(_p(a), _p(w), _p(out), M, N, K, epi, int(variant), _stream()))


class RowFactor:
    """The second half of an RMSNorm cut in two around a product: sums of x^2 per
    workgroup of the product that wrote the stream (`ssq` [16, n_part], float32), from
    which the reading product makes rsqrt(sum / size + eps) per row."""

    def __init__(self, ssq: torch.Tensor, n_part: int, size: int, eps: float):
        self.ssq, self.n_part, self.size, self.eps = ssq, int(n_part), int(size), float(eps)


def norm_split_ok(a: torch.Tensor, w: torch.Tensor) -> bool:
    """Can `gemm_bf16_norm` take this product (bfloat16, at most 16 rows)?"""
    return bf16_gemm_ok(a, w) and a.shape[0] <= 16


def gemm_bf16_norm(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor, accumulate: bool = False,
                   silu_pair: bool = False, factor: Optional[RowFactor] = None,
                   norm_weight: Optional[torch.Tensor] = None, xt: Optional[torch.Tensor] = None,
                   ssq_out: Optional[torch.Tensor] = None, tiles: Optional[torch.Tensor] = None, pair_act: str = "silu") -> int:
    """`gemm_bf16` for at most 16 rows with the halves of an RMSNorm around it.
    `factor`: every row of the result is multiplied by its rsqrt(mean(x^2) + eps).
    `norm_weight`, `xt`, `ssq_out` (with `accumulate`): out += product, xt =
    bfloat16(out * norm_weight), ssq_out[m, g] = the sum of out[m, :]^2 over workgroup g's
    channels.  `tiles`: see `gemm_bf16`.  Returns the number of workgroups (the reader's n_part)."""
    M, K = a.shape
    N = w.shape[0]
    _req(a, "gemm.a", torch.bfloat16)
    _req(w, "gemm.w", torch.bfloat16, (N, K))
    th = _req_tiles(tiles, N, K)
    if silu_pair:
        if accumulate or N % 64:
            raise KernelError("gemm: the paired epilogue stores, and needs N to be a multiple of 64")
        _req(out, "gemm.out", torch.bfloat16, (M, N // 2))
        epi = _pair_epilogue(pair_act)
    else:
        _req(out, "gemm.out", torch.float32, (M, N))
        epi = EPI_ACCUMULATE if accumulate else EPI_STORE
    ssq_in, n_part, inv_h, eps = None, 0, 0.0, 0.0
    if factor is not None:
        _req(factor.ssq, "gemm.factor", torch.float32)
        if factor.ssq.numel() < factor.n_part * 16 or factor.n_part < 1:
            raise KernelError(f"gemm.factor: {factor.ssq.numel()} floats for {factor.n_part} workgroups")
        ssq_in, n_part, inv_h, eps = factor.ssq, factor.n_part, 1.0 / factor.size, factor.eps
    cap = 0
    if norm_weight is not None:
        _req(norm_weight, "gemm.norm_weight", torch.float32, (N,))
        _req(xt, "gemm.xt", torch.bfloat16, (M, N))
        _req(ssq_out, "gemm.ssq_out", torch.float32)
        cap = ssq_out.numel()
    groups = ctypes.c_int(0)
    _check(lib().tl_gemm_bf16_norm(_p(a), _p(w), _p(tiles), th, _p(out), M, N, K, epi, _p(ssq_in), n_part,
                                   ctypes.c_float(inv_h), ctypes.c_float(eps), _p(norm_weight), _p(xt),
                                   _p(ssq_out), cap, ctypes.byref(groups), _stream()))
    return groups.value


MID_ROWS = 128      # most rows of the kernels that share a step's activations through LDS
RING_K = 128        # the kernel that brings both operands into a ring of LDS stages takes K in multiples of this
LIBRARY_ROWS = 64   # where K is no such multiple, the BLAS library's product beats ours above this many rows


def own_rows(K: int) -> int:
    """The most rows for which a bfloat16 product over K runs in this package's own kernels (more
    go to the BLAS library)."""
    return MID_ROWS if K % RING_K == 0 else LIBRARY_ROWS


_UNITS: dict = {}


def compute_units(device) -> int:
    """Compute units of the device (256 on an MI355X)."""
    key = str(device)
    if key not in _UNITS:
        _UNITS[key] = int(torch.cuda.get_device_properties(device).multi_processor_count)
    return _UNITS[key]


def mid_splits(M: int, N: int, K: int, units: int) -> int:
    """For 17..MID_ROWS rows: into how many slices K is cut, each a workgroup's own, whose partial
    sums the next kernel adds up; 1 where N alone gives the workgroups.

    K a multiple of RING_K (the ring kernel: 128 channels a workgroup, which holds a compute unit by
    itself): as many slices as make one round of workgroups over the `units` compute units, each
    with four stages of 128 k at least (o and down of the 7B shape at 64 rows: 8 slices, 256
    workgroups, 9.4 and 22.2 us; q|k|v: 5).

    Other K (gemm_mid: 64 channels a workgroup, steps of 256 k): so that some 400 workgroups or more
    are at work, a power of two; twice as many where only that fills the compute units evenly."""
    if K % RING_K == 0:
        blocks = -(-N // 128)
        return max(1, min(units // blocks, (K // RING_K) // 4, 16))
    blocks = -(-N // 64)
    steps = -(-K // 256)
    want = -(-400 // blocks)
    S = 1
    while S < want and S < 16:
        S *= 2
    if 1 < S < 16 and 2 * S <= steps and (blocks * S) % units != 0 and (blocks * 2 * S) % units == 0:
        S *= 2
    while S > steps:
        S //= 2
    return max(1, S)


def gemm_mid_bf16(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor, n_split: int = 1,
                  accumulate: bool = False, silu_pair: bool = False, pair_act: str = "silu") -> None:
    """The product for 17..MID_ROWS rows (the ring kernel where K is a multiple of RING_K, else
    gemm_mid).  n_split == 1: out as in `gemm_bf16`.  n_split > 1: out is float32 [n_split, M, N]
    and receives partial sums that the next kernel adds up (`add_rmsnorm`, `add_partials`,
    `rope_commit`)."""
    M, K = a.shape
    N = w.shape[0]
    _req(a, "gemm.a", torch.bfloat16)
    _req(w, "gemm.w", torch.bfloat16, (N, K))
    if n_split > 1:
        if accumulate or silu_pair:
            raise KernelError("gemm_mid: partial sums cannot be accumulated or paired")
        _req(out, "gemm.out", torch.float32, (n_split, M, N))
        epi = EPI_STORE
    elif silu_pair:
        _req(out, "gemm.out", torch.bfloat16, (M, N // 2))
        epi = _pair_epilogue(pair_act)
    else:
        _req(out, "gemm.out", torch.float32, (M, N))
        epi = EPI_ACCUMULATE if accumulate else EPI_STORE
    _check(lib().tl_gemm_mid_bf16(_p(a), _p(w), _p(out), M, N, K, int(n_split), epi, _stream()))


def gemm_ring_bf16(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor, n_split: int = 1, accumulate: bool = False,
                   silu_pair: bool = False, waves: int = 4, kc: int = 128, pair_act: str = "silu") -> None:
    """`gemm_mid_bf16` through the kernel that brings both operands into a ring of stages in LDS
    (K a multiple of 128); `waves`: 4, 7 or 8 waves a workgroup with 16 channels each; `kc`: the k
    of a stage, 64 or 128."""
    M, K = a.shape
    N = w.shape[0]
    _req(a, "gemm.a", torch.bfloat16)
    _req(w, "gemm.w", torch.bfloat16, (N, K))
    if n_split > 1:
        if accumulate or silu_pair:
            raise KernelError("gemm_ring: partial sums cannot be accumulated or paired")
        _req(out, "gemm.out", torch.float32, (n_split, M, N))
        epi = EPI_STORE
    elif silu_pair:
        _req(out, "gemm.out", torch.bfloat16, (M, N // 2))
        epi = _pair_epilogue(pair_act)
    else:
        _req(out, "gemm.out", torch.float32, (M, N))
        epi = EPI_ACCUMULATE if accumulate else EPI_STORE
    _check(lib().tl_gemm_ring_bf16(_p(a), _p(w), _p(out), M, N, K, int(n_split), epi, int(waves), int(kc), _stream()))


def add_rmsnorm(x: torch.Tensor, parts: torch.Tensor, w: torch.Tensor, eps: float, out: torch.Tensor) -> None:
    """x += parts[0] + parts[1] + ... (float32 [S, n, H]); out = rmsnorm(x)."""
    n, H = x.shape
    _req(x, "add_rmsnorm.x", torch.float32)
    _req(parts, "add_rmsnorm.parts", torch.float32)
    if parts.dim() != 3 or tuple(parts.shape[1:]) != (n, H):
        raise KernelError(f"add_rmsnorm.parts: shape {tuple(parts.shape)}, kernel needs [S, {n}, {H}]")
    _req(w, "add_rmsnorm.w", torch.float32, (H,))
    _req(out, "add_rmsnorm.out", None, (n, H))
    _check(lib().tl_add_rmsnorm(_p(x), _p(parts), parts.shape[0], _p(w), ctypes.c_float(eps), _p(out),
                                _code(out.dtype), n, H, _stream()))


def add_partials(x: torch.Tensor, parts: torch.Tensor) -> None:
    """x += parts[0] + parts[1] + ... (float32 [S, n, H])."""
    n, H = x.shape
    _req(x, "add_partials.x", torch.float32)
    _req(parts, "add_partials.parts", torch.float32)
    if parts.dim() != 3 or tuple(parts.shape[1:]) != (n, H):
        raise KernelError(f"add_partials.parts: shape {tuple(parts.shape)}, kernel needs [S, {n}, {H}]")
    _check(lib().tl_add_partials(_p(x), _p(parts), parts.shape[0], n, H, _stream()))


def gemm_library(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor, accumulate: bool = False) -> None:
    """out[M,N] (+)= a[M,K] @ w[N,K]^T through the BLAS library (hipBLASLt below
    torch): bfloat16 operands, float32 accumulation; out is float32, or bfloat16
    when it is only stored.  The reference hands its products to the vendor's
    library likewise (src/kernels/cuda/mod.rs:462-552, src/kernels/rocm/mod.rs)."""
    M, K = a.shape
    N = w.shape[0]
    _req(a, "gemm.a", torch.bfloat16)
    _req(w, "gemm.w", torch.bfloat16, (N, K))
    _req(out, "gemm.out", None, (M, N))
    if out.dtype == torch.float32:
        if accumulate:
            torch.addmm(out, a, w.t(), out_dtype=torch.float32, out=out)
        else:
            torch.mm(a, w.t(), out_dtype=torch.float32, out=out)
    elif out.dtype == torch.bfloat16 and not accumulate:
        torch.mm(a, w.t(), out=out)
    else:
        raise KernelError(f"gemm_library: cannot {'accumulate into' if accumulate else 'store'} {out.dtype}")


def bf16_gemm_ok(a: torch.Tensor, w: torch.Tensor) -> bool:
    return (a.dtype == torch.bfloat16 and w.dtype == torch.bfloat16 and a.shape[1] % 8 == 0
            and a.data_ptr() % 16 == 0 and w.data_ptr() % 16 == 0)


def gemm(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor, accumulate: bool = False,
         tiles: Optional[torch.Tensor] = None) -> None:
    """out[M,N] (+)= a[M,K] @ w[N,K]^T with float32 accumulation.  The kernel
    follows from the operand types: bfloat16 x bfloat16 goes to the matrix
    cores (our kernels up to `own_rows(K)` rows, the library's above), anything
    with float32 in it to the plain FMA kernel.  `tiles`: see `gemm_bf16`."""
    if bf16_gemm_ok(a, w):
        if a.shape[0] > own_rows(a.shape[1]):
            gemm_library(a, w, out, accumulate)
        elif a.shape[0] > LIBRARY_ROWS:
            gemm_mid_bf16(a, w, out, 1, accumulate)
        else:
            gemm_bf16(a, w, out, accumulate, tiles=tiles)
    else:
        gemm_plain(a, w, out, accumulate)


def rope_commit(qkv: torch.Tensor, row_pos, rotation, table, ring_pages: int, nq: int, nkv: int, d: int,
                q: torch.Tensor, pages: torch.Tensor) -> None:
    """Single-token steps: rotate q and k (`rotation`: see `rope_split`), write q [n,nq,d] and
    put k and v of row n straight into sequence n's page for its position.  qkv may be
    [S, n, width]: partial products that are added up on the way in."""
    n_parts = qkv.shape[0] if qkv.dim() == 3 else 1
    n = qkv.shape[-2]
    _req(qkv, "rope.qkv", torch.float32, ((n_parts,) if qkv.dim() == 3 else ()) + (n, (nq + 2 * nkv) * d))
    _req(row_pos, "rope.row_pos", torch.int32, (n,))
    rot = _rotation(rotation, d, "rope")
    _req(q, "rope.q", pages.dtype, (n, nq, d))
    _req(table, "rope.table", torch.int32)
    _req(pages, "rope.pages")
    if pages.dim() != 5 or tuple(pages.shape[1:]) != (2, nkv, PAGE, d):
        raise KernelError(f"rope.pages: shape {tuple(pages.shape)}, kernel needs [*, 2, {nkv}, {PAGE}, {d}]")
    if table.dim() != 2 or table.shape[0] != n:
        raise KernelError("rope.table: needs one row per sequence")
    _check(lib().tl_rope_commit(_p(qkv), n_parts, _p(row_pos), _p(rot.inv_freq), rot.rotary_dim,
                                int(rot.interleaved), _p(table), table.shape[1], ring_pages,
                                n, nq, nkv, d, _p(q), _p(pages), _code(q.dtype), _stream()))


def qkv_rope_commit_ok(a: torch.Tensor, w: torch.Tensor, d: int, pages: torch.Tensor) -> bool:
    """Whether `qkv_rope_commit` serves this step: bfloat16 all through, at most 16 rows."""
    return bf16_gemm_ok(a, w) and a.shape[0] <= 16 and d % 16 == 0 and pages.dtype == torch.bfloat16


def qkv_rope_commit(a: torch.Tensor, w: torch.Tensor, row_pos, rotation, table, ring_pages: int, nq: int,
                    nkv: int, d: int, q: torch.Tensor, pages: torch.Tensor,
                    factor: Optional[RowFactor] = None, units: int = 0,
                    tiles: Optional[torch.Tensor] = None) -> None:
    """For a step with one token a sequence (at most 16): the product a @ w^T with w = q|k|v,
    the rotation of q and k, q into its buffer and k, v into the pages, in one kernel; the
    same bits as `gemm` and then `rope_commit`.  `factor`: see `gemm_bf16_norm`.  `units`
    (tests): how many units of 8 weight rows a workgroup owns, 1 to 4; 0 leaves it to the launcher.
    `tiles`: `tile_weights(w, qkv_tile_rows(nq, nkv, d, device, rotation))`, read instead of w.
    `rotation`: see `rope_split`."""
    n, K = a.shape
    _req(a, "qkv_rope_commit.a", torch.bfloat16)
    _req(w, "qkv_rope_commit.w", torch.bfloat16, ((nq + 2 * nkv) * d, K))
    _req_tiles(tiles, (nq + 2 * nkv) * d, K, height=16)
    _req(row_pos, "qkv_rope_commit.row_pos", torch.int32, (n,))
    rot = _rotation(rotation, d, "qkv_rope_commit")
    _req(q, "qkv_rope_commit.q", torch.bfloat16, (n, nq, d))
    _req(table, "qkv_rope_commit.table", torch.int32)
    _req(pages, "qkv_rope_commit.pages", torch.bfloat16)
    if pages.dim() != 5 or tuple(pages.shape[1:]) != (2, nkv, PAGE, d):
        raise KernelError(f"qkv_rope_commit.pages: shape {tuple(pages.shape)}, kernel needs [*, 2, {nkv}, {PAGE}, {d}]")
    if table.dim() != 2 or table.shape[0] != n:
        raise KernelError("qkv_rope_commit.table: needs one row per sequence")
    ssq_in, n_part, inv_h, eps = None, 0, 0.0, 0.0
    if factor is not None:
        _req(factor.ssq, "qkv_rope_commit.factor", torch.float32)
        if factor.ssq.numel() < factor.n_part * 16 or factor.n_part < 1:
            raise KernelError(f"qkv_rope_commit.factor: {factor.ssq.numel()} floats for {factor.n_part} workgroups")
        ssq_in, n_part, inv_h, eps = factor.ssq, factor.n_part, 1.0 / factor.size, factor.eps
    _check(lib().tl_gemm_qkv_rope_commit(_p(a), _p(w), _p(tiles), n, K, _p(row_pos), _p(rot.inv_freq),
                                         rot.rotary_dim, int(rot.interleaved), _p(table),
                                         table.shape[1], int(ring_pages), nq, nkv, d, _p(q), _p(pages),
                                         _p(ssq_in), n_part, ctypes.c_float(inv_h), ctypes.c_float(eps),
                                         int(units), _stream()))


def aligned_columns(n_cached, n_new):
    """Column offsets (and their total) at which sequences lie when each is
    given room from the last multiple of 64 below its cached length up to its
    end, rounded up to 64: positions that are multiples of 64 then lie on
    columns that are.  The total is the row length of buffers laid out so (kept
    off multiples of 512: rows a power of two apart would all fall on the same
    memory channels).  The rule is the host library's, which lays out steps."""
    import numpy as np
    from ..cache import native
    c = np.ascontiguousarray(np.asarray(list(n_cached), dtype=np.int64))
    n = np.ascontiguousarray(np.asarray(list(n_new), dtype=np.int64))
    off = np.zeros(len(c), dtype=np.int32)
    total = native.lib().tl_aligned_columns(len(c), c.ctypes.data, n.ctypes.data, off.ctypes.data)
    return off.tolist(), int(total)


PREFILL_BLOCK = 128            # rows of a sequence that one workgroup of the multi-token attention takes
PREFILL_CUT_TILES = 8          # fewest tiles of 64 keys of a run into which a block's keys are cut
PREFILL_MAX_WAYS = 8           # most runs of a block


class PrefillCuts:
    """How the host lays out the work of the multi-token attention for a step with fewer workgroups than
    the device has compute units: `items` int32 [n, 4] on the device, rows (sequence, block, first tile of
    keys, one past the last | slot << 24 | (ways - 1) << 27 | 1 << 30) with the dearest last for one of the
    `ways` runs into which a block's keys are cut, (sequence, block, 0, 0) for a whole block; `blocks` int32 [n_cut, 4], the (sequence,
    block, ways, 0) that are cut; `ways`: the most runs of any block (the places a row has for its sums)."""

    def __init__(self, entries, blocks, n_seqs: int, n_tiles: int, device):
        self.n_items, self.n_cut, self.n_seqs, self.n_tiles = len(entries), len(blocks), n_seqs, n_tiles
        self.ways = max(w for _, _, w in blocks)
        flat = torch.tensor([v for e in entries for v in e] + [v for b in blocks for v in (*b, 0)], dtype=torch.int32)
        dev = flat.to(device)
        self.items = dev[:4 * len(entries)].view(-1, 4)
        self.blocks = dev[4 * len(entries):].view(-1, 4)


def prefill_layout(n_new, len_before, window: Optional[int], nq: int, units: int):
    """The host's side of `prefill_cuts`: (entries, cut blocks, number of blocks), or None where the
    kernel's own order serves.  A launch with fewer workgroups (blocks of 128 rows x heads) than
    compute units leaves units idle while its longest chain of key tiles runs: then a block's keys are cut
    into as many runs as there are units for (`PREFILL_MAX_WAYS` at most, `PREFILL_CUT_TILES` tiles a run at
    least), each run a workgroup of its own, and a second kernel merges their sums.  (A launch that fills the
    device gains nothing: one prompt of 2,048 tokens takes 81 us cut in two against 75.)"""
    global _last_layout
    key = (tuple(int(n) for n in n_new), tuple(int(c) for c in len_before), window, nq, units, PREFILL_CUT_TILES)
    if _last_layout is not None and _last_layout[0] == key:       # every layer of a step asks the same
        return _last_layout[1]
    laid = _prefill_layout(key[0], key[1], window, nq, units)
    _last_layout = (key, laid)
    return laid


_last_layout = None


def _prefill_layout(n_new, len_before, window, nq, units):
    n_blocks = sum(-(-n // PREFILL_BLOCK) for n in n_new)
    if n_blocks == 0 or n_blocks * nq > units:
        return None
    # with a workgroup for more than every other unit only chains twice as long are worth the merge
    # (1,024 tokens alone, 256 workgroups of at most 16 tiles: 43.8 us with the last block cut in two against 40.3)
    run = PREFILL_CUT_TILES * (1 if n_blocks * nq * 2 <= units else 2)
    if max(c + n for c, n in zip(len_before, n_new)) <= (2 * run - 1) * PAGE:
        return None                               # no sequence reaches into the last tile of two runs
    blocks = [(b, t) for b, n in enumerate(n_new) for t in range(-(-n // PREFILL_BLOCK))]
    most = min(PREFILL_MAX_WAYS, 2 * units // (len(blocks) * nq))      # (a compute unit holds two workgroups)
    entries, cut = [], []
    for b, t in blocks:
        first = int(len_before[b])
        p_lo = first + t * PREFILL_BLOCK
        p_hi = first + min((t + 1) * PREFILL_BLOCK, int(n_new[b])) - 1
        j_lo = max(0, p_lo - window + 1) if window else 0
        jt_first, jt_last = j_lo // PAGE, p_hi // PAGE
        tiles = jt_last - jt_first + 1
        ways = min(most, tiles // run)
        if ways < 2:
            entries.append((tiles, (b, t, 0, 0)))
            continue
        cut.append((b, t, ways))
        for w in range(ways):
            lo, hi = jt_first + tiles * w // ways, jt_first + tiles * (w + 1) // ways
            if hi >= 1 << 24:
                return None                   # (a tile index beyond the entry's 24 bits)
            entries.append((hi - lo, (b, t, lo, hi | (w << 24) | ((ways - 1) << 27) | (1 << 30))))
    if not cut:
        return None
    entries.sort(key=lambda e: e[0])
    return [e[1] for e in entries], cut, len(blocks)


def prefill_cuts(n_new, len_before, window: Optional[int], nq: int, units: int, device) -> Optional[PrefillCuts]:
    """The layout (`prefill_layout`) for a step whose sequences bring `n_new` rows after `len_before`
    positions, on the device, or None where the kernel's own order serves."""
    laid = prefill_layout(n_new, len_before, window, nq, units)
    if laid is None:
        return None
    return PrefillCuts(laid[0], laid[1], len(n_new), laid[2], device)


def prefill_serves(dtype: torch.dtype, d: int) -> bool:
    """Does the multi-token attention on the matrix cores serve this dtype and head size?"""
    return dtype == torch.bfloat16 and d % 16 == 0 and 16 <= d <= 256


def _prefill_args(q, k_new, vt_new, tile_off, pages, table, row_pos, cu_seqlens, n_cached, out) -> None:
    """The operands of the attention for steps with many rows, checked against what its grid assumes."""
    n, nq, d = q.shape
    nkv = pages.shape[2]
    B = n_cached.shape[0]
    _req(q, "attn.q", torch.bfloat16)
    _req(k_new, "attn.k_new", torch.bfloat16, (n, nkv, d))
    _req(vt_new, "attn.vt_new", torch.bfloat16)
    if vt_new.dim() != 3 or tuple(vt_new.shape[:2]) != (nkv, d) or vt_new.shape[2] % PAGE:
        raise KernelError(f"attn.vt_new: shape {tuple(vt_new.shape)}, kernel needs [{nkv}, {d}, a multiple of {PAGE}]")
    _req(tile_off, "attn.tile_off", torch.int32, (B,))
    _req(pages, "attn.pages", torch.bfloat16)
    if pages.dim() != 5 or tuple(pages.shape[1:]) != (2, nkv, PAGE, d):
        raise KernelError(f"attn.pages: shape {tuple(pages.shape)}, kernel needs [*, 2, nkv, {PAGE}, {d}]")
    _req(table, "attn.table", torch.int32)
    _req(row_pos, "attn.row_pos", torch.int32, (n,))
    _req(cu_seqlens, "attn.cu_seqlens", torch.int32, (B + 1,))
    _req(n_cached, "attn.n_cached", torch.int32, (B,))
    _req(out, "attn.out", torch.bfloat16, (n, nq, d))
    if table.dim() != 2 or table.shape[0] != B:
        raise KernelError("attn.table: needs one row per sequence")


def attn_prefill_bf16(q, k_new, vt_new, tile_off, pages, table, ring_pages: int, row_pos, cu_seqlens,
                      n_cached, n_tiles: int, window: Optional[int], scale: float, out,
                      cuts: Optional[PrefillCuts] = None, part: Optional[torch.Tensor] = None) -> None:
    """bfloat16 attention for steps with many rows per sequence.  `vt_new`:
    this step's values transposed [nkv, d, cols] at the columns that
    `aligned_columns` gives (`tile_off`).  `n_tiles`: sum over the sequences
    of ceil(rows / 128).  `cuts` (`prefill_cuts` of this step) with `part`, float32 scratch of
    n * nq * cuts.ways * (d + 4) elements: the keys of long blocks go to several workgroups each."""
    n, nq, d = q.shape
    nkv = pages.shape[2]
    B = n_cached.shape[0]
    _prefill_args(q, k_new, vt_new, tile_off, pages, table, row_pos, cu_seqlens, n_cached, out)
    if cuts is None:
        _check(lib().tl_attn_prefill_bf16(_p(q), _p(k_new), _p(vt_new), vt_new.shape[2], _p(tile_off), _p(pages),
                                          _p(table), table.shape[1], ring_pages, _p(row_pos), _p(cu_seqlens),
                                          _p(n_cached), B, int(n_tiles), nq, nkv, d, int(window or 0),
                                          ctypes.c_float(scale), _p(out), None, None, 0, None, 0,
                                          ctypes.c_longlong(0), n, _stream()))
        return
    if cuts.n_seqs != B or cuts.n_tiles != int(n_tiles):
        raise KernelError(f"attn.cuts: laid out for {cuts.n_seqs} sequences and {cuts.n_tiles} blocks, "
                          f"the step has {B} and {int(n_tiles)}")
    if part is None:
        raise KernelError("attn.part: blocks cut in halves need room for their sums")
    _req(part, "attn.part", torch.float32)
    _req(cuts.items, "attn.cuts.items", torch.int32, (cuts.n_items, 4))
    _req(cuts.blocks, "attn.cuts.blocks", torch.int32, (cuts.n_cut, 4))
    _check(lib().tl_attn_prefill_bf16(_p(q), _p(k_new), _p(vt_new), vt_new.shape[2], _p(tile_off), _p(pages),
                                      _p(table), table.shape[1], ring_pages, _p(row_pos), _p(cu_seqlens),
                                      _p(n_cached), B, cuts.n_items, nq, nkv, d, int(window or 0),
                                      ctypes.c_float(scale), _p(out), _p(cuts.items), _p(cuts.blocks), cuts.n_cut,
                                      _p(part), cuts.ways, ctypes.c_longlong(part.numel()), n, _stream()))


def _decode_args(q, pages, table, row_pos, part, out, n_splits: int) -> None:
    """The operands of single-token attention, checked against what its grid assumes."""
    B, nq, d = q.shape
    nkv = pages.shape[2]
    _req(q, "attn.q", torch.bfloat16)
    _req(pages, "attn.pages", torch.bfloat16)
    if pages.dim() != 5 or tuple(pages.shape[1:]) != (2, nkv, PAGE, d):
        raise KernelError(f"attn.pages: shape {tuple(pages.shape)}, kernel needs [*, 2, nkv, {PAGE}, {d}]")
    _req(table, "attn.table", torch.int32)
    _req(row_pos, "attn.row_pos", torch.int32, (B,))
    _req(part, "attn.part", torch.float32)
    _req(out, "attn.out", torch.bfloat16, (B, nq, d))
    if table.dim() != 2 or table.shape[0] != B:
        raise KernelError("attn.table: needs one row per sequence")
    if part.numel() < B * nq * n_splits * (d + 2):
        raise KernelError(f"attn.part: {part.numel()} elements, kernel needs {B * nq * n_splits * (d + 2)}")


def attn_decode_bf16(q, pages, table, ring_pages: int, row_pos, window: Optional[int], scale: float,
                     n_splits: int, part, out) -> None:
    """bfloat16 attention of one new token per sequence over its pages (the
    token's own key is already committed).  `part`: float32 scratch of at
    least B * nq * n_splits * (d + 2) elements."""
    B, nq, d = q.shape
    nkv = pages.shape[2]
    _decode_args(q, pages, table, row_pos, part, out, n_splits)
    _check(lib().tl_attn_decode_bf16(_p(q), _p(pages), _p(table), table.shape[1], ring_pages, _p(row_pos),
                                     B, nq, nkv, d, int(window or 0), ctypes.c_float(scale),
                                     int(n_splits), _p(part), _p(out), _stream()))


def decode_through_lds(on: bool) -> bool:
    """For tests and measurements: whether single-token attention with heads of 64, 128 or 256 goes
    through the kernel that stages the pages in LDS (the default) or, like every other head size,
    through the one that reads them into registers.  Returns the setting before the call."""
    return bool(lib().tl_attn_decode_through_lds(int(bool(on))))


def decode_groups(B: int, nq: int, nkv: int) -> int:
    """Workgroups of a decode step's attention before splitting: one per
    (sequence, KV head, 16 query heads of its group)."""
    return B * nkv * (-(-(nq // nkv) // 16))


SPLIT_PAGES = 4             # fewest pages a part of the keys has
SPLIT_COST = 0.15           # what a part more costs in the merge, in pages of a workgroup's way (8 sequences of
                            # 8 KV heads over 4,096 keys: 4 parts 3.91 ms a step, 8 parts 3.96, 6 parts 4.08)
FULL_UNIT_HEAD = 128        # the kernel that reads the pages into registers: the head size from which one workgroup
                            # has enough bytes under way to keep a compute unit streaming; smaller heads get
                            # FULL_UNIT_HEAD // head_dim workgroups a unit (heads of 48 ...)
LDS_DECODE_PER_UNIT = {64: 2, 128: 2, 256: 1}    # the kernel that stages the pages in LDS (these head sizes): its
                            # workgroups hold 64 KB of LDS each (128 KB with heads of 256), so two share a unit, and
                            # a round of workgroups is twice the units (64 sequences of 8 KV heads of 128 over 4,096
                            # keys, 512 workgroups: 162 us with two a unit, 169 with one holding 128 KB)


def decode_workgroups_per_unit(head_dim: int) -> int:
    """How many workgroups of a decode step's attention a compute unit holds at a time."""
    return LDS_DECODE_PER_UNIT.get(int(head_dim), max(1, FULL_UNIT_HEAD // max(1, int(head_dim))))


@functools.lru_cache(maxsize=4096)
def _decode_splits(groups: int, max_pages: int, units: int) -> int:
    most = max(1, min(-(-max_pages // SPLIT_PAGES), -(-4 * units // groups), 4096))
    # rounds of workgroups over the compute units x pages a workgroup goes through, and the merge
    cost = lambda s: -(-groups * s // units) * -(-max_pages // s) + SPLIT_COST * s
    return min(range(1, most + 1), key=lambda s: (cost(s), s))


def decode_splits(B: int, nq: int, nkv: int, max_pages: int, units: int, head_dim: int) -> int:
    """Into how many parts the keys of a decode step are cut.  A compute unit streams at a rate of
    its own, so the step's attention takes as long as the unit with the most to read: rounds of
    workgroups over the `units` compute units times the pages a workgroup has, plus the merge's
    share for every part; parts have at least four pages.  A round is as many workgroups as the
    units hold at a time (`decode_workgroups_per_unit`): eight sequences with eight KV heads of 128
    are 8 parts, 512 workgroups, two a unit (28.2 us a layer over 4,096 keys against 30.3 in 4 parts).
    With heads of less than 64 the kernel that reads into registers has too few bytes under way to
    keep a unit busy with one workgroup, and a round is 128 // head size a unit (32 sequences of 4 KV
    heads of 32 take 19.2 us in 4 parts, 27.2 in 2)."""
    return _decode_splits(decode_groups(B, nq, nkv), int(max_pages), int(units) * decode_workgroups_per_unit(head_dim))


def uses_transposed_values(dtype: torch.dtype, d: int, all_single: bool) -> bool:
    """Does `attention` take this step's values transposed (`vt_new`)?"""
    return dtype == torch.bfloat16 and d % 16 == 0 and 16 <= d <= 256 and not all_single


def attention(q, k_new, v_new, pages, table, ring_pages: int, ctx, n_cached, window, scale: float,
              out, vt_new=None) -> None:
    """Attention of a step's rows: keys j < n_cached[b] from the pages, later
    ones from this step's rows (`k_new`/`v_new`; None when everything is in
    the pages).  bfloat16 with head sizes in steps of 16 runs on the matrix
    cores, single-token steps and steps with longer rows each in their own
    kernel (the latter takes the values transposed, `vt_new`, see
    `rope_split`); everything else runs in the plain kernel."""
    n, nq, d = q.shape
    fast = q.dtype == torch.bfloat16 and d % 16 == 0 and 16 <= d <= 256
    if fast and k_new is None and ctx.all_single:
        nkv = pages.shape[2]
        splits = decode_splits(n, nq, nkv, table.shape[1], compute_units(q.device), d)   # by the table's width: fixed while a graph lives
        part = ctx.workspace.get("attn_part", (n * nq * splits * (d + 2),), torch.float32)
        attn_decode_bf16(q, pages, table, ring_pages, ctx.row_pos, window, scale, splits, part, out)
    elif fast and k_new is not None and vt_new is not None:
        n_tiles = int(sum(-(-int(x) // PREFILL_BLOCK) for x in ctx.host["n_new"]))
        cuts = part = None
        if not ctx.host.get("fixed_launches"):   # (a captured graph's launches must not be shaped by lengths)
            at = ("prefill_cuts", window, nq)
            if at not in ctx.host:                               # the same for every layer of the step
                ctx.host[at] = prefill_cuts(ctx.host["n_new"], ctx.host["len_before"], window, nq,
                                            compute_units(q.device), q.device)
            cuts = ctx.host[at]
            if cuts is not None:
                part = ctx.workspace.get("attn_prefill_part", (n * nq * cuts.ways * (d + 4),), torch.float32)
        attn_prefill_bf16(q, k_new, vt_new, ctx.tile_off, pages, table, ring_pages, ctx.row_pos,
                          ctx.cu_seqlens, n_cached, n_tiles, window, scale, out, cuts=cuts, part=part)
    else:
        attn_plain(q, k_new, v_new, pages, table, ring_pages, ctx.row_seq, ctx.row_pos, ctx.cu_seqlens,
                   n_cached, window, scale, out)


READ_SHAPES = {0: "8 loads a lane, a grid stride apart", 1: "16 loads a lane", 2: "32 loads a lane",
               3: "8 loads a lane, a contiguous share a workgroup", 4: "16 loads a lane, contiguous",
               5: "8 loads a lane, non-temporal", 6: "16 loads a lane, non-temporal, contiguous",
               7: "8 loads a wave straight into LDS", 8: "16 loads a wave straight into LDS"}


def _measure_lib() -> ctypes.CDLL:
    """The library of the kernels that only measure the machine (built apart from the model's)."""
    L = load_measure()
    L.tl_measure_last_error.restype = ctypes.c_char_p
    return L


def _check_measure(rc: int) -> None:
    if rc != 0:
        raise KernelError(_measure_lib().tl_measure_last_error().decode())


def measure_ceilings(device="cuda:0", gib: float = 8.0, shapes=None) -> dict:
    """What the simplest kernels get on this machine: GB/s of one read of a buffer far larger
    than the caches, in every shape of `READ_SHAPES` (the best is reported with its shape, the
    others beside it), GB/s of a copy (bytes read plus bytes written), and TFLOP/s of independent
    bfloat16 MFMAs on registers (the best of a few runs and launch shapes each)."""
    import time
    units = compute_units(device)
    quantum = units * 32 * 256 * 32 * 16          # whole iterations of every shape at every number of workgroups (1 GiB)
    n_bytes = max(1, round(gib * 2 ** 30 / quantum)) * quantum
    buf = torch.empty(n_bytes // 4, dtype=torch.float32, device=device).normal_()
    sink = torch.zeros(units * 32, dtype=torch.float32, device=device)

    def timed(launch):
        torch.cuda.synchronize()
        t = time.perf_counter()
        _check_measure(launch())
        torch.cuda.synchronize()
        return time.perf_counter() - t

    by_shape = {}
    for shape in (READ_SHAPES if shapes is None else shapes):
        best = 0.0
        for blocks in (units, units * 2, units * 4, units * 8, units * 16, units * 32):
            for _ in range(3):
                dt = timed(lambda: _measure_lib().tl_stream_read_shape(_p(buf), ctypes.c_size_t(n_bytes), _p(sink), blocks,
                                                              shape, _stream()))
                best = max(best, n_bytes / dt / 1e9)
        by_shape[shape] = round(best, 1)
    top = max(by_shape, key=by_shape.get)
    half = n_bytes // 2
    dst = buf.view(-1)[half // 4:]
    best_copy = 0.0
    for blocks in (units, units * 2, units * 4, units * 8):
        for _ in range(3):
            dt = timed(lambda: _measure_lib().tl_stream_copy(_p(buf), _p(dst), ctypes.c_size_t(half), blocks, _stream()))
            best_copy = max(best_copy, 2 * half / dt / 1e9)
    del buf, dst
    best_mfma = 0.0
    for blocks in (units, units * 2, units * 4):
        iters = 8192
        for _ in range(3):
            dt = timed(lambda: _measure_lib().tl_mfma_chain(iters, blocks, _p(sink), _stream()))
            flop = blocks * 4 * iters * 8 * 2 * 32 * 32 * 16
            best_mfma = max(best_mfma, flop / dt / 1e12)
    return {"hbm_read_GBs": by_shape[top], "hbm_read_shape": READ_SHAPES[top],
            "hbm_read_by_shape_GBs": {READ_SHAPES[k]: v for k, v in by_shape.items()},
            "hbm_copy_GBs": round(best_copy, 1), "mfma_bf16_TFLOPs": round(best_mfma, 1)}


def measure_pipes(device="cuda:0", iters: int = 20000) -> dict:
    """Whether a SIMD's matrix pipe and vector pipe work at the same time (`pipes_kernel` in
    csrc/measure/ceilings.hip): nanoseconds an iteration of one workgroup a compute unit, for the same work a
    SIMD laid out in five ways.  `mfma_only`, `vector_only`: one wave a SIMD with one kind of work
    (4 MFMAs 32x32x16, or 32 FMAs and 8 exponentials, an iteration); `both_in_one_wave`: one wave a SIMD
    does both; `both_in_two_waves`: two waves a SIMD, each both, half the iterations (what the prefill
    attention does); `split_roles`: two waves a SIMD, one with the MFMAs and one with the vector work."""
    import time
    units = compute_units(device)
    sink = torch.zeros(16, dtype=torch.float32, device=device)

    def run(role, waves, n):
        best = float("inf")
        for _ in range(3):
            torch.cuda.synchronize()
            t = time.perf_counter()
            _check_measure(_measure_lib().tl_pipes(role, waves, n, units, _p(sink), _stream()))
            torch.cuda.synchronize()
            best = min(best, time.perf_counter() - t)
        return round(best / iters * 1e9, 2)

    return {"mfma_only": run(0, 4, iters), "vector_only": run(1, 4, iters), "both_in_one_wave": run(2, 4, iters),
            "both_in_two_waves": run(2, 8, iters // 2), "split_roles": run(3, 8, iters)}
