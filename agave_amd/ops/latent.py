"""Python faces of ``csrc/latent.hip`` and ``csrc/attention_latent.hip``: the rows of the attention that caches one small
row per position, the small products per (token, head) around its attention kernel, and its decode attention.

A rotation is given as a :class:`Turn`: float64 frequencies, one per pair, and whether the pairs are neighbours
(2e, 2e + 1) or halves (e, e + pairs); the elements behind the pairs stay as they are.

Every function checks on the host what its kernel and grid assume and launches on the current stream.
"""
from __future__ import annotations

from typing import NamedTuple, Optional, Tuple

import torch

from . import kernels, library
from .attention_biased import _check_row_pages
from .kernels import _P, _I, _L, _F, _dev, _f32vec, _i32, _rows, dt, ptr, stream

LIBRARY, ATTENTION = "latent", "attention_latent"
MAX_SPLITS = 64          # workgroups that share a row's pages at most
MAX_PAIRS = 256          # pairs a rotation turns at most

kernels.register_signatures(LIBRARY, {
    "agave_latent_prepare": [_I, _P, _L, _P, _P, _L, _I, _I, _I, _P, _L, _P, _P, _L, _I, _I, _P, _I, _I, _F, _P, _P, _P, _I, _P, _I, _I,
                             _P, _P, _I, _F, _P],
    "agave_latent_turn_queries": [_I, _P, _L, _P, _L, _I, _I, _I, _P, _I, _I, _F, _P, _I, _P],
    "agave_latent_decode_rows_ok": [_I, _I, _I, _I],
    "agave_latent_decode_rows": [_P, _L, _P, _P, _L, _I, _I, _P, _L, _P, _P, _L, _I, _I, _P, _I, _I, _F, _P, _P, _P, _I, _P, _I, _I, _P, _P,
                                 _I, _F, _P],
    "agave_latent_fresh_pages": [_P, _L, _I, _P, _L, _I, _P, _P, _P, _I, _I, _P, _I, _I, _I, _I, _I, _I, _P],
    "agave_gate_rows": [_I, _P, _L, _P, _L, _I, _I, _P],
    "agave_heads_product": [_I, _I, _P, _L, _I, _P, _P, _L, _I, _P, _L, _P, _I, _I, _F, _I, _P, _I, _I, _I, _I, _I, _P],
})
kernels.register_signatures(ATTENTION, {
    "agave_latent_decode_ok": [_I, _I, _I, _I],
    "agave_latent_decode": [_P, _L, _P, _P, _P, _I, _P, _I, _P, _I, _I, _I, _I, _F, _I, _P, _I, _P, _P, _P],
    "agave_latent_values": [_P, _P, _I, _P, _P, _L, _P, _L, _I, _I, _I, _I, _P],
})


class Turn(NamedTuple):
    freq: Optional[torch.Tensor]         # float64 [pairs], or None: nothing is turned
    neighbours: bool = False             # pairs (2e, 2e + 1) instead of (e, e + pairs)
    magnitude: float = 1.0               # multiplies sine and cosine


NO_TURN = Turn(None)


class CachePages(NamedTuple):
    """Where a step's key/value rows go: one memory's pages with the step's table of them."""
    k_pages: torch.Tensor
    v_pages: torch.Tensor
    table: torch.Tensor
    base: torch.Tensor
    packed: bool


def _lib():
    return kernels.lib(LIBRARY)


def _attn():
    return kernels.lib(ATTENTION)


def _f32rows(t: torch.Tensor, what: str, n: int, cols: int) -> int:
    if t.dtype != torch.float32 or t.dim() != 2 or t.stride(1) != 1 or tuple(t.shape) != (n, cols):
        raise ValueError(f"{what}: expected float32 rows [{n}, {cols}], got {tuple(t.shape)} {t.dtype} strides {t.stride()}")
    return t.stride(0)


def _typed_rows(t: torch.Tensor, what: str, n: int, cols: int, dtype: torch.dtype) -> int:
    if t.dtype != dtype or tuple(t.shape) != (n, cols):
        raise ValueError(f"{what}: expected {dtype} rows [{n}, {cols}], got {tuple(t.shape)} {t.dtype}")
    return _rows(t, what)


def _turn(turn: Turn, rot_dim: int, what: str) -> int:
    """The number of pairs, after a look at the frequencies."""
    if turn.freq is None:
        return 0
    f = turn.freq
    if f.dtype != torch.float64 or f.dim() != 1 or not f.is_contiguous():
        raise TypeError(f"{what}: frequencies are a contiguous float64 vector")
    if 2 * f.numel() > rot_dim or f.numel() > MAX_PAIRS:
        raise ValueError(f"{what}: {2 * f.numel()} rotated elements exceed the {rot_dim} there are (or {2 * MAX_PAIRS})")
    return f.numel()


def _pages(pages: Optional[CachePages], kd: int, vd: int, dtype: torch.dtype):
    """The arguments (k pages, v pages, table, width, base, number of pages, packed) of a kernel that fills pages."""
    if pages is None:
        return (None, None, None, 0, None, 0, 0)
    _dev(pages.k_pages, pages.v_pages, pages.table, pages.base)
    n = _check_row_pages(pages.k_pages, pages.v_pages, 1, kd, vd, dtype, pages.packed)
    width = kernels._check_table(pages.table, pages.base, None)
    return (ptr(pages.k_pages), ptr(pages.v_pages), ptr(pages.table), width, ptr(pages.base), n, 1 if pages.packed else 0)


def latent_prepare(step, eps: float, turn: Turn, rot_dim: int, *, q_raw: Optional[torch.Tensor] = None,
                   q_weight: Optional[torch.Tensor] = None, q_out: Optional[torch.Tensor] = None, q_heads: int = 0, q_dim: int = 0,
                   kv_raw: Optional[torch.Tensor] = None, kv_weight: Optional[torch.Tensor] = None,
                   k_row: Optional[torch.Tensor] = None, kv_rank: int = 0, pages: Optional[CachePages] = None) -> None:
    """What a step's first product left (float32 rows, column slices are fine) becomes rows of ``q_out``'s / ``k_row``'s type.

    Queries: ``q_out = q_raw / rms(q_raw) * q_weight`` (a query latent), or, with ``q_heads``, the rows themselves, each head
    [``q_dim`` | ``rot_dim``] with its last ``rot_dim`` elements turned.
    Keys and values: ``k_row = [kv_raw[:, :kv_rank] / rms(..) * kv_weight | the last rot_dim elements turned]``, and with
    ``pages`` the same row (and its first ``kv_rank`` elements as values) into its place in the cache.
    Either side may be absent; eps stands inside the root."""
    _dev(q_raw, q_weight, q_out, kv_raw, kv_weight, k_row, turn.freq)
    n = step.n_tokens
    some = q_out if q_out is not None else k_row
    if some is None:
        raise ValueError("latent_prepare: nothing to prepare")
    dtype = some.dtype
    half = _turn(turn, rot_dim, "latent_prepare")
    _i32(step.tok_pos, "positions", n)
    ldq = ldqo = ldkv = ldkr = q_rank = 0
    if q_raw is not None:
        cols = q_heads * (q_dim + rot_dim) if q_heads else q_raw.shape[1]
        ldq, ldqo = _f32rows(q_raw, "queries", n, cols), _typed_rows(q_out, "q_out", n, cols, dtype)
        if not q_heads:
            q_rank = cols
            _f32vec(q_weight, "query latent's weight", q_rank)
            if q_weight is None:
                raise ValueError("latent_prepare: a query latent has a weight")
    page_args = (None, None, None, 0, None, 0, 0)
    if kv_raw is not None:
        ldkv = _f32rows(kv_raw, "key/value latent", n, kv_rank + rot_dim)
        _f32vec(kv_weight, "key/value latent's weight", kv_rank)
        if kv_weight is None:
            raise ValueError("latent_prepare: the key/value latent has a weight")
        ldkr = _typed_rows(k_row, "k_row", n, kv_rank + rot_dim, dtype)
        page_args = _pages(pages, kv_rank + rot_dim, kv_rank, dtype)
        _i32(step.tok_seq, "sequences", n)
    library.call(_lib(), "agave_latent_prepare", dt(some), ptr(q_raw), ldq, ptr(q_weight), ptr(q_out), ldqo, q_rank, q_heads, q_dim,
                 ptr(kv_raw), ldkv, ptr(kv_weight), ptr(k_row), ldkr, kv_rank, rot_dim, ptr(turn.freq), half,
                 1 if turn.neighbours else 0, float(turn.magnitude), *page_args, ptr(step.tok_seq), ptr(step.tok_pos), n, float(eps), stream())


def turn_queries(q: torch.Tensor, q_out: torch.Tensor, n_heads: int, dim: int, rot_dim: int, turn: Turn, tok_pos: torch.Tensor) -> None:
    """Every head of ``q`` [N, heads * (dim + rot_dim)] with its last ``rot_dim`` elements turned; ``q_out`` may be ``q``."""
    _dev(q, q_out, turn.freq, tok_pos)
    n, cols = q.shape[0], n_heads * (dim + rot_dim)
    ldq, ldqo = _typed_rows(q, "q", n, cols, q.dtype), _typed_rows(q_out, "q_out", n, cols, q.dtype)
    _i32(tok_pos, "positions", n)
    library.call(_lib(), "agave_latent_turn_queries", dt(q), ptr(q), ldq, ptr(q_out), ldqo, n_heads, dim, rot_dim, ptr(turn.freq),
                 _turn(turn, rot_dim, "turn_queries"), 1 if turn.neighbours else 0, float(turn.magnitude), ptr(tok_pos), n, stream())


def heads_product(x: torch.Tensor, w: torch.Tensor, y: torch.Tensor, n_heads: int, x_head: int, y_head: int, *,
                  tail: int = 0, turn: Turn = NO_TURN, tok_pos: Optional[torch.Tensor] = None,
                  gate: Optional[torch.Tensor] = None, force_plain: bool = False) -> None:
    """For every token t and head h:  y[t, h * y_head + c] = sum_k w[h, c, k] * x[t, h * x_head + k]  (``w`` is
    [heads, n_out, K]); the head's next ``tail`` input elements are copied behind the product, turned at tok_pos[t]; with
    ``gate`` (float32 [N, heads * n_out]) the product is multiplied by sigmoid(gate).  ``x``'s rows are of ``y``'s type or
    float32.  Sums are 32-bit; bfloat16 results with K a multiple of 8 run on the matrix cores."""
    _dev(x, w, y, turn.freq, tok_pos, gate)
    n = x.shape[0]
    ldx, ldy = _rows(x, "x"), _rows(y, "y")
    if w.dim() != 3 or w.shape[0] != n_heads or not w.is_contiguous() or w.dtype != y.dtype or x.dtype not in (y.dtype, torch.float32):
        raise ValueError(f"heads_product: w must be contiguous [{n_heads}, n_out, K] of y's dtype, x of it or float32")
    n_out, k = int(w.shape[1]), int(w.shape[2])
    if y.shape[0] != n or x_head < k + tail or y_head < n_out + tail or x.shape[1] < (n_heads - 1) * x_head + k + tail \
            or y.shape[1] < (n_heads - 1) * y_head + n_out + tail:
        raise ValueError(f"heads_product: rows of {tuple(x.shape)} and {tuple(y.shape)} do not hold {n_heads} heads of "
                         f"{k} + {tail} in (every {x_head}) and {n_out} + {tail} out (every {y_head})")
    half = 0
    if tail:
        if tok_pos is None:
            raise ValueError("heads_product: trailing elements need the tokens' positions")
        _i32(tok_pos, "positions", n)
        half = _turn(turn, tail, "heads_product")
    ldg = 0
    if gate is not None:
        ldg = _f32rows(gate, "gate", n, n_heads * n_out)
    if (k + tail) * 4 > 60 * 1024:
        raise ValueError(f"heads_product: a head of {k + tail} input elements is too long")
    library.call(_lib(), "agave_heads_product", dt(y), 1 if x.dtype == torch.float32 else 0, ptr(x), ldx, x_head, ptr(w), ptr(y), ldy,
                 y_head, ptr(gate), ldg, ptr(turn.freq), half, 1 if turn.neighbours else 0, float(turn.magnitude), tail, ptr(tok_pos), n, n_heads, n_out, k,
                 1 if force_plain else 0, stream())


def decode_rows_ok(q_raw: torch.Tensor, n_heads: int, dim: int, rot_dim: int) -> bool:
    """Whether :func:`decode_rows` takes a bfloat16 decode step whose queries are these float32 rows."""
    return (q_raw.dtype == torch.float32 and q_raw.data_ptr() % 16 == 0 and
            bool(_lib().agave_latent_decode_rows_ok(q_raw.shape[0], dim, rot_dim, q_raw.stride(0) % 4)))


def decode_rows(q_raw: torch.Tensor, fold: torch.Tensor, folded: torch.Tensor, n_heads: int, dim: int, rot_dim: int, turn: Turn,
                kv_raw: torch.Tensor, kv_weight: torch.Tensor, kv_rank: int, pages: CachePages, step, eps: float) -> None:
    """A bfloat16 decode step's :func:`heads_product` of the queries (``fold`` [heads, kv_rank, dim]) and
    :func:`latent_prepare` of the key/value rows (only into their pages), in one launch."""
    _dev(q_raw, fold, folded, turn.freq, kv_raw, kv_weight)
    n, qd, kd, bf = step.n_tokens, dim + rot_dim, kv_rank + rot_dim, torch.bfloat16
    ldq = _f32rows(q_raw, "queries", n, n_heads * qd)
    if tuple(fold.shape) != (n_heads, kv_rank, dim) or not fold.is_contiguous() or fold.dtype != bf:
        raise ValueError(f"decode_rows: fold must be contiguous bfloat16 [{n_heads}, {kv_rank}, {dim}]")
    ldf, ldkv = _typed_rows(folded, "folded", n, n_heads * kd, bf), _f32rows(kv_raw, "key/value latent", n, kd)
    _f32vec(kv_weight, "key/value latent's weight", kv_rank)
    _i32(step.tok_pos, "positions", n)
    _i32(step.tok_seq, "sequences", n)
    library.call(_lib(), "agave_latent_decode_rows", ptr(q_raw), ldq, ptr(fold), ptr(folded), ldf, n_heads, dim, ptr(kv_raw), ldkv,
                 ptr(kv_weight), None, 0, kv_rank, rot_dim, ptr(turn.freq), _turn(turn, rot_dim, "decode_rows"),
                 1 if turn.neighbours else 0, float(turn.magnitude), *_pages(pages, kd, kv_rank, bf), ptr(step.tok_seq), ptr(step.tok_pos), n, float(eps),
                 stream())


def fresh_pages(up: torch.Tensor, k_row: torch.Tensor, kv_rank: int, k_pages: torch.Tensor, v_pages: torch.Tensor,
                table: torch.Tensor, step, n_heads: int, dim: int, rot_dim: int, v_head_dim: int) -> None:
    """Every head's keys [``up[:, h * dim ..]`` | ``k_row[:, kv_rank ..]``] and values (``up``'s columns behind the keys') of a
    step whose sequences all start at position 0, into pages in operand order: sequence b's i-th page is ``table[b, i]``.  All
    64 places of every page are written (zeros past the sequence's end)."""
    _dev(up, k_row, k_pages, v_pages, table)
    n, bf = step.n_tokens, torch.bfloat16
    ldu = _typed_rows(up, "up", n, n_heads * (dim + v_head_dim), bf)
    ldkr = _typed_rows(k_row, "k_row", n, kv_rank + rot_dim, bf)
    n_pages = _check_row_pages(k_pages, v_pages, n_heads, dim + rot_dim, v_head_dim, bf, True)
    if table.dtype != torch.int32 or table.dim() != 2 or table.shape[0] != step.n_seqs or not table.is_contiguous():
        raise ValueError(f"fresh_pages: the table must be contiguous int32 [{step.n_seqs}, pages]")
    max_rows = max(b - a for a, b in zip(step.cu[:-1], step.cu[1:]))
    if table.shape[1] * 64 < max_rows:
        raise ValueError(f"fresh_pages: a table of {table.shape[1]} pages for {max_rows} rows")
    _i32(step.cu_dev, "cu", step.n_seqs + 1)
    library.call(_lib(), "agave_latent_fresh_pages", ptr(up), ldu, n_heads * dim, ptr(k_row), ldkr, kv_rank, ptr(k_pages), ptr(v_pages),
                 ptr(table), table.shape[1], n_pages, ptr(step.cu_dev), step.n_seqs, max_rows, n_heads, dim, rot_dim, v_head_dim, stream())


def gate_rows(x: torch.Tensor, gate: torch.Tensor) -> None:
    """x *= sigmoid(gate) in place; ``gate`` is float32 of ``x``'s shape (column slices are fine)."""
    _dev(x, gate)
    n, cols = x.shape
    ldx = _rows(x, "x")
    ldg = _f32rows(gate, "gate", n, cols)
    library.call(_lib(), "agave_gate_rows", dt(x), ptr(x), ldx, ptr(gate), ldg, n, cols, stream())


# ------------------------------------------------------------------ decode attention
def decode_attention_ok(kd: int, kv_rank: int, v_head_dim: int) -> bool:
    """Whether cached rows of ``kd`` elements with values of ``kv_rank`` run on the decode kernels of their own."""
    return bool(_attn().agave_latent_decode_ok(kd, kv_rank, v_head_dim, 0))


def decode_splits(n_rows: int, n_heads: int, table_width: int) -> int:
    """How many workgroups share a row's pages: as many as put one on every compute unit, never more than there are
    pages.  It depends on nothing that changes from step to step, so a recorded step stays valid."""
    groups = max(1, n_rows * ((n_heads + 15) // 16))
    return max(1, min(MAX_SPLITS, table_width, 256 // groups))


def decode_attention(q: torch.Tensor, v_up: torch.Tensor, out: torch.Tensor, gate: Optional[torch.Tensor], k_pages: torch.Tensor,
                     v_pages: torch.Tensor, table: torch.Tensor, base: torch.Tensor, step, n_heads: int, kd: int, kv_rank: int,
                     scale: float, window: Optional[int], sink: Optional[torch.Tensor], workspace, splits: Optional[int] = None) -> None:
    """A decode step (one row a sequence) over cached rows in operand order: for every row and head, the softmax of ``scale *
    q.row`` over the visible rows weighs their first ``kv_rank`` elements, and ``out[t, h] = v_up[h] @ that`` (``v_up`` [heads,
    v, kv_rank]), times sigmoid(gate) where a gate is given (float32).  ``window`` W: only positions p-W+1 .. p; ``sink``:
    exp(sink_h) joins the denominator."""
    _dev(q, v_up, out, gate, k_pages, v_pages, table, base, sink)
    n, bf = step.n_tokens, torch.bfloat16
    if not step.is_decode or n != step.n_seqs:
        raise ValueError("decode_attention: one row a sequence")
    v_dim = int(v_up.shape[1])
    if tuple(v_up.shape) != (n_heads, v_dim, kv_rank) or v_up.dtype != bf or not v_up.is_contiguous():
        raise ValueError(f"decode_attention: v_up must be contiguous bfloat16 [{n_heads}, v, {kv_rank}]")
    ldq, ldo = _typed_rows(q, "q", n, n_heads * kd, bf), _typed_rows(out, "out", n, n_heads * v_dim, bf)
    ldg = _f32rows(gate, "gate", n, n_heads * v_dim) if gate is not None else 0
    n_pages = _check_row_pages(k_pages, v_pages, 1, kd, kv_rank, bf, True)
    width = kernels._check_table(table, base, None)
    _f32vec(sink, "sink", n_heads)
    _i32(step.tok_pos, "positions", n)
    if splits is None:
        splits = decode_splits(n, n_heads, width)
    part_o = workspace.get("latent_parts", n * n_heads * splits, kv_rank, torch.float32)
    part_ml = workspace.get("latent_parts_ml", n * n_heads * splits, 2, torch.float32)
    library.call(_attn(), "agave_latent_decode", ptr(q), ldq, ptr(k_pages), ptr(v_pages), ptr(table), width, ptr(base), n_pages,
                 ptr(step.tok_pos), n, n_heads, kd, kv_rank, float(scale), int(window or 0), ptr(sink), splits, ptr(part_o),
                 ptr(part_ml), stream())
    library.call(_attn(), "agave_latent_values", ptr(part_o), ptr(part_ml), splits, ptr(v_up), ptr(out), ldo, ptr(gate), ldg, n,
                 n_heads, kv_rank, v_dim, stream())
