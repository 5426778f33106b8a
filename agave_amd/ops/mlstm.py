"""Python faces of ``csrc/mlstm.hip``: the matrix memory with exponential gates, from the rows of a mixer's first product to
the rows of its output product.

Every function checks on the host what its kernel and grid assume and launches on the current stream.
"""
from __future__ import annotations

from typing import NamedTuple

import torch

from . import kernels, library
from .kernels import _P, _I, _L, _F, _dev, _f32vec, _i32, _rows, dt, ptr, stream

LIBRARY = "mlstm"
MAX_KEY, MAX_VALUE = 1024, 1024          # the largest heads

_COMMON = [_I] + [_P] * 6 + [_L] + [_P] * 3 + [_F] * 4 + [_P] * 5
kernels.register_signatures(LIBRARY, {
    "agave_mlstm_step": _COMMON + [_I, _I, _I, _I, _P, _P, _P, _L, _P],
    "agave_mlstm_chunks": _COMMON + [_I] * 6 + [_P] * 4 + [_L, _P, _L, _P],
    "agave_mlstm_chunk_size": [],
})


def _lib():
    return kernels.lib(LIBRARY)


def chunk_size() -> int:
    return int(_lib().agave_mlstm_chunk_size())


class Gates(NamedTuple):
    """What the mixer adds to the rows: the gates' biases [heads], their cap, the read-out's weight [heads * dv] and eps, the
    number in the divisor, the factor on q."""
    i_bias: torch.Tensor
    f_bias: torch.Tensor
    cap: float
    weight: torch.Tensor
    norm_eps: float
    floor_eps: float
    q_scale: float


def mlstm(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, gate: torch.Tensor, i_in: torch.Tensor, f_in: torch.Tensor,
          gates: Gates, out: torch.Tensor, S: torch.Tensor, n: torch.Tensor, m: torch.Tensor, step, heads: int, dk: int, dv: int,
          workspace) -> None:
    """Advance ``S`` [slots, heads, dv, dk], ``n`` [slots, heads, dk] and ``m`` [slots, heads] (float32) over the step's tokens,
    sequence by sequence, and write each token's normed and gated read-out to ``out`` [N, heads * dv]:

    with i = cap tanh((i_in + i_bias) / cap) and f = logsigmoid(cap tanh((f_in + f_bias) / cap)) per head,
    m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T (n with k alone);
    o = S^T (q_scale q) / (max(|n . q_scale q|, exp(-m')) + floor_eps);  out = o / rms(o) * weight * sigmoid(gate).

    The inputs are column slices of the same float32 rows: q, k [N, heads * dk], v, gate [N, heads * dv], i_in, f_in [N, heads].
    A step of one token a sequence updates the state in place; other steps run in chunks of tokens."""
    _dev(q, k, v, gate, i_in, f_in, out, S, n, m, gates.i_bias, gates.f_bias, gates.weight)
    rows = step.n_tokens
    for t, what, cols in ((q, "q", heads * dk), (k, "k", heads * dk), (v, "v", heads * dv), (gate, "gate", heads * dv),
                          (i_in, "i", heads), (f_in, "f", heads)):
        if t.dtype != torch.float32 or t.dim() != 2 or t.stride(1) != 1 or tuple(t.shape) != (rows, cols) or t.stride(0) != q.stride(0):
            raise ValueError(f"mlstm: {what} must be float32 [{rows}, {cols}] columns of the same rows as q, got {tuple(t.shape)} "
                             f"{t.dtype} strides {t.stride()}")
    for t, what, shape in ((S, "S", (heads, dv, dk)), (n, "n", (heads, dk)), (m, "m", (heads,))):
        if t.dtype != torch.float32 or not t.is_contiguous() or tuple(t.shape[1:]) != shape or t.shape[0] != S.shape[0]:
            raise ValueError(f"mlstm: {what} must be contiguous float32 [slots, {', '.join(map(str, shape))}], got {tuple(t.shape)}")
    if max(step.slots) >= S.shape[0]:
        raise ValueError("mlstm: a slot lies outside the state")
    if dk > MAX_KEY or dv > MAX_VALUE:
        raise ValueError(f"mlstm: heads of {dk} key and {dv} value elements (at most {MAX_KEY} and {MAX_VALUE})")
    _f32vec(gates.i_bias, "input gate's bias", heads)
    _f32vec(gates.f_bias, "forget gate's bias", heads)
    _f32vec(gates.weight, "read-out's weight", heads * dv)
    ldo = _rows(out, "out")
    if tuple(out.shape) != (rows, heads * dv):
        raise ValueError(f"mlstm: out must be [{rows}, {heads * dv}], got {tuple(out.shape)}")
    _i32(step.cu_dev, "cu", step.n_seqs + 1)
    _i32(step.slots_dev, "slots", step.n_seqs)
    common = (dt(out), ptr(q), ptr(k), ptr(v), ptr(gate), ptr(i_in), ptr(f_in), q.stride(0), ptr(gates.i_bias), ptr(gates.f_bias),
              ptr(gates.weight), float(gates.cap), float(gates.floor_eps), float(gates.norm_eps), float(gates.q_scale), ptr(S), ptr(n),
              ptr(m), ptr(step.cu_dev), ptr(step.slots_dev))
    if step.is_decode and rows == step.n_seqs:
        num = workspace.get("mlstm_num", rows, heads * dv, torch.float32)
        nq = workspace.get("mlstm_nq", rows, heads, torch.float32)
        library.call(_lib(), "agave_mlstm_step", *common, step.n_seqs, heads, dk, dv, ptr(num), ptr(nq), ptr(out), ldo, stream())
        return
    chunk = chunk_size()
    numbers = rows // chunk + step.n_seqs
    max_rows = max(b - a for a, b in zip(step.cu[:-1], step.cu[1:]))
    sums = workspace.get("mlstm_gates", 3 * numbers, heads * chunk, torch.float64)
    totals = workspace.get("mlstm_totals", 2 * numbers, heads, torch.float64)
    m0 = workspace.get("mlstm_maxima", numbers + step.n_seqs, heads, torch.float32)
    part = workspace.get("mlstm_parts", numbers, heads * (dv + 1) * dk, torch.float32)
    library.call(_lib(), "agave_mlstm_chunks", *common, rows, step.n_seqs, max_rows, heads, dk, dv, ptr(sums), ptr(totals), ptr(m0),
                 ptr(part), numbers, ptr(out), ldo, stream())
