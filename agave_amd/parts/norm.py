"""Norms as parts.  A norm owns two things a block asks of it around the 32-bit residual stream
``h``: adding a branch it normalises (``h += norm(branch)``, the norm *after* a sublayer), and
normalising ``h`` for the next sublayer (the norm *before* it), optionally of chosen rows only.
A block never does either itself; it calls ``add_and_norm`` of the norm that comes next, which
also receives the branch that is still to be added (with the norm after its sublayer, if any),
so that a kind of norm that can do both in one pass over ``h`` does so.

:class:`Norm` is the general form: ``apply`` and ``add_to`` are what a new kind writes, and
``add_and_norm`` is put together from them.  :class:`RmsNorm` overrides it with the one fused
kernel when the norm after the sublayer is an RMS norm too (or none).

RMSNorm: ``y = x * (1/sqrt(mean(x^2) + eps)) * g`` (``src/backend/kernels/cpu/norm.zig:7-40``);
for HF checkpoints ``g = 1 + w``, folded into a 32-bit gain once at load as the reference's
``warmNormCache`` does (``src/models/gemma3.zig:908-954``).
"""
from __future__ import annotations

from typing import List, Optional, Tuple

import torch

from ..config.spec import NormSpec
from ..ops import kernels
from ..weights.loader import TensorNeed
from .base import BuildEnv, register

# (branch, the norm after its sublayer | None[, base]).  ``base``: the tensor that holds the residual
# stream at this moment if that is not ``h`` (a product that made its own normalised rows summed the
# stream up in other memory, see NormedRows); whoever adds the branch reads the rows there and
# writes them to ``h``.
Pending = Optional[Tuple]


def unpack_pending(pending: Pending):
    """(branch, post norm, base), each None where there is none."""
    if pending is None:
        return None, None, None
    if len(pending) == 2:
        return pending[0], pending[1], None
    return pending


def add_branch(h: torch.Tensor, pending: Pending) -> None:
    """h += post(branch) for a branch that is still to be added (post None: h += branch).  The
    branch may be 32-bit slices [slices, rows, hidden] that add up to it."""
    branch, post, base = unpack_pending(pending)
    if branch is None:
        if base is not None:
            h.copy_(base)
        return
    if post is None:
        kernels.residual_norm(h, branch, None, 0.0, None, None, 0.0, src=base)
    elif isinstance(post, RmsNorm):
        kernels.residual_norm(h, branch, post.gain, post.eps, None, None, 0.0, src=base)
    elif isinstance(post, LayerNorm):
        kernels.residual_layernorm(h, branch, post.weight, post.bias, post.eps, None, None, None, 0.0, src=base)
    else:
        # (other kinds, the norm of the residual sum among them: what they write for themselves)
        if base is not None:
            h.copy_(base)
        post.add_to(h, branch)


class NormedRows:
    """``norm(h + post(branch))`` as a promise: the rows that a sublayer is given, not yet computed.

    Whoever takes them either calls :meth:`rows` (the norm's kernel runs, ``h`` holds the sum, and
    the rows come back as a tensor), or, being a product that can make them in its own kernel,
    takes :meth:`rms_arguments` and reports with :meth:`made_by_consumer` where it left the sum
    (it cannot write ``h`` in place: its other workgroups still read it).  ``shape`` and ``dtype``
    are those of the rows to be."""

    def __init__(self, h: torch.Tensor, pending: Pending, norm, workspace, dtype: torch.dtype):
        self.h, self.pending, self.norm = h, pending, norm
        self.workspace = workspace
        self.shape, self.dtype = h.shape, dtype
        self.base: Optional[torch.Tensor] = None      # afterwards: where the stream is, if not in h
        self._rows: Optional[torch.Tensor] = None
        self.taken = False

    def rows(self) -> torch.Tensor:
        if self._rows is None:
            if self.taken:
                raise RuntimeError("these rows were made inside a product's kernel and exist nowhere else")
            x = self.workspace.get("normed", self.shape[0], self.shape[1], self.dtype)
            self.norm.add_and_norm(self.h, self.pending, x)
            self._rows, self.taken = x, True
        return self._rows

    def rms_arguments(self):
        """(h_in, h_out, branch, post_gain, post_eps, pre_gain, pre_eps) if nothing was computed yet and
        both norms are RMS norms (the one on the branch may be absent), else None."""
        if self.taken:
            return None
        branch, post, base = unpack_pending(self.pending)
        if not isinstance(self.norm, RmsNorm) or (post is not None and not isinstance(post, RmsNorm)):
            return None
        h_in = base if base is not None else self.h
        h_out = None
        if branch is not None:
            h_out = self.h if base is not None else self.workspace.get("residual_aside", self.shape[0], self.shape[1],
                                                                       torch.float32)
        return (h_in, h_out, branch, post.gain if (branch is not None and post is not None) else None,
                post.eps if (branch is not None and post is not None) else 0.0, self.norm.gain, self.norm.eps)

    def made_by_consumer(self, h_in: torch.Tensor, h_out: Optional[torch.Tensor]) -> None:
        self.taken = True
        now = h_out if h_out is not None else h_in
        self.base = None if now is self.h or now.data_ptr() == self.h.data_ptr() else now


def rows_as_they_are(h: torch.Tensor, pending: Pending, out: torch.Tensor, rows: Optional[torch.Tensor] = None) -> None:
    """What stands where a norm would for a model without one: the pending branch is added and
    the (chosen) rows of ``h`` are handed on, rounded to ``out``'s element type.  One kernel where the
    branch's norm is an RMS norm (or none) and all rows are wanted, as with a norm in front."""
    branch, post, base = unpack_pending(pending)
    if isinstance(post, NormOfSum) and base is None and rows is None and (branch.dim() == 3 or branch.dtype == out.dtype):
        kernels.norm_of_sum(h, branch, post.alpha, post.bias, post.gain, post.eps, out)
        return
    fused = rows is None and branch is not None and (post is None or isinstance(post, RmsNorm))
    if fused and branch.dim() == 2 and branch.dtype != out.dtype:
        fused = False
    if fused:
        kernels.residual_norm(h, branch, post.gain if post is not None else None, post.eps if post is not None else 0.0,
                              out, None, 0.0, None, src=base)
        return
    add_branch(h, pending)
    kernels.gather_rows(h, rows, out)


class Norm:
    """The interface of a norm, with ``add_and_norm`` composed of the two pieces a kind must
    write.  Fields: ``size`` (the length of the rows it normalises)."""
    size: int

    def apply(self, x: torch.Tensor, out: torch.Tensor, rows: Optional[torch.Tensor] = None) -> None:
        """out[i] = norm(x[rows[i]]) (all rows if ``rows`` is None).  ``x`` is the 32-bit residual
        stream [n, size]; ``out`` has the activations' element type."""
        raise NotImplementedError

    def add_to(self, h: torch.Tensor, branch: torch.Tensor) -> None:
        """h += norm(branch).  ``branch`` is [n, size] in the activations' element type, or 32-bit
        slices [slices, n, size] that add up to it."""
        raise NotImplementedError

    def add_and_norm(self, h: torch.Tensor, pending: Pending, out: Optional[torch.Tensor],
                     rows: Optional[torch.Tensor] = None) -> None:
        """Add the pending branch to ``h``, then out = self(h) (of the chosen rows) if asked."""
        add_branch(h, pending)
        if out is not None:
            self.apply(h, out, rows)


class RmsNorm(Norm):
    def __init__(self, spec: NormSpec, weights, env: BuildEnv):
        w = weights.get(spec.weight).to(torch.float32)
        if spec.add_one:
            w = w + 1.0
        self.gain = w.contiguous().to(env.device)
        self.eps = float(spec.eps)
        self.size = spec.size

    @staticmethod
    def tensor_needs(spec: NormSpec) -> List[TensorNeed]:
        return [TensorNeed(spec.weight, (spec.size,))]

    def apply(self, x, out, rows=None) -> None:
        kernels.residual_norm(x, None, None, 0.0, out, self.gain, self.eps, rows)

    def add_to(self, h, branch) -> None:
        kernels.residual_norm(h, branch, self.gain, self.eps, None, None, 0.0)

    def add_and_norm(self, h, pending, out, rows=None) -> None:
        """One kernel adds the branch (through the RMS norm after its sublayer, if it has one) and
        computes this norm, reading and writing ``h`` once."""
        branch, post, base = unpack_pending(pending)
        if isinstance(post, NormOfSum) and out is not None and rows is None and base is None \
                and (branch.dim() == 3 or branch.dtype == out.dtype):
            kernels.norm_of_sum(h, branch, post.alpha, post.bias, post.gain, post.eps, out, self.gain, self.eps)
            return
        if branch is not None and post is not None and not isinstance(post, RmsNorm):
            add_branch(h, (branch, post, base))     # another kind of norm after the sublayer: its own kernel
            branch = post = base = None
        if rows is not None and (branch is not None or base is not None):
            add_branch(h, (branch, post, base))     # the fused kernel gathers rows only without a branch
            branch = post = base = None
        if branch is None and out is None:
            add_branch(h, (None, None, base))
            return
        kernels.residual_norm(h, branch, post.gain if (branch is not None and post) else None,
                              post.eps if (branch is not None and post) else 0.0,
                              out, self.gain if out is not None else None, self.eps if out is not None else 0.0, rows,
                              src=base)


class NormOfSum(Norm):
    """The norm behind the residual sum, ``h <- rms(alpha h + branch + bias) * gain``, as the post norm of a pending branch:
    an RMS norm's weight and eps, the factor on the stream, and a bias that the branch was left without (None: none).
    Whoever takes the branch adds it, norms the sum and makes its own rows of it in one kernel."""

    def __init__(self, norm: RmsNorm, alpha: float, bias: Optional[torch.Tensor] = None):
        self.gain, self.eps, self.size = norm.gain, norm.eps, norm.size
        self.alpha, self.bias = float(alpha), bias

    def add_to(self, h, branch) -> None:
        kernels.norm_of_sum(h, branch, self.alpha, self.bias, self.gain, self.eps)


class LayerNorm(Norm):
    """``y = (x - mean(x)) / sqrt(var(x) + eps) * w + b`` with the variance the mean of the squared
    deviations.  A vector ``scale_by`` and a number ``mult`` that multiply the result (a layer scale and a
    multiplier on a residual branch) are folded into weight and bias once at load, in 32-bit.  One kernel
    adds a pending branch through the layer norm after its sublayer and computes this norm."""

    def __init__(self, spec: NormSpec, weights, env: BuildEnv):
        w = weights.get(spec.weight).to(torch.float32)
        b = weights.get(spec.bias).to(torch.float32) if spec.bias else None
        if spec.add_one:
            w = w + 1.0
        if spec.scale_by:
            by = weights.get(spec.scale_by).to(torch.float32)
            w = w * by
            b = b * by if b is not None else None
        if spec.mult != 1.0:
            w = w * float(spec.mult)
            b = b * float(spec.mult) if b is not None else None
        self.weight = w.contiguous().to(env.device)
        self.bias = b.contiguous().to(env.device) if b is not None else None
        self.eps = float(spec.eps)
        self.size = spec.size

    @staticmethod
    def tensor_needs(spec: NormSpec) -> List[TensorNeed]:
        needs = [TensorNeed(spec.weight, (spec.size,))]
        if spec.bias:
            needs.append(TensorNeed(spec.bias, (spec.size,)))
        if spec.scale_by:
            needs.append(TensorNeed(spec.scale_by, (spec.size,)))
        return needs

    def apply(self, x, out, rows=None) -> None:
        kernels.residual_layernorm(x, None, None, None, 0.0, out, self.weight, self.bias, self.eps, rows)

    def add_to(self, h, branch) -> None:
        kernels.residual_layernorm(h, branch, self.weight, self.bias, self.eps, None, None, None, 0.0)

    def add_and_norm(self, h, pending, out, rows=None) -> None:
        branch, post, base = unpack_pending(pending)
        if branch is not None and post is not None and not isinstance(post, LayerNorm):
            add_branch(h, (branch, post, base))     # another kind of norm after the sublayer: its own kernel
            branch = post = base = None
        if rows is not None and (branch is not None or base is not None):
            add_branch(h, (branch, post, base))     # the fused kernel gathers rows only without a branch
            branch = post = base = None
        if branch is None and out is None:
            add_branch(h, (None, None, base))
            return
        with_post = branch is not None and post is not None
        kernels.residual_layernorm(h, branch, post.weight if with_post else None, post.bias if with_post else None,
                                   post.eps if with_post else 0.0, out, self.weight if out is not None else None,
                                   self.bias if out is not None else None, self.eps if out is not None else 0.0, rows,
                                   src=base)


register("norm", "rmsnorm", RmsNorm)
register("norm", "layernorm", LayerNorm)
