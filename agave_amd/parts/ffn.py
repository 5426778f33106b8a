"""Dense gated feed-forward: ``W_down (act(W_gate x) * (W_up x))``.

Reference: ``src/models/gemma3.zig:830-880`` (gate and up products, ``geluMul``, down
product); the activation is the tanh form of GELU
(``src/backend/kernels/cpu/activation.zig:69-113``).  Gate and up are one stacked product.

The activation is the spec's (``GatedFfnSpec.activation``, one of
``agave_amd.ops.kernels.GATE_ACTIVATIONS``).  On the matrix cores the product itself ends in the tanh form of
GELU, SiLU and the clamped swish (one form with four numbers, ``agave_amd.ops.gemm_mfma.GateForm``); with any other, and
in 32-bit, the stacked product is followed by the elementwise kernel, which takes the activation as a parameter.
"""
from __future__ import annotations

from typing import List, Optional

import torch

import math

from ..config.spec import DenseFfnSpec, GatedFfnSpec
from ..ops import gemm_mfma, kernels
from ..weights.loader import TensorNeed
from .base import BuildEnv, register
from .linear import Linear


class GatedFfn:
    prompt_steps_can_be_recorded = True        # a multi-token step is the same launches whatever its tokens are
    takes_rows_to_be_normed = True             # its first product may make the normalised rows itself (NormedRows)

    def __init__(self, spec: GatedFfnSpec, weights, env: BuildEnv):
        if spec.activation not in kernels.GATE_ACTIVATIONS:
            raise ValueError(f"gated feed-forward: unsupported activation {spec.activation!r}; "
                             f"known: {sorted(kernels.GATE_ACTIVATIONS)}")
        self.spec = spec
        self.env = env
        # [gate; up] stacked; on the matrix cores their rows are interleaved so that the product ends in the
        # activation (where it has such a form; biases on both are added inside it)
        def bias(name):
            return weights.get(name) if name else None

        form = gemm_mfma.gate_form_of(spec.activation, spec.act_limit, spec.act_alpha)
        fused = form is not None and bool(spec.gate_bias) == bool(spec.up_bias)
        self.gate_up = Linear([weights.get(spec.gate_proj), weights.get(spec.up_proj)], env, "gate_up",
                              interleave_ff=spec.intermediate if fused else 0,
                              biases=[bias(spec.gate_bias), bias(spec.up_bias)], gate_form=form or gemm_mfma.GELU_TANH)
        self.down = Linear([weights.get(spec.down_proj)], env, "ffn_down", biases=[bias(spec.down_bias)])

    @staticmethod
    def tensor_needs(spec: GatedFfnSpec) -> List[TensorNeed]:
        needs = [TensorNeed(spec.gate_proj, (spec.intermediate, spec.hidden)),
                 TensorNeed(spec.up_proj, (spec.intermediate, spec.hidden)),
                 TensorNeed(spec.down_proj, (spec.hidden, spec.intermediate))]
        for name, size in ((spec.gate_bias, spec.intermediate), (spec.up_bias, spec.intermediate),
                           (spec.down_bias, spec.hidden)):
            if name:
                needs.append(TensorNeed(name, (size,)))
        return needs

    def hand_over_bias(self) -> Optional[torch.Tensor]:
        """The bias of what :meth:`forward` returns, for a block whose next kernel adds it: from now on the result is
        without it."""
        return self.down.hand_over_bias()

    def forward(self, x: torch.Tensor, step, slices_ok: bool = True, tag: str = "ffn") -> torch.Tensor:
        """``slices_ok`` False: the result is wanted as rows of the activations' type (a caller that is no
        block and adds something to it); ``tag`` keeps the buffers of two feed-forwards of one layer apart."""
        ff = self.spec.intermediate
        n = x.shape[0]
        act = self.env.workspace.get(tag + "_act", n, ff, x.dtype)
        if not self.gate_up.forward_gated(x, act):
            gu = self.gate_up.forward(x, tag="gate_up" if tag == "ffn" else tag + "_gate_up")
            kernels.gated_act(gu[:, :ff], gu[:, ff:], act, self.spec.activation, self.spec.act_limit, self.spec.act_alpha)
        return self.down.forward(act, tag=tag + "_down", slices_ok=slices_ok)    # the block adds it to the residual stream


class DenseFfn:
    """``W_down act(W_up x)`` without a gate.  The activation is the spec's, one of
    ``agave_amd.ops.kernels.UNARY_ACTIVATIONS``.  ``relu2`` is the square of ReLU; ``xielu`` has two learned numbers p and q in a tensor
    of its own:  z > 0: softplus(p) z^2 + z/2;  z <= 0: (1/2 + softplus(q)) (exp(z) - 1 - z) + z/2;
    the two factors are made once at load."""
    prompt_steps_can_be_recorded = True

    def __init__(self, spec: DenseFfnSpec, weights, env: BuildEnv):
        if spec.activation not in kernels.UNARY_ACTIVATIONS:
            raise ValueError(f"dense feed-forward: unsupported activation {spec.activation!r}; "
                             f"known: {sorted(kernels.UNARY_ACTIVATIONS)}")
        self.spec, self.env = spec, env
        self.up = Linear([weights.get(spec.up_proj)], env, "ffn_up")
        self.down = Linear([weights.get(spec.down_proj)], env, "ffn_down")
        self.p0 = self.p1 = 0.0
        if spec.activation == "xielu":
            if not spec.act_params:
                raise ValueError("dense feed-forward: xielu needs the tensor of its two numbers")
            a = weights.get(spec.act_params).to(torch.float64).view(-1)
            softplus = lambda v: math.log1p(math.exp(-abs(v))) + max(v, 0.0)
            self.p0, self.p1 = softplus(float(a[0])), 0.5 + softplus(float(a[1]))

    @staticmethod
    def tensor_needs(spec: DenseFfnSpec) -> List[TensorNeed]:
        needs = [TensorNeed(spec.up_proj, (spec.intermediate, spec.hidden)),
                 TensorNeed(spec.down_proj, (spec.hidden, spec.intermediate))]
        if spec.activation == "xielu":
            needs.append(TensorNeed(spec.act_params, (2,)))
        return needs

    def forward(self, x: torch.Tensor, step) -> torch.Tensor:
        n = x.shape[0]
        z = self.up.forward(x, tag="ffn_up")
        act = self.env.workspace.get("ffn_act", n, self.spec.intermediate, z.dtype)
        kernels.unary_act(z, act, self.spec.activation, self.p0, self.p1)
        return self.down.forward(act, tag="ffn_down", slices_ok=True)    # the block adds it to the residual stream


register("ffn", "gated_dense", GatedFfn)
register("ffn", "dense", DenseFfn)
