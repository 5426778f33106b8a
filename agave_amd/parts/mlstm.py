"""The matrix memory with exponential gates, as a mixer (the mLSTM of Beck et al., "xLSTM: Extended Long Short-Term Memory").

In the order of its steps: one product for everything that reads the mixer's input (q, k, v, the output gate, the two gates'
logits; 32-bit rows out); the recurrence with its gates, the division by the normaliser, the norm per head, the weight and the
output gate (``ops.mlstm``); the output product.  Between the first product and the rows of the output product everything is
32-bit.  State per sequence: S [heads, vdim, dim] (a column's rows together), n [heads, dim] and the running maximum m [heads].
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..cache import GroupKey, StateNeed
from ..config.spec import MlstmSpec
from ..ops import mlstm as ops
from ..weights.loader import TensorNeed
from .base import BuildEnv, register, state_tensor
from .linear import Linear


class Mlstm:
    @staticmethod
    def kernel_libraries(spec, dtype):
        return ("mlstm",)

    def __init__(self, spec: MlstmSpec, weights, env: BuildEnv):
        s = spec
        if s.head_dim > ops.MAX_KEY or s.v_head_dim > ops.MAX_VALUE:
            raise ValueError(f"mlstm: heads of {s.head_dim} key and {s.v_head_dim} value elements (at most {ops.MAX_KEY} and {ops.MAX_VALUE})")
        if s.gate_cap <= 0:
            raise ValueError("mlstm: the gates' cap must be positive")
        self.spec, self.env = spec, env
        kd, self.vd = s.n_heads * s.head_dim, s.n_heads * s.v_head_dim
        mats = [weights.get(n) for n in (s.q_proj, s.k_proj, s.v_proj, s.gate_proj, s.i_gate, s.f_gate)]
        bounds = [0, kd, 2 * kd, 2 * kd + self.vd, 2 * (kd + self.vd), 2 * (kd + self.vd) + s.n_heads, 2 * (kd + self.vd + s.n_heads)]
        odd = -bounds[-1] % 4
        if odd:                     # rows in whole steps of 16 bytes
            mats.append(torch.zeros((odd, s.hidden), dtype=mats[-1].dtype, device=mats[-1].device))
            bounds.append(bounds[-1] + odd)
        self._bounds = tuple(bounds)
        self.proj = Linear(mats, env, "mlstm_in")

        def vec(name):
            return weights.get(name).to(torch.float32).contiguous().view(-1).to(env.device)
        self.gates = ops.Gates(vec(s.i_bias), vec(s.f_bias), s.gate_cap, vec(s.out_norm), s.norm_eps, s.floor_eps, s.head_dim ** -0.5)
        self.o = Linear([weights.get(s.o_proj)], env, "mlstm_o")

    @staticmethod
    def tensor_needs(spec: MlstmSpec) -> List[TensorNeed]:
        s = spec
        kd, vd = s.n_heads * s.head_dim, s.n_heads * s.v_head_dim
        return [TensorNeed(s.q_proj, (kd, s.hidden)), TensorNeed(s.k_proj, (kd, s.hidden)), TensorNeed(s.v_proj, (vd, s.hidden)),
                TensorNeed(s.gate_proj, (vd, s.hidden)), TensorNeed(s.i_gate, (s.n_heads, s.hidden)), TensorNeed(s.i_bias, (s.n_heads,)),
                TensorNeed(s.f_gate, (s.n_heads, s.hidden)), TensorNeed(s.f_bias, (s.n_heads,)), TensorNeed(s.out_norm, (vd,)),
                TensorNeed(s.o_proj, (s.hidden, vd))]

    def kv_need(self) -> Optional[GroupKey]:
        return None

    def state_need(self) -> Dict[str, StateNeed]:
        s = self.spec
        return {"S": StateNeed((s.n_heads, s.v_head_dim, s.head_dim), torch.float32), "n": StateNeed((s.n_heads, s.head_dim), torch.float32),
                "m": StateNeed((s.n_heads,), torch.float32)}

    def forward(self, x: torch.Tensor, step, memory: int, writes: bool = True) -> torch.Tensor:
        s, ws = self.spec, self.env.workspace
        if not writes:
            raise ValueError("a recurrent mixer advances its own state; it cannot read another run's")
        proj = self.proj.forward(x, out_dtype=torch.float32, tag="mlstm_in")
        q, k, v, gate, i, f = ws.columns(proj, self._bounds)[:6]
        ctx = ws.get("mlstm_ctx", x.shape[0], self.vd, self.env.dtype)
        ops.mlstm(q, k, v, gate, i, f, self.gates, ctx, state_tensor(step, memory, "S"), state_tensor(step, memory, "n"),
                  state_tensor(step, memory, "m"), step, s.n_heads, s.head_dim, s.v_head_dim, ws)
        return self.o.forward(ctx, tag="mlstm_o", slices_ok=True)       # the block adds it to the residual stream


register("mixer", "mlstm", Mlstm)
