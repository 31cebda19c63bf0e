"""Linear attention whose memory fades by a constant per head (`config.spec.LightningSpec` states the recurrence; the kernels are
`csrc/lightning.hip`).

One product with the stacked matrix [q; k; v; output gate] gives the 32-bit projections of a step's rows; one kernel takes q, k and
v through SiLU and steps every request's memories over its rows of this step, in order, from the request's state slot and back into
it; one kernel divides the heads' outputs side by side by their root mean square, multiplies by the norm's weights and the sigmoid of
the gate and stores the rows as the output product reads them.  The memories, their decays and everything between the projections
and the output product are 32-bit, whatever the compute dtype.  In bfloat16 a request's long run of rows (a prompt) is cut into
chunks that run at once (`ops.lightning_scan`); in float32 the rows are always taken one after the other, so that the bits do not
depend on how a prompt was cut into steps.

The runs of rows that belong to one request are found on the device, so a captured pass may contain the mixer."""
from __future__ import annotations

import torch

from ..cache.needs import StateNeed
from ..kernels import ops
from ..weights.loader import TensorNeed
from .attention import _pad_rows
from .base import Mixer, register_mixer
from .linear import activation_dtype_for, linear, linear_onto, takes_handed_norm


class Lightning(Mixer):
    graph_safe = True
    accepts_deferred_norm = True      # its input goes into `linear` only
    hands_norm_on = True              # `forward` takes `then`, the norm that reads the residual next
    can_overwrite = True              # `forward(..., overwrite=True)` stores its result in `residual` instead of adding onto it

    def __init__(self, spec, tensors, dtype, device):
        super().__init__(spec, tensors, dtype, device)
        s = spec
        if not 0 < s.key_dim <= ops.LIGHTNING_MAX_KEY_DIM:
            raise ValueError(f"lightning: key_dim = {s.key_dim} is outside what the kernels take (1 to {ops.LIGHTNING_MAX_KEY_DIM})")
        qk, vv = s.n_heads * s.key_dim, s.n_heads * s.value_dim
        self.q_at, self.k_at, self.v_at, self.g_at = 0, qk, 2 * qk, 2 * qk + vv
        self.w_in = _pad_rows(torch.cat([tensors[n] for n in (s.q_proj, s.k_proj, s.v_proj, s.gate_proj)], dim=0).contiguous())
        self.out_norm, self.w_o = tensors[s.out_norm], tensors[s.o_proj]
        self.powers = ops.lightning_powers(s.decay, device)
        self.in_dtype = activation_dtype_for(self.w_in, dtype)
        self.mid_dtype = activation_dtype_for(self.w_o, dtype)

    @classmethod
    def tensor_needs(cls, spec):
        s, d = spec, spec.hidden_size
        qk, vv = s.n_heads * s.key_dim, s.n_heads * s.value_dim
        return [TensorNeed(s.q_proj, (qk, d)), TensorNeed(s.k_proj, (qk, d)), TensorNeed(s.v_proj, (vv, d)), TensorNeed(s.gate_proj, (vv, d)),
                TensorNeed(s.o_proj, (d, vv)), TensorNeed(s.out_norm, (vv,), "norm")]

    @classmethod
    def cache_need(cls, spec):
        return StateNeed((spec.n_heads * spec.key_dim * spec.value_dim,), torch.float32)

    def takes_handed_norm(self, n_rows: int) -> bool:
        return self.in_dtype == torch.bfloat16 and takes_handed_norm(self.w_in, n_rows)

    def input_weight(self):
        return self.w_in

    def use_input_weight(self, view):
        self.w_in = view

    def forward(self, h, residual, ctx, cache, then=None, overwrite=False, projected=None):
        s, T = self.spec, ctx.n_rows
        vv = s.n_heads * s.value_dim
        proj = projected
        if proj is None:
            proj = torch.empty((T, self.w_in.shape[0]), dtype=torch.float32, device=ctx.device)
            linear(h, self.w_in, proj)
        seg_start, seg_len = ops.segments(ctx)
        out = torch.empty((T, vv), dtype=torch.float32, device=ctx.device)
        ops.lightning_scan(proj, (self.q_at, self.k_at, self.v_at), self.powers, seg_start, seg_len, ctx.row_slot, cache.state, out, s.n_heads, s.key_dim, s.value_dim,
                           rows_per_request=ctx.seg_len if self.dtype == torch.bfloat16 else None)
        mid = torch.empty((T, vv), dtype=self.mid_dtype, device=ctx.device)
        ops.row_norm_gate(out, proj[:, self.g_at:self.g_at + vv], self.out_norm, s.norm_eps, mid)
        if overwrite:
            linear(mid, self.w_o, residual)
            return None
        return linear_onto(mid, self.w_o, residual, then)


register_mixer("lightning", Lightning)
