"""Elementwise changes of float32 rows in place, for the two places a model may ask for one: between the token
table and the first layer (`ModelSpec.after_embedding`; a row of a learned table per position, or per pair of neighbouring tokens, among them) and on the logits
(`ModelSpec.after_head`)."""
from __future__ import annotations

import torch

from ..cache.needs import StateNeed
from ..kernels import ops
from ..weights.loader import TensorNeed
from .base import RowTransform, register_row_transform


class ScaleRows(RowTransform):
    graph_safe = True

    def __call__(self, x):
        ops.scale_rows(x, float(self.spec.factor))


class SoftCap(RowTransform):
    graph_safe = True

    def __call__(self, x):
        ops.softcap_rows(x, float(self.spec.cap))


class LearnedPositions(RowTransform):
    """x[t] += table[position of row t].  (Behind a scale, or alone, it runs as one kernel with the token table's: `DecoderModel._embed`.)"""
    graph_safe = True
    needs_context = True

    def __init__(self, spec, tensors, dtype, device):
        super().__init__(spec, tensors, dtype, device)
        self.table = tensors[spec.table]
        self.position_limit = int(spec.positions)

    @classmethod
    def tensor_needs(cls, spec):
        return [TensorNeed(spec.table, (spec.positions, spec.hidden_size))]

    def weights_read_per_step(self):
        return []                         # (a row per token, as the token table)

    def __call__(self, x, ctx):
        ops.add_position_rows(x, self.table, ctx.row_pos)


class TokenPairs(RowTransform):
    """x[t] += the row of the pair (the token before, the token), as one kernel with the token table's (`config.spec.TokenPairSpec`).  The
    token before a request's first row of a step is kept in the request's slot of a state of one number."""
    graph_safe = True
    fetches_token_rows = True

    def __init__(self, spec, tensors, dtype, device):
        super().__init__(spec, tensors, dtype, device)
        self.table = tensors[spec.table]

    @classmethod
    def tensor_needs(cls, spec):
        return [TensorNeed(spec.table, (spec.buckets + 1, spec.hidden_size))]

    @classmethod
    def cache_need(cls, spec):
        return StateNeed((1,), torch.int32)

    def weights_read_per_step(self):
        return []                         # (a row per token, as the token table)

    def fetch(self, table, x, ctx, cache, keep=None):
        """The token rows with the pairs' rows added, into x (and into `keep`)."""
        ops.embed_pairs(table, self.table, ctx.tokens, ctx.row_pos, ctx.row_slot, ops.segments(ctx), cache.state, self.spec.mul_before, self.spec.mul_token, x, keep)


register_row_transform("scale", ScaleRows)
register_row_transform("token_pairs", TokenPairs)
register_row_transform("learned_positions", LearnedPositions)
register_row_transform("softcap", SoftCap)
