"""A decoder assembled from a `ModelSpec`: token table, the layers in their run order, final
norm, output head.  It knows parts and the order they run in, not an architecture."""
from __future__ import annotations

import math
from pathlib import Path
from typing import Dict, List, Optional

import torch

from ..config import ModelSpec, read_config
from ..kernels import ops
from ..parts import LayerCache, StepContext, block_class, linear, model_tensor_needs, norm_class, row_transform_class, stream_part_class, weight_bytes
from ..parts.linear import activation_dtype_for
from ..parts.norm import HandedRows, ReadyRows, norm_to_hand_on
from ..parts.transform import LearnedPositions, ScaleRows
from ..weights import load_tensors, random_tensors

_DTYPES = {"bfloat16": torch.bfloat16, "bf16": torch.bfloat16, "float32": torch.float32, "fp32": torch.float32,
           torch.bfloat16: torch.bfloat16, torch.float32: torch.float32}


def compute_dtype(name) -> torch.dtype:
    try:
        return _DTYPES[name]
    except KeyError:
        raise ValueError(f"unknown dtype {name!r}: bfloat16 or float32") from None


class _Head:
    """The output head as the reader of the final norm: asked, like a part, whether it takes that norm half applied."""
    accepts_deferred_norm = True
    takes_ready_rows = True                  # ... or wholly applied by whoever wrote the rows

    def __init__(self, weight: torch.Tensor, in_dtype: torch.dtype):
        self.weight, self.in_dtype = weight, in_dtype

    def takes_handed_norm(self, n_rows: int) -> bool:
        return self.in_dtype == torch.bfloat16 and ops.gemm_bf16_takes_norm(n_rows, self.weight.shape[0], self.weight.shape[1])


class DecoderModel:
    def __init__(self, spec: ModelSpec, tensors: Dict[str, torch.Tensor], dtype: torch.dtype, device):
        self.spec, self.dtype, self.device = spec, dtype, torch.device(device)
        self.embedding = tensors[spec.embedding]
        self.lm_head = tensors[spec.lm_head]
        self.layers = [block_class(l.block)(l, tensors, dtype, device) for l in spec.layers]
        self.n_streams = int(getattr(spec, "n_streams", 1))          # copies of the residual stream the layers carry side by side
        if self.n_streams > 1:
            for l, layer in zip(spec.layers, self.layers):
                if not getattr(layer, "stream_aware", False) or getattr(layer, "n_streams", 1) != self.n_streams:
                    raise ValueError(f"the model carries {self.n_streams} copies of the residual stream, which a '{l.block}' layer does not (or not as many)")
            if any(l.after for l in spec.layers) or any(e.before is not None for e in spec.run_order):
                raise ValueError("parts between the layers change one residual stream, not several copies of it")
        self.final_norm = norm_class(spec.final_norm)(spec.final_norm, tensors, dtype, device)
        self.head_in_dtype = activation_dtype_for(self.lm_head, dtype)
        self.head = _Head(self.lm_head, self.head_in_dtype)
        self.after_embedding = [row_transform_class(t)(t, tensors, dtype, device) for t in spec.after_embedding]
        self.after_head = [row_transform_class(t)(t, tensors, dtype, device) for t in spec.after_head]
        if any(t.fetches_token_rows for t in self.after_embedding[1:]):
            raise ValueError("a transform that fetches the token rows itself must be the first one behind the token table")
        # those of them that keep a state per request: theirs follows the run order's in the list of cache needs
        self.transform_entry = {}
        for t in spec.after_embedding:
            if row_transform_class(t).cache_need(t) is not None:
                self.transform_entry[t] = len(spec.run_order) + len(self.transform_entry)
        # the longest sequence the parts behind the token table allow (a table of positions ends somewhere), or None
        self.position_limit = min((t.position_limit for t in self.after_embedding if getattr(t, "position_limit", None) is not None), default=None)
        self.run_order = spec.run_order
        for e in spec.run_order:                   # a mixer whose pages another entry reads keeps nothing but keys and values there
            if e.cache_of is not None:
                shared = getattr(getattr(self.layers[spec.run_order[e.cache_of].layer], "mixer", None), "pages_are_shared", None)
                if shared is not None:
                    shared()
        # parts that change the residual stream between layers: behind a layer (every time it runs), before a run-order entry
        self.after_layer = [[stream_part_class(t)(t, tensors, dtype, device) for t in l.after] for l in spec.layers]
        self.before_entry = [None if e.before is None else stream_part_class(e.before)(e.before, tensors, dtype, device) for e in spec.run_order]
        stream_parts = [p for parts in self.after_layer for p in parts] + [p for p in self.before_entry if p is not None]
        self.keeps_token_rows = any(getattr(p, "needs_token_rows", False) for p in stream_parts)
        self.trace = None                        # see set_trace
        self.graph_safe = all(getattr(p, "graph_safe", False) for p in (*self.layers, self.final_norm, *self.after_embedding, *self.after_head, *stream_parts))

    # ----------------------------------------------------------------------------- what it needs
    def cache_needs(self):
        """Per run-order entry: its cache need, and the entry whose cache it reads (or None); then the needs of what keeps a state behind
        the token table."""
        needs = [block_class(self.spec.layers[e.layer].block).cache_need(self.spec.layers[e.layer]) for e in self.run_order]
        needs += [row_transform_class(t).cache_need(t) for t in self.transform_entry]
        return needs, [e.cache_of for e in self.run_order] + [None] * len(self.transform_entry)

    def weight_bytes_read_per_step(self) -> int:
        """Bytes of weights one step reads when it uses every matrix once: what every part of the run order holds (a
        layer named twice is read twice), the final norm and the head; the token table is read by row and not counted."""
        return (sum(weight_bytes(self.layers[e.layer]) + weight_bytes(self.after_layer[e.layer]) for e in self.run_order)
                + weight_bytes([p for p in self.before_entry if p is not None]) + weight_bytes(self.final_norm) + weight_bytes(self.lm_head)
                + weight_bytes(self.after_embedding) + weight_bytes(self.after_head))

    # ------------------------------------------------------------------------------- the pass
    def forward(self, ctx: StepContext, cache, logit_rows: Optional[torch.Tensor], n_logit_rows: int):
        """Runs the step's rows through every layer of the run order; returns float32 logits
        [n_logit_rows, vocab] of the rows listed in `logit_rows`, or None if there are none."""
        x = torch.empty((ctx.n_rows, self.spec.hidden_size), dtype=torch.float32, device=self.device)
        trace = self.trace
        handed = self._embed(ctx, x, cache)      # the next block's first norm, where whoever wrote x could leave it half applied
        if trace is not None:
            trace("embedding", -1, x)
        if self.keeps_token_rows and "token_rows" not in ctx.memo:
            ctx.memo["token_rows"] = x.clone()
        if self.n_streams > 1:            # every copy starts as the token rows
            x = ops.streams_spread(x, torch.empty((ctx.n_rows, self.n_streams * self.spec.hidden_size), dtype=torch.float32, device=self.device), self.n_streams)
        for i, entry in enumerate(self.run_order):
            ctx.trace = None if trace is None else (lambda tag, rows, i=i: trace(tag, i, rows))
            layer, extras = self.layers[entry.layer], self.after_layer[entry.layer]
            before = self.before_entry[i]
            if before is not None:                        # (it changes x: a norm handed on by whoever wrote x last is void)
                if getattr(before, "hands_norm_on", False):
                    handed = before.forward(x, ctx, handed=None, next_reader=self._first_reader(layer))
                else:
                    before.forward(x, ctx)
                    handed = None
            if i + 1 == len(self.run_order):              # the head reads every row of the final norm, or a selection, which is not handed on
                behind = (self.final_norm, self.head) if ctx.every_row_wanted and trace is None else None
            elif self.before_entry[i + 1] is not None:    # (x changes again before anybody reads it)
                behind = None
            else:
                behind = self._first_reader(self.layers[self.run_order[i + 1].layer])
            stages = [layer, *extras]                     # the block and what follows it, each a reader of x and a writer of it
            for j, stage in enumerate(stages):
                caches = (cache.layer_cache(i),) if j == 0 else ()
                if getattr(stage, "hands_norm_on", False):
                    reader = self._first_reader(stages[j + 1]) if j + 1 < len(stages) else behind
                    handed = stage.forward(x, ctx, *caches, handed=handed, next_reader=reader)
                else:
                    stage.forward(x, ctx, *caches)
                    handed = None
            if extras and trace is not None:
                trace("layer_out", i, x)
        ctx.trace = None
        if n_logit_rows == 0:
            return None
        if self.n_streams > 1:            # the copies are added up before the final norm
            x = ops.streams_norm_shift(x, self.n_streams, torch.empty((ctx.n_rows, self.spec.hidden_size), dtype=torch.float32, device=self.device))
        logits = torch.empty((n_logit_rows, self.spec.vocab_size), dtype=torch.float32, device=self.device)
        if handed is not None and handed.norm is self.final_norm and ctx.every_row_wanted:
            normed = handed
        elif hasattr(self.final_norm, "deferred"):
            normed = self.final_norm.deferred(x, self.head_in_dtype, rows=logit_rows)
        else:
            picked = torch.empty((n_logit_rows, self.spec.hidden_size), dtype=torch.float32, device=self.device)
            normed = self.final_norm(ops.gather_rows(x, logit_rows, picked), self.head_in_dtype)
        if trace is not None:
            trace("final_norm", -1, normed if torch.is_tensor(normed) else self.final_norm(ops.gather_rows(x, logit_rows, torch.empty(
                (n_logit_rows, self.spec.hidden_size), dtype=torch.float32, device=self.device)), torch.float32))
        linear(normed, self.lm_head, logits)
        for transform in self.after_head:
            transform(logits)
        return logits

    @staticmethod
    def _first_reader(stage):
        return stage.first_reader() if getattr(stage, "hands_norm_on", False) else None

    def _embed(self, ctx: StepContext, x: torch.Tensor, cache):
        """The rows of the token table into x.  Where the first block's first norm can be taken half applied (`HandedRows`: a few
        single rows of decoding requests in bfloat16, a norm of the form g * x * rsqrt(mean square + eps), a reader whose product
        finishes it), the kernel that fetches the rows does the norm's first half too and the `HandedRows` are returned; None otherwise."""
        first = self.layers[self.run_order[0].layer] if self.run_order else None
        if (first is not None and not self.after_embedding and self.trace is None and self.dtype == torch.bfloat16 and self.before_entry[0] is None
                and getattr(first, "hands_norm_on", False) and ctx.max_seg_len == 1):         # (decode steps: the one norm kernel of a step that is all launches)
            norm = norm_to_hand_on(first.first_reader(), ctx.n_rows)
            if norm is not None:
                scaled = torch.empty((ctx.n_rows, self.spec.hidden_size), dtype=torch.bfloat16, device=self.device)
                squares = torch.empty((ctx.n_rows, 1), dtype=torch.float32, device=self.device)
                ops.embed_handing(self.embedding, ctx.tokens, x, norm.handed_weight(), scaled, squares)
                return HandedRows(norm, x, scaled, squares)
        transforms = self.after_embedding
        # a scale and a table of positions behind the token table are one kernel with the fetch, which also leaves the rows as the
        # first product reads them where they are read without a norm
        if transforms and type(transforms[-1]) is LearnedPositions and all(type(t) is ScaleRows for t in transforms[:-1]):
            reader = self._first_reader(first) if first is not None and self.before_entry[0] is None else None
            norm, part = reader if reader is not None else (None, None)
            low = None
            if getattr(norm, "is_identity", False) and getattr(part, "in_dtype", self.dtype) == torch.bfloat16:
                low = torch.empty(x.shape, dtype=torch.bfloat16, device=self.device)
            ops.embed_positioned(self.embedding, ctx.tokens, math.prod(float(t.spec.factor) for t in transforms[:-1]), transforms[-1].table, ctx.row_pos, x, low)
            return None if low is None else ReadyRows(norm, x, low)
        if transforms and transforms[0].fetches_token_rows:
            entry = self.transform_entry.get(transforms[0].spec)
            if self.keeps_token_rows and len(transforms) == 1:
                ctx.memo["token_rows"] = torch.empty_like(x)          # (the same kernel writes both)
            transforms[0].fetch(self.embedding, x, ctx, None if entry is None else cache.layer_cache(entry), ctx.memo.get("token_rows"))
            transforms = transforms[1:]
        else:
            ops.embed(self.embedding, ctx.tokens, x)
        for transform in transforms:
            if transform.needs_context:
                transform(x, ctx)
            else:
                transform(x)
        return None

    def set_trace(self, trace) -> None:
        """Debugging, as the reference's Model::set_trace (src/model/model.h): `trace(tag, run-order entry or -1, rows)` is
        called with the step's residual stream after the embedding ("embedding"), after each half of every block
        ("attn_out", "ffn_out"), behind the parts that follow a block, where a layer has such ("layer_out"), and with the normed rows that the logits are taken from ("final_norm").  While a trace is
        set no step is replayed from a captured graph."""
        self.trace = trace


def load_model(folder, dtype="bfloat16", device="cuda:0") -> DecoderModel:
    """The model a folder (config.json, model.safetensors) describes; the class of its
    configuration is chosen by config.json."""
    dtype = compute_dtype(dtype)
    config = read_config(folder)
    if hasattr(config, "fit_to_tensors"):          # an architecture some of whose parts or sizes only the tensors tell looks at their names and shapes
        from ..weights.safetensors_io import SafetensorsFile
        st = SafetensorsFile(Path(folder) / "model.safetensors")
        try:
            config = config.fit_to_tensors({name: entry.shape for name, entry in st.entries.items()})
        finally:
            st.close()
    spec = config.model_spec()
    tensors = load_tensors(folder, model_tensor_needs(spec), dtype, device, spec.ignorable_tensors)
    model = DecoderModel(spec, tensors, dtype, device)
    model.config = config
    return model


def random_model(config, seed: int, dtype="bfloat16", device="cuda:0", std: float = 0.02, draw_on_device: bool = False) -> DecoderModel:
    """A model of `config` with seeded random weights, without a folder in between.  With
    `draw_on_device` the numbers are made on the device by a formula of (seed, tensor name, element index)
    (`weights.random_init`: fast for large models, and anybody can re-make them; other numbers than the
    host generator gives for the same seed)."""
    dtype = compute_dtype(dtype)
    spec = config.model_spec()
    if draw_on_device:
        from ..weights import formula_tensors
        tensors = formula_tensors(model_tensor_needs(spec), seed, dtype, std, device)
    else:
        host = random_tensors(model_tensor_needs(spec), seed, dtype, std)
        tensors = {k: v.to(device) for k, v in host.items()}
    model = DecoderModel(spec, tensors, dtype, device)
    model.config = config
    return model
