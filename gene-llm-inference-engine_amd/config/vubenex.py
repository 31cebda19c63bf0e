"""Typed configuration of the Vubenex decoder, read from its own config.json keys.

A Vubenex model is a list of layers of two kinds, in any order.  The sublayers read the residual stream as it is; what a sublayer
puts out passes an RMS norm and is then added.  The mixer is either linear attention whose memory fades by a constant per head
(`lightning`), or grouped-query attention (`attention`) without a rotation: a norm on every query and key head, the unnormed keys
as values, queries that grow with the position in steps, a score scale of its own, a one in the softmax's denominator and a gate on every
channel of the heads' outputs.  The feed-forward, if the layer has one, is gated with SiLU.  Behind every layer the stream takes a
second, small input from the token itself (a slice of a second token table, gated by the stream, projected, normed and added).
The token table is scaled on the way in, where a learned vector per position joins it, and serves unscaled as the output head.

config.json:
    architecture  "Vubenex"
    vocab, width  sizes of the token table
    embedding     {scale}
    norm          {eps}: every RMS norm of the model
    layers        [{type: "lightning" | "attention", mixer: {...}, mlp: null | {kind: "dense", ff}}]
      lightning mixer  {heads, dim, vdim, decay: [one number per head]}
      attention mixer  {heads, kv_heads, dim, vdim, scale, q_temp: {coef, every}}     (vdim = dim; q_temp may be absent or null)
    token_side    {dim}: every layer reads `dim` columns of the second token table, layer i its own
    max_positions rows of the table of positions and so the longest sequence
Tensors: embed, pos, side.embed, final.norm, and per layer i under "l<i>.": norm1, (norm2,) mix.{q,k,v,g,norm,o} or
mix.{q,k,q.norm,k.norm,g,o}, (mlp.{gate,up,down},) side.{gate,proj,norm}.
"""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Optional, Tuple

from .errors import ConfigError
from .fekorax import _int, _number
from .registry import register_architecture
from .spec import (AttentionSpec, LayerSpec, LearnedPositionsSpec, LightningSpec, ModelSpec, NoNormSpec, RmsNormSpec, RunEntry, ScaleSpec, SwiGluSpec,
                   TokenSideInputSpec)


@dataclass(frozen=True)
class VubenexLightning:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class VubenexAttention:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    growth: Optional[Tuple[float, float]] = None          # (coef, every)


@dataclass(frozen=True)
class VubenexLayer:
    mixer: object                        # VubenexLightning or VubenexAttention
    ff: Optional[int] = None             # the feed-forward's inner size, or None for a layer without one


@dataclass(frozen=True)
class VubenexConfig:
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    layers: Tuple[VubenexLayer, ...]
    side_dim: int
    max_positions: int
    architecture: str = "Vubenex"

    # ------------------------------------------------------------------------------------- reading
    @classmethod
    def from_dict(cls, cfg: dict) -> "VubenexConfig":
        if not isinstance(cfg.get("layers"), list) or not cfg["layers"]:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(cfg["layers"]):
            where = f"layer {i}"
            if not isinstance(entry, dict) or not isinstance(entry.get("mixer"), dict):
                raise ConfigError(f"config.json: {where} needs a 'type' and a 'mixer'")
            m, kind = entry["mixer"], entry.get("type")
            if kind == "lightning":
                mixer = cls._lightning(m, where)
            elif kind == "attention":
                mixer = cls._attention(m, where)
            else:
                raise ConfigError(f"config.json: {where} has the unknown type {kind!r} (lightning or attention)")
            mlp, ff = entry.get("mlp"), None
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind", "dense") != "dense":
                    raise ConfigError(f"config.json: {where} has a feed-forward of an unknown kind (dense, or null for none)")
                ff = _int(mlp, "ff", where + ", mlp")
            layers.append(VubenexLayer(mixer, ff))
        return cls(vocab=_int(cfg, "vocab", "the model"), width=_int(cfg, "width", "the model"),
                   embedding_scale=_number(cfg.get("embedding"), "scale", "'embedding'", positive=False), norm_eps=_number(cfg.get("norm"), "eps", "'norm'"),
                   layers=tuple(layers), side_dim=_int(cfg.get("token_side"), "dim", "'token_side'"), max_positions=_int(cfg, "max_positions", "the model"))

    @staticmethod
    def _lightning(m, where):
        heads, decay = _int(m, "heads", where), m.get("decay")
        if not isinstance(decay, list) or len(decay) != heads or any(isinstance(d, bool) or not isinstance(d, (int, float)) or not 0 <= d <= 1 for d in decay):
            raise ConfigError(f"config.json: {where} needs 'decay', a number between 0 and 1 for each of its {heads} heads")
        return VubenexLightning(heads, _int(m, "dim", where), _int(m, "vdim", where), tuple(float(d) for d in decay))

    @staticmethod
    def _attention(m, where):
        heads, kv_heads, dim = _int(m, "heads", where), _int(m, "kv_heads", where), _int(m, "dim", where)
        if heads % kv_heads:
            raise ConfigError(f"config.json: {where}: 'heads' must be a multiple of 'kv_heads'")
        if m.get("vdim") is not None and _int(m, "vdim", where) != dim:
            raise ConfigError(f"config.json: {where}: 'vdim' must equal 'dim', the values are the keys")
        growth = None
        if m.get("q_temp") is not None:
            w = where + ", q_temp"
            growth = (_number(m["q_temp"], "coef", w, positive=False), _number(m["q_temp"], "every", w))
        return VubenexAttention(heads, kv_heads, dim, _number(m, "scale", where, positive=False), growth)

    def fit_to_tensors(self, shapes) -> "VubenexConfig":
        """The configuration of a folder whose tensors have these shapes (name -> shape): the table of positions says how many there are."""
        table = shapes.get("pos")
        return self if table is None or len(table) != 2 else replace(self, max_positions=int(table[0]))

    def to_dict(self) -> dict:
        """config.json content that `from_dict` reads back to an equal configuration."""
        layers = []
        for layer in self.layers:
            m = layer.mixer
            if isinstance(m, VubenexLightning):
                mixer, kind = dict(heads=m.heads, dim=m.dim, vdim=m.vdim, decay=list(m.decay)), "lightning"
            else:
                mixer, kind = dict(heads=m.heads, kv_heads=m.kv_heads, dim=m.dim, vdim=m.dim, scale=m.scale), "attention"
                if m.growth is not None:
                    mixer["q_temp"] = dict(coef=m.growth[0], every=m.growth[1])
            layers.append(dict(type=kind, mixer=mixer, mlp=None if layer.ff is None else dict(kind="dense", ff=layer.ff)))
        return dict(architecture=self.architecture, vocab=self.vocab, width=self.width, embedding=dict(scale=self.embedding_scale),
                    norm=dict(eps=self.norm_eps), layers=layers, token_side=dict(dim=self.side_dim), max_positions=self.max_positions)

    # ------------------------------------------------------------------------------------ as parts
    def model_spec(self) -> ModelSpec:
        eps, width = self.norm_eps, self.width
        norm = lambda name: RmsNormSpec(width, eps, name)
        specs = []
        for i, layer in enumerate(self.layers):
            p, m = f"l{i}.", layer.mixer
            x = p + "mix."
            if isinstance(m, VubenexLightning):
                mixer = LightningSpec(hidden_size=width, n_heads=m.heads, key_dim=m.dim, value_dim=m.vdim, decay=m.decay, norm_eps=eps, q_proj=x + "q",
                                      k_proj=x + "k", v_proj=x + "v", gate_proj=x + "g", out_norm=x + "norm", o_proj=x + "o")
            else:
                mixer = AttentionSpec(hidden_size=width, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, q_proj=x + "q", k_proj=x + "k", v_proj="",
                                      o_proj=x + "o", scale=m.scale, q_norm=x + "q.norm", k_norm=x + "k.norm", qk_norm_eps=eps, values_are_keys=True,
                                      query_growth=m.growth, sink_score=0.0, output_gate=x + "g")
            ff = None if layer.ff is None else SwiGluSpec(width, layer.ff, p + "mlp.gate", p + "mlp.up", p + "mlp.down", activation="silu")
            side = TokenSideInputSpec(hidden_size=width, vocab_size=self.vocab, dim=self.side_dim, table="side.embed", table_width=self.side_dim * len(self.layers),
                                      first_column=i * self.side_dim, gate_proj=p + "side.gate", out_proj=p + "side.proj", norm=norm(p + "side.norm"),
                                      activation="gelu_tanh")
            specs.append(LayerSpec(mixer=mixer, feed_forward=ff, mixer_norm=NoNormSpec(width), feed_forward_norm=None if ff is None else NoNormSpec(width),
                                   block="sandwich", mixer_post_norm=norm(p + "norm1"), feed_forward_post_norm=None if ff is None else norm(p + "norm2"), after=(side,)))
        return ModelSpec(architecture=self.architecture, vocab_size=self.vocab, hidden_size=width, max_positions=self.max_positions, embedding="embed",
                         final_norm=norm("final.norm"), lm_head="embed", layers=tuple(specs), run_order=tuple(RunEntry(i) for i in range(len(self.layers))),
                         after_embedding=(ScaleSpec(self.embedding_scale), LearnedPositionsSpec(width, self.max_positions, "pos")))


register_architecture(VubenexConfig.architecture, VubenexConfig, model_type="vubenex")
