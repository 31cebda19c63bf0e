"""Typed configuration of the Puzorax decoder, read from its own config.json keys.

A Puzorax model is a list of parallel layers: one norm (mean removed, divided by the standard deviation, weight and bias), whose rows
both the mixer and the feed-forward (if the layer has one) read, and both results join the residual stream.  The mixer is one of
  latent_attention  queries straight from the rows, keys and values through one low-rank latent with a rotated key part that all
                    heads share (pairs (i, i + r/2)), a sliding window, a learned score per head in the softmax's denominator, a
                    gate on every channel of the heads' outputs;
  channel_delta     the delta rule with a decay for every head and key channel, behind short causal convolutions; decays and output
                    gates come through narrow middles.
The feed-forward is a mixture of SiLU-gated experts: a softmax over all of the router's outputs scores them, score plus a learned
correction chooses, the chosen scores, renormalised and scaled, weigh the outputs; the last `identity` outputs stand for experts that
return their input.  The token's row gets the row of a hashed pair (the token before, the token) added.  A run of layers may be walked
several times with the same weights (`loop`): every walk keeps caches and states of its own; before every walk but the first the
token rows are added to the stream, before every walk a vector of its own.

config.json:
    architecture  "Puzorax"
    vocab, width  sizes of the token table
    norm          {eps}: every norm of the model
    embedding     {bigram: {buckets, mul_prev, mul_cur}} (optional)
    layers        [{type: "latent_attention", mixer: {heads, dim, rot_dim, vdim, kv_rank, scale, rot: {base, dims}, mask: {size}}, mlp},
                   {type: "channel_delta", mixer: {heads, kv_heads, dim, vdim, conv}, mlp}]
                  mlp: null | {kind: "moe", router: {experts, top, identity, scale}, expert: {ff}}   (mask may be absent)
    loop          optional {start, stop, times}: layers start .. stop - 1 are walked `times` times in a row
    max_positions optional: the longest sequence (default 131072)
The ranks of the narrow middles are in no key: the tensors `a1` and `g1` of a layer tell them (`fit_to_tensors`), or the mixer's
optional keys `decay_rank` and `gate_rank` where there is no folder to look into (default: the key size).
Tensors: embed, bigram, loop.step, final.norm, final.norm.b, head, and per layer i under "l<i>.": norm1, norm1.b,
mix.{q,dkv,dkv.norm,uk,uv,sink,g,o} or mix.{q,k,v, q.conv,k.conv,v.conv, b,A_log,norm,a1,a2,dt_bias,g1,g2,o},
mlp.{router, correction, e<j>.{gate,up,down}}.
"""
from __future__ import annotations

import dataclasses
from dataclasses import dataclass
from typing import Optional, Tuple, Union

from .errors import ConfigError
from .fekorax import _int, _number
from .registry import register_architecture
from .spec import AddRowsSpec, GatedDeltaSpec, LatentAttentionSpec, LayerNormSpec, LayerSpec, ModelSpec, RotarySpec, RoutedExpertsSpec, RunEntry, TokenPairSpec


@dataclass(frozen=True)
class PuzoraxAttention:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    window: Optional[int] = None


@dataclass(frozen=True)
class PuzoraxDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int
    gate_rank: int


@dataclass(frozen=True)
class PuzoraxExperts:
    ff: int
    experts: int
    top: int
    identity: int
    scale: float


@dataclass(frozen=True)
class PuzoraxLayer:
    mixer: Union[PuzoraxAttention, PuzoraxDelta]
    mlp: Optional[PuzoraxExperts]


@dataclass(frozen=True)
class PuzoraxPairs:
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass(frozen=True)
class PuzoraxLoop:
    start: int
    stop: int
    times: int


def _attention(m, where):
    rot_dim, rot = _int(m, "rot_dim", where, least=2), m.get("rot")
    dims = _int(rot, "dims", where + ", rot", least=2)
    if dims != rot_dim or rot_dim % 2:
        raise ConfigError(f"config.json: {where}: rot.dims and rot_dim must be the same even number")
    mask = m.get("mask")
    return PuzoraxAttention(_int(m, "heads", where), _int(m, "dim", where), rot_dim, _int(m, "vdim", where), _int(m, "kv_rank", where),
                            _number(m, "scale", where, positive=False), _number(rot, "base", where + ", rot"), None if mask is None else _int(mask, "size", where + ", mask"))


def _delta(m, where):
    heads, kv_heads, dim = _int(m, "heads", where), _int(m, "kv_heads", where), _int(m, "dim", where)
    if heads % kv_heads:
        raise ConfigError(f"config.json: {where}: 'heads' must be a multiple of 'kv_heads'")
    rank = lambda key: dim if m.get(key) is None else _int(m, key, where)
    return PuzoraxDelta(heads, kv_heads, dim, _int(m, "vdim", where), _int(m, "conv", where), rank("decay_rank"), rank("gate_rank"))


@dataclass(frozen=True)
class PuzoraxConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[PuzoraxLayer, ...]
    pairs: Optional[PuzoraxPairs] = None
    loop: Optional[PuzoraxLoop] = None
    max_positions: int = 131072
    architecture: str = "Puzorax"

    @classmethod
    def from_dict(cls, cfg: dict) -> "PuzoraxConfig":
        if not isinstance(cfg.get("layers"), list) or not cfg["layers"]:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(cfg["layers"]):
            where = f"layer {i}"
            if not isinstance(entry, dict) or not isinstance(entry.get("mixer"), dict):
                raise ConfigError(f"config.json: {where} needs a 'type' and a 'mixer'")
            readers = {"latent_attention": _attention, "channel_delta": _delta}
            if entry.get("type") not in readers:
                raise ConfigError(f"config.json: {where} has the unknown type {entry.get('type')!r} ({', '.join(readers)})")
            mixer, mlp = readers[entry["type"]](entry["mixer"], where), entry.get("mlp")
            if mlp is not None:
                w = where + ", mlp"
                if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
                    raise ConfigError(f"config.json: {where} has a feed-forward of an unknown kind (moe, or null for none)")
                router = mlp.get("router")
                experts, top = _int(router, "experts", w + ", router"), _int(router, "top", w + ", router")
                identity = 0 if router.get("identity") is None else _int(router, "identity", w + ", router", least=0)
                if top > experts + identity:
                    raise ConfigError(f"config.json: {w}: 'top' cannot exceed the number of experts")
                mlp = PuzoraxExperts(_int(mlp.get("expert"), "ff", w + ", expert"), experts, top, identity,
                                     1.0 if router.get("scale") is None else _number(router, "scale", w + ", router", positive=False))
            layers.append(PuzoraxLayer(mixer, mlp))
        pairs, loop, max_positions = (cfg.get("embedding") or {}).get("bigram"), cfg.get("loop"), cfg.get("max_positions")
        if pairs is not None:
            pairs = PuzoraxPairs(*(_int(pairs, key, "'embedding.bigram'", least=least) for key, least in (("buckets", 1), ("mul_prev", 0), ("mul_cur", 0))))
        if loop is not None:
            loop = PuzoraxLoop(_int(loop, "start", "'loop'", least=0), _int(loop, "stop", "'loop'", least=0), _int(loop, "times", "'loop'", least=1))
            if not loop.start < loop.stop <= len(layers):
                raise ConfigError("config.json: 'loop' needs 0 <= start < stop <= the number of layers")
        return cls(vocab=_int(cfg, "vocab", "the model"), width=_int(cfg, "width", "the model"), norm_eps=_number(cfg.get("norm"), "eps", "'norm'"), layers=tuple(layers),
                   pairs=pairs, loop=loop, max_positions=131072 if max_positions is None else _int(cfg, "max_positions", "the model"))

    def to_dict(self) -> dict:
        """config.json content that `from_dict` reads back to an equal configuration."""
        layers = []
        for layer in self.layers:
            m, mlp = layer.mixer, layer.mlp
            if isinstance(m, PuzoraxAttention):
                kind, mixer = "latent_attention", dict(heads=m.heads, dim=m.dim, rot_dim=m.rot_dim, vdim=m.vdim, kv_rank=m.kv_rank, scale=m.scale,
                                                       rot=dict(base=m.rot_base, dims=m.rot_dim))
                if m.window is not None:
                    mixer["mask"] = dict(size=m.window)
            else:
                kind, mixer = "channel_delta", dataclasses.asdict(m)
            if mlp is not None:
                mlp = dict(kind="moe", router=dict(experts=mlp.experts, top=mlp.top, identity=mlp.identity, scale=mlp.scale), expert=dict(ff=mlp.ff))
            layers.append(dict(type=kind, mixer=mixer, mlp=mlp))
        out = dict(architecture=self.architecture, vocab=self.vocab, width=self.width, norm=dict(eps=self.norm_eps), layers=layers, max_positions=self.max_positions)
        if self.pairs is not None:
            out["embedding"] = dict(bigram=dataclasses.asdict(self.pairs))
        if self.loop is not None:
            out["loop"] = dataclasses.asdict(self.loop)
        return out

    def fit_to_tensors(self, shapes) -> "PuzoraxConfig":
        """The configuration of a folder with these tensors (shapes by name): the ranks of the narrow middles are theirs."""
        layers = []
        for i, layer in enumerate(self.layers):
            if isinstance(layer.mixer, PuzoraxDelta):
                rank = lambda name, otherwise: int(shapes[f"l{i}.mix.{name}"][0]) if len(shapes.get(f"l{i}.mix.{name}", ())) == 2 else otherwise
                layer = dataclasses.replace(layer, mixer=dataclasses.replace(layer.mixer, decay_rank=rank("a1", layer.mixer.decay_rank), gate_rank=rank("g1", layer.mixer.gate_rank)))
            layers.append(layer)
        return dataclasses.replace(self, layers=tuple(layers))

    # ------------------------------------------------------------------------------------ as parts
    def layer_order(self):
        """[(layer, number of the walk that begins with this entry, or None)] in the order the layers run."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        lp = self.loop
        order = [(i, None) for i in range(lp.start)]
        for t in range(lp.times):
            order += [(i, t if i == lp.start else None) for i in range(lp.start, lp.stop)]
        return order + [(i, None) for i in range(lp.stop, n)]

    def model_spec(self) -> ModelSpec:
        eps, width = self.norm_eps, self.width
        specs = []
        for i, layer in enumerate(self.layers):
            p, x, a = f"l{i}.", f"l{i}.mix.", layer.mixer
            if isinstance(a, PuzoraxAttention):
                mixer = LatentAttentionSpec(hidden_size=width, n_heads=a.heads, head_dim=a.dim, rotary_dim=a.rot_dim, value_dim=a.vdim, q_rank=0, kv_rank=a.kv_rank,
                                            scale=a.scale, norm_eps=eps, dq_proj="", dq_norm="", uq_proj="", q_proj=x + "q", dkv_proj=x + "dkv", dkv_norm=x + "dkv.norm",
                                            uk_proj=x + "uk", uv_proj=x + "uv", o_proj=x + "o", position=RotarySpec(a.rot_dim, a.rot_base), window=a.window, sinks=x + "sink",
                                            output_gate=x + "g")
            else:
                mixer = GatedDeltaSpec(hidden_size=width, n_heads=a.heads, n_kv_heads=a.kv_heads, key_dim=a.dim, value_dim=a.vdim, conv_taps=a.conv, norm_eps=eps,
                                       q_proj=x + "q", k_proj=x + "k", v_proj=x + "v", q_conv=x + "q.conv", k_conv=x + "k.conv", v_conv=x + "v.conv", a_proj=x + "a2",
                                       a_log=x + "A_log", dt_bias=x + "dt_bias", b_proj=x + "b", gate_proj=x + "g2", out_norm=x + "norm", o_proj=x + "o", channel_decay=True,
                                       a_down=x + "a1", a_rank=a.decay_rank, gate_down=x + "g1", gate_rank=a.gate_rank, gate_activation="sigmoid")
            ff, m = None, p + "mlp."
            if layer.mlp is not None:
                e, r = range(layer.mlp.experts), layer.mlp
                ff = RoutedExpertsSpec(hidden_size=width, intermediate_size=r.ff, n_experts=r.experts, top=r.top, router=m + "router", gate_projs=tuple(f"{m}e{j}.gate" for j in e),
                                       up_projs=tuple(f"{m}e{j}.up" for j in e), down_projs=tuple(f"{m}e{j}.down" for j in e), score="softmax", renormalize=True, weigh="output",
                                       renormalize_floor=1e-20, correction=m + "correction", n_identity=r.identity, weight_scale=r.scale)
            specs.append(LayerSpec(mixer=mixer, feed_forward=ff, mixer_norm=LayerNormSpec(width, eps, p + "norm1", p + "norm1.b"), feed_forward_norm=None, block="parallel"))
        times = self.loop.times if self.loop is not None else 0
        run_order = tuple(RunEntry(i, before=None if walk is None else AddRowsSpec(width, "loop.step", times, walk, token_rows=walk > 0)) for i, walk in self.layer_order())
        pairs = () if self.pairs is None else (TokenPairSpec(width, self.pairs.buckets, self.pairs.mul_prev, self.pairs.mul_cur, "bigram"),)
        return ModelSpec(architecture=self.architecture, vocab_size=self.vocab, hidden_size=width, max_positions=self.max_positions, embedding="embed",
                         final_norm=LayerNormSpec(width, eps, "final.norm", "final.norm.b"), lm_head="head", layers=tuple(specs), run_order=run_order, after_embedding=pairs)


register_architecture("Puzorax", PuzoraxConfig, model_type="puzorax")
