"""Small Vubenex model folders for the tests, written without the engine's code (config.json and a safetensors file made by
`model_folders.write_safetensors_by_hand`), so that the engine's loader reads files it did not write.

Matrices are 0.2 * N(0, 1), which makes scores and logits of order one; norm weights lie around one; the rows of positions are of the
token rows' size.  The configurations differ from one another in every size and option: memories that never fade, fade at once and
in between, with keys shorter and longer than values; one, several and as many key/value heads as query heads; queries that grow
every 3, 7 and 50 positions (also with a count that is no whole number) and queries that do not grow; layers without a feed-forward of
either type; models that begin with either type; one configuration whose sizes are multiples of nothing and two of the sizes the
matrix-core kernels take."""
from __future__ import annotations

import json
from pathlib import Path

import numpy as np
import torch

from model_folders import write_safetensors_by_hand


def _lightning(dim, vdim, decay, ff=None):
    return dict(type="lightning", mixer=dict(heads=len(decay), dim=dim, vdim=vdim, decay=list(decay)), mlp=None if ff is None else dict(kind="dense", ff=ff))


def _attention(heads, kv_heads, dim, scale, growth=None, ff=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale)
    if growth is not None:
        m["q_temp"] = dict(coef=growth[0], every=growth[1])
    return dict(type="attention", mixer=m, mlp=None if ff is None else dict(kind="dense", ff=ff))


VUBENEX_A = dict(architecture="Vubenex", vocab=300, width=64, embedding=dict(scale=3.0), norm=dict(eps=1e-5), token_side=dict(dim=10), max_positions=400, layers=[
    _lightning(8, 12, [0.9, 0.5, 1.0], 48),
    _attention(4, 2, 16, 0.2, (0.7, 7)),
    _lightning(20, 6, [0.99, 0.0]),
    _attention(6, 1, 24, 0.3, (0.4, 3), 56),
])
# Sizes the matrix-core kernels take: heads of 64 channels, everything a multiple of 16.
VUBENEX_B = dict(architecture="Vubenex", vocab=512, width=128, embedding=dict(scale=5.0), norm=dict(eps=1e-6), token_side=dict(dim=32), max_positions=1000, layers=[
    _lightning(64, 64, [0.95, 0.999]),
    _attention(4, 2, 64, 0.15, (0.5, 50), 256),
    _lightning(32, 96, [0.7, 0.98, 1.0, 0.9], 192),
])
# Sizes that are multiples of nothing; one head; queries that grow every 2.5 positions.
VUBENEX_C = dict(architecture="Vubenex", vocab=211, width=50, embedding=dict(scale=0.8), norm=dict(eps=1e-4), token_side=dict(dim=3), max_positions=357, layers=[
    _attention(3, 3, 10, 0.4, (1.1, 2.5)),
    _lightning(5, 7, [0.97], 30),
    _attention(2, 1, 33, -0.2, (-0.3, 40), 22),
])
# Begins with attention; heads of 128 and of 32 channels; queries that do not grow; keys longer than values.
VUBENEX_D = dict(architecture="Vubenex", vocab=150, width=96, embedding=dict(scale=1.0), norm=dict(eps=1e-5), token_side=dict(dim=16), max_positions=600, layers=[
    _attention(2, 1, 128, 0.1, None, 64),
    _attention(9, 3, 32, 0.25, (0.2, 1)),
    _lightning(96, 40, [0.999, 0.6, 0.3], 80),
])
CONFIGS = {"A": VUBENEX_A, "B": VUBENEX_B, "C": VUBENEX_C, "D": VUBENEX_D}
PAGE_SIZE = {"A": 4, "B": 16, "C": 3, "D": 32}


def tensor_layout(cfg):
    """(name, shape) of every tensor of a model, in the model's order."""
    d, s = cfg["width"], cfg["token_side"]["dim"]
    out = [("embed", (cfg["vocab"], d)), ("pos", (cfg["max_positions"], d)), ("side.embed", (cfg["vocab"], s * len(cfg["layers"]))), ("final.norm", (d,))]
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        x = p + "mix."
        out.append((p + "norm1", (d,)))
        qk, vv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        if layer["type"] == "lightning":
            out += [(x + "q", (qk, d)), (x + "k", (qk, d)), (x + "v", (vv, d)), (x + "g", (vv, d)), (x + "o", (d, vv)), (x + "norm", (vv,))]
        else:
            out += [(x + "q", (qk, d)), (x + "k", (m["kv_heads"] * m["dim"], d)), (x + "q.norm", (m["dim"],)), (x + "k.norm", (m["dim"],)), (x + "g", (vv, d)),
                    (x + "o", (d, vv))]
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out += [(p + "norm2", (d,)), (p + "mlp.gate", (ff, d)), (p + "mlp.up", (ff, d)), (p + "mlp.down", (d, ff))]
        out += [(p + "side.gate", (s, d)), (p + "side.proj", (d, s)), (p + "side.norm", (d,))]
    return out


def random_weights(cfg, seed, std=0.2):
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in tensor_layout(cfg):
        z = rng.standard_normal(shape)
        last = name.split(".")[-1]
        t = 1.0 + 0.1 * z if last.startswith("norm") else 0.6 * z if name in ("pos", "side.embed") else std * z
        w[name] = torch.from_numpy(np.asarray(t, dtype=np.float32))
    return w


def write_model(folder, cfg, seed=0, dtype=torch.bfloat16, std=0.2, weights=None):
    """Writes the folder; returns the float32 weights before rounding to the storage dtype."""
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg, indent=2))
    w = weights if weights is not None else random_weights(cfg, seed, std)
    write_safetensors_by_hand(folder / "model.safetensors", {n: t.to(dtype) for n, t in w.items()}, shuffle_seed=seed + 5)
    return w
