"""Small Puzorax model folders for the tests, written without the engine's code (config.json and a safetensors file made by
`model_folders.write_safetensors_by_hand`), so that the engine's loader reads files it did not write.

Matrices are 0.2 * N(0, 1), which makes scores and logits of order one; norm weights 1 + 0.1 * N(0, 1), their biases, sinks and the
decays' parameters of order one so that leaving one out shows.  The routers' logits are spread out (about 8 times N(0, 1)): which of
two experts serves a row then turns on a close call only where both count for little, and rounding cannot move a row's result far.
The configurations differ from one another in every size and option: memories with as many key heads as value heads and fewer, values
longer and shorter than keys, one tap and five, narrow middles longer and shorter than a head; latents longer and shorter than the
heads, windows shorter than a page, of one position, no multiple of anything and longer than the sequence, more heads than one matrix
instruction has columns; experts of which one, several or all serve a row, with one, three and no outputs that return their input; layers
without a feed-forward; walks from the first layer and later, over one layer, several and all, once and several times, and none; a model
without a table of pairs; one configuration whose sizes are multiples of nothing and two of sizes the matrix-core kernels take."""
from __future__ import annotations

import json
from pathlib import Path

import numpy as np
import torch

from model_folders import write_safetensors_by_hand


def _att(heads, dim, rot_dim, vdim, kv_rank, scale, base, window, mlp=None):
    return dict(type="latent_attention", mixer=dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale, rot=dict(base=base, dims=rot_dim),
                                                    mask=dict(size=window)), mlp=mlp)


def _delta(heads, kv_heads, dim, vdim, conv, mlp=None):
    return dict(type="channel_delta", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), mlp=mlp)


def _moe(experts, identity, top, ff, scale):
    return dict(kind="moe", router=dict(experts=experts, identity=identity, top=top, scale=scale), expert=dict(ff=ff))


def _pairs(buckets, mul_prev, mul_cur):
    return dict(bigram=dict(buckets=buckets, mul_prev=mul_prev, mul_cur=mul_cur))


# (the ranks of the narrow middles of every memory are in RANKS: no key of config.json names them)
PUZORAX_A = dict(architecture="Puzorax", vocab=300, width=64, norm=dict(eps=1e-5), embedding=_pairs(97, 31, 5), loop=dict(start=1, stop=3, times=2), layers=[
    _delta(4, 2, 16, 24, 4, _moe(5, 2, 2, 24, 1.5)),
    _att(4, 16, 8, 24, 32, 0.2, 1000.0, 20, _moe(3, 1, 1, 40, 0.8)),
    _delta(2, 1, 24, 18, 2),
    _att(3, 12, 4, 10, 20, 0.3, 40.0, 9, _moe(6, 0, 4, 16, 1.0)),
])
# Sizes the matrix-core kernels take: experts' rows grouped, latents of 64, keys of 96 channels.
PUZORAX_B = dict(architecture="Puzorax", vocab=512, width=128, norm=dict(eps=1e-6), embedding=_pairs(1000, 100003, 77), loop=dict(start=0, stop=1, times=3), layers=[
    _att(4, 32, 32, 64, 64, 0.15, 10000.0, 48, _moe(8, 3, 3, 64, 2.5)),
    _delta(2, 2, 64, 64, 4, _moe(4, 1, 2, 128, 1.0)),
    _att(20, 16, 16, 16, 64, 0.2, 500.0, 33),
])
# Sizes that are multiples of nothing; one tap, every expert serves every row; no walks, no pairs.
PUZORAX_C = dict(architecture="Puzorax", vocab=211, width=50, norm=dict(eps=1e-4), layers=[
    _delta(5, 5, 3, 5, 3, _moe(3, 1, 4, 10, 0.7)),
    _att(3, 6, 2, 5, 9, 0.4, 9.0, 5, _moe(2, 0, 1, 22, 3.0)),
    _delta(1, 1, 7, 9, 1),
])
# No page anywhere: memories only, walked as a whole.
PUZORAX_D = dict(architecture="Puzorax", vocab=128, width=48, norm=dict(eps=1e-5), embedding=_pairs(7, 3, 2), loop=dict(start=0, stop=2, times=2), layers=[
    _delta(2, 1, 40, 12, 3),
    _delta(3, 3, 8, 32, 5, _moe(4, 2, 2, 32, 1.2)),
])
# Attention only: a window of one position, and one longer than any sequence here; the last layer walked once.
PUZORAX_E = dict(architecture="Puzorax", vocab=260, width=64, norm=dict(eps=1e-5), embedding=_pairs(50, 1, 1), loop=dict(start=1, stop=2, times=1), layers=[
    _att(2, 8, 8, 16, 24, 0.3, 100.0, 1, _moe(4, 1, 2, 48, 2.0)),
    _att(16, 1, 8, 8, 40, 0.3, 20.0, 4096),
])
CONFIGS = {"A": PUZORAX_A, "B": PUZORAX_B, "C": PUZORAX_C, "D": PUZORAX_D, "E": PUZORAX_E}
RANKS = {"A": (6, 10), "B": (24, 40), "C": (5, 1), "D": (50, 3), "E": (1, 1)}          # (decays' middle, gates' middle)
PAGE_SIZE = {"A": 4, "B": 16, "C": 16, "D": 4, "E": 16}


def tensor_layout(cfg, ranks):
    d, V = cfg["width"], cfg["vocab"]
    out = [("embed", (V, d)), ("final.norm", (d,)), ("final.norm.b", (d,)), ("head", (V, d))]
    if cfg.get("embedding"):
        out.append(("bigram", (cfg["embedding"]["bigram"]["buckets"] + 1, d)))
    if cfg.get("loop"):
        out.append(("loop.step", (cfg["loop"]["times"], d)))
    for i, layer in enumerate(cfg["layers"]):
        p, x, m, mlp = f"l{i}.", f"l{i}.mix.", layer["mixer"], layer["mlp"]
        out += [(p + "norm1", (d,)), (p + "norm1.b", (d,))]
        H = m["heads"]
        if layer["type"] == "channel_delta":
            qk, vv, n, (ra, rg) = m["kv_heads"] * m["dim"], H * m["vdim"], m["conv"], ranks
            out += [(x + "q", (qk, d)), (x + "q.conv", (qk, n)), (x + "k", (qk, d)), (x + "k.conv", (qk, n)), (x + "v", (vv, d)), (x + "v.conv", (vv, n)), (x + "b", (H, d)),
                    (x + "A_log", (H,)), (x + "norm", (m["vdim"],)), (x + "a1", (ra, d)), (x + "a2", (H * m["dim"], ra)), (x + "dt_bias", (H * m["dim"],)), (x + "g1", (rg, d)),
                    (x + "g2", (vv, rg)), (x + "o", (d, vv))]
        else:
            r, rank = m["rot_dim"], m["kv_rank"]
            out += [(x + "q", (H * (m["dim"] + r), d)), (x + "dkv", (rank + r, d)), (x + "dkv.norm", (rank,)), (x + "uk", (H * m["dim"], rank)), (x + "uv", (H * m["vdim"], rank)),
                    (x + "sink", (H,)), (x + "g", (H * m["vdim"], d)), (x + "o", (d, H * m["vdim"]))]
        if mlp is not None:
            ff, n = mlp["expert"]["ff"], mlp["router"]["experts"] + mlp["router"]["identity"]
            for e in range(mlp["router"]["experts"]):
                out += [(f"{p}mlp.e{e}.gate", (ff, d)), (f"{p}mlp.e{e}.up", (ff, d)), (f"{p}mlp.e{e}.down", (d, ff))]
            out += [(p + "mlp.router", (n, d)), (p + "mlp.correction", (n,))]
    return out


def random_weights(cfg, ranks, seed, std=0.2):
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in tensor_layout(cfg, ranks):
        z = rng.standard_normal(shape)
        last = name.split(".")[-1]
        if last in ("norm", "norm1"):
            t = 1.0 + 0.1 * z
        elif last == "b" and len(shape) == 1:                             # a norm's bias
            t = 0.3 * z
        elif last == "sink":
            t = 1.0 + z
        elif last == "dt_bias":
            t = 0.7 * z
        elif last == "A_log":                                             # decays between about 0.2 and 0.95 a token
            t = -1.0 + 0.8 * z
        elif last == "conv":
            t = 0.5 * z
        elif last == "router":
            t = 8.0 / cfg["width"] ** 0.5 * z
        elif last == "correction":
            t = 0.05 * z
        elif last in ("a2", "g2"):                                        # (pre-activations of order one, whatever the middle's width)
            t = 1.0 / (std * (shape[1] * cfg["width"]) ** 0.5) * z
        elif last in ("bigram", "step"):
            t = 0.3 * z
        else:
            t = std * z
        w[name] = torch.from_numpy(np.asarray(t, dtype=np.float32))
    return w


def write_model(folder, cfg, ranks=(4, 4), seed=0, dtype=torch.bfloat16, std=0.2, weights=None):
    """Writes the folder; returns the float32 weights before rounding to the storage dtype."""
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg, indent=2))
    w = weights if weights is not None else random_weights(cfg, ranks, seed, std)
    write_safetensors_by_hand(folder / "model.safetensors", {n: t.to(dtype) for n, t in w.items()}, shuffle_seed=seed + 5)
    return w


def stored_weights(folder):
    """The folder's tensors as the file holds them (read with the safetensors package, not the engine's reader)."""
    from safetensors.torch import load_file
    return load_file(str(Path(folder) / "model.safetensors"))
