"""A plain, slow statement of the Vubenex decoder on the CPU, one function per mechanism, for the tests to hold the engine
against.  It shares no code with the engine: every function takes tensors and numbers, works on one whole sequence (rows =
positions 0 .. T-1) in the dtype of its inputs (the tests use float64), and keeps no cache.

A Vubenex model starts from scaled token rows plus a learned row per position.  Its sublayers read the residual stream as it is;
what a sublayer puts out is normed and then added.  Behind every layer a second, small input from the token itself joins the
stream.  Mixers: a linear attention whose memory fades by a constant per head, or softmax attention without a rotation whose
values are its unnormed keys, whose queries grow with the position in steps, with a one in the softmax's denominator and a gate on every
channel of the heads' outputs.

`store`, where a function takes it, is applied to what an engine that computes in bfloat16 would keep in bfloat16 (rows that go
into a matrix product, cached keys and values); the identity by default.
"""
from __future__ import annotations

import json
import math
from pathlib import Path

import torch


def same(x):
    return x


def to_bfloat16_and_back(x):
    return x.to(torch.bfloat16).to(x.dtype)


def rms_norm(x, weight, eps):
    """x / sqrt(mean(x^2) + eps) * weight over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * weight


def silu(z):
    return z / (1 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------------------------------------------ the stream's start
def token_and_position_rows(tokens, table, scale, positions):
    """The tokens' rows of the table times `scale`, plus row p of the learned positions (unscaled) for the token at position p."""
    return table[torch.tensor(tokens)] * scale + positions[:len(tokens)]


# ------------------------------------------------------------------------------------------------ mixers
def fading_memory(q, k, v, decay):
    """q, k [T, heads, d], v [T, heads, e], decay: one number per head.  Per head a memory S [d, e], zero at the start: every token
    first lets it fade, then adds k v^T, then reads it with q."""
    T, heads, d = q.shape
    out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
    for a in range(heads):
        S = torch.zeros(d, v.shape[2], dtype=q.dtype)
        for t in range(T):
            S = float(decay[a]) * S + torch.outer(k[t, a], v[t, a])
            out[t, a] = S.T @ q[t, a]
    return out


def fading_memory_as_weights(q, k, v, decay):
    """The same as a weighted sum over the rows so far: row i reads row j <= i with weight decay^(i - j) (q_i . k_j)."""
    T = q.shape[0]
    back = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(q.dtype)
    out = torch.zeros(T, q.shape[1], v.shape[2], dtype=q.dtype)
    for a in range(q.shape[1]):
        fade = torch.where(back >= 0, float(decay[a]) ** back.clamp(min=0), torch.zeros_like(back))
        out[:, a] = (fade * (q[:, a] @ k[:, a].T)) @ v[:, a]
    return out


def lightning_mixer(h, w, m, eps, store=same, memory=fading_memory_as_weights):
    """w: the mixer's tensors by their short names (q, k, v, g, norm, o); m: the mixer's entry of the configuration."""
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    q, k, v = silu(h @ w["q"].T).reshape(T, H, d), silu(h @ w["k"].T).reshape(T, H, d), silu(h @ w["v"].T).reshape(T, H, e)
    y = memory(q, k, v, m["decay"]).reshape(T, H * e)
    y = rms_norm(y, w["norm"], eps) * torch.sigmoid(h @ w["g"].T)
    return store(y) @ w["o"].T


def query_growth(position, coef, every):
    """What the query at a position is multiplied by: it grows with the logarithm of how many times `every` tokens have gone by."""
    return 1.0 + coef * math.log(math.floor((position + 1) / every) + 1)


def attention_with_an_empty_seat(q, k, v, scale):
    """Causal attention, q [T, heads, d], k [T, groups, d], v [T, groups, e]; query head a reads group a // (heads / groups).  The
    weights of a row are exp(s_j) / (1 + sum exp(s_j)): they may sum to less than one."""
    T, heads, _ = q.shape
    per = heads // k.shape[1]
    seen = torch.tril(torch.ones(T, T, dtype=torch.bool))
    out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
    for a in range(heads):
        s = ((q[:, a] @ k[:, a // per].T) * scale).masked_fill(~seen, float("-inf"))
        top = s.max(dim=1, keepdim=True).values.clamp(min=0)
        p = torch.exp(s - top)
        out[:, a] = (p / (torch.exp(-top) + p.sum(dim=1, keepdim=True))) @ v[:, a // per]
    return out


def attention_mixer(h, w, m, eps, store=same):
    """w: the mixer's tensors by their short names (q, k, q.norm, k.norm, g, o); m: the mixer's entry of the configuration."""
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q, k = (h @ w["q"].T).reshape(T, H, d), (h @ w["k"].T).reshape(T, G, d)
    v = k                                                     # the values are the keys as projected, before their norm
    q, k = rms_norm(q, w["q.norm"], eps), rms_norm(k, w["k.norm"], eps)
    if m.get("q_temp") is not None:
        q = q * torch.tensor([query_growth(p, m["q_temp"]["coef"], m["q_temp"]["every"]) for p in range(T)], dtype=q.dtype)[:, None, None]
    y = attention_with_an_empty_seat(store(q), store(k), store(v), m["scale"]).reshape(T, H * d)
    return store(y * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ------------------------------------------------------------------------------------------------ feed-forward, second input
def gated_feed_forward(h, gate, up, down, store=same):
    return store(silu(h @ gate.T) * (h @ up.T)) @ down.T


def token_side_input(x, tokens, table, layer, dim, gate, proj, norm, eps, store=same):
    """What joins the stream behind layer number `layer`: the token's `dim` columns of the second table for this layer, gated by the stream."""
    e = table[torch.tensor(tokens)][:, layer * dim:(layer + 1) * dim]
    y = store(gelu_tanh(store(x) @ gate.T) * e) @ proj.T
    return rms_norm(y, norm, eps)


# ------------------------------------------------------------------------------------------------ the model
class PlainVubenex:
    def __init__(self, folder=None, dtype=torch.float64, storage=None, config=None, tensors=None):
        if folder is not None:
            from safetensors.torch import load_file
            config, tensors = json.loads((Path(folder) / "config.json").read_text()), load_file(str(Path(folder) / "model.safetensors"))
        self.cfg, self.w = config, {k: t.to(dtype) for k, t in tensors.items()}
        self.store = same if storage is None else to_bfloat16_and_back

    def layer(self, i, x, tokens):
        """The stream behind layer i."""
        c, w, layer, eps, store = self.cfg, self.w, self.cfg["layers"][i], self.cfg["norm"]["eps"], self.store
        p = f"l{i}."
        mix = {name[len(p + "mix."):]: t for name, t in w.items() if name.startswith(p + "mix.")}
        mixer = {"lightning": lightning_mixer, "attention": attention_mixer}[layer["type"]]
        x = x + rms_norm(mixer(store(x), mix, layer["mixer"], eps, store), w[p + "norm1"], eps)
        if layer["mlp"] is not None:
            x = x + rms_norm(gated_feed_forward(store(x), w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"], store), w[p + "norm2"], eps)
        return x + token_side_input(x, tokens, w["side.embed"], i, c["token_side"]["dim"], w[p + "side.gate"], w[p + "side.proj"], w[p + "side.norm"], eps, store)

    def layer_runs(self, tokens):
        """([the stream behind every layer], logits of every position)."""
        c, w = self.cfg, self.w
        x = token_and_position_rows(tokens, w["embed"], c["embedding"]["scale"], w["pos"])
        runs = []
        for i in range(len(c["layers"])):
            x = self.layer(i, x, tokens)
            runs.append(x)
        return runs, self.store(rms_norm(x, w["final.norm"], c["norm"]["eps"])) @ w["embed"].T

    def logits(self, tokens):
        return self.layer_runs(tokens)[1]

    def greedy(self, tokens, n):
        """The n tokens that follow, the largest logit each time."""
        tokens = list(tokens)
        for _ in range(n):
            tokens.append(int(self.logits(tokens)[-1].argmax()))
        return tokens[-n:]
