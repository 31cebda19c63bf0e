"""A plain, slow statement of the Puzorax decoder on the CPU, one function per mechanism, for the tests to hold the engine
against.  It shares no code with the engine: every function takes tensors and numbers, works on one whole sequence (rows =
positions 0 .. T-1) in the dtype of its inputs (the tests use float64), and keeps no cache.

A Puzorax layer is "parallel": with h = norm(x), a norm that removes the mean, x <- x + mixer(h) + experts(h).  The mixer is one of
  latent_attention   queries straight from h, keys and values through one low-rank latent, one rotated key part shared by all
                     heads (pairs i, i + r/2), a sliding window, a learned score per head in the softmax's denominator, and a gate
                     on every channel of the heads' outputs;
  channel_delta      the delta rule with a decay of its own for every head and key channel, behind short causal convolutions.
The feed-forward is a mixture of gated experts, of which some do nothing but pass their input on; a correction per expert takes
part in the choice and not in the weights.  The token rows get the row of a hashed pair (the token before, the token) added, and
a run of layers may be walked several times: the token rows join again before every walk but the first, a vector before every one.

`store`, where a function takes it, is applied to what an engine that computes in bfloat16 would keep in bfloat16 (rows that go
into a matrix product, cached latents and keys); the identity by default.  It serves to measure what such rounding alone does.
"""
from __future__ import annotations

import torch


def same(x):
    return x


def to_bfloat16_and_back(x):
    return x.to(torch.bfloat16).to(x.dtype)


def layer_norm(x, weight, bias, eps):
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * weight + bias


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * weight


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def silu(z):
    return z * torch.sigmoid(z)


def pair_rows(tokens, mul_prev, mul_cur, buckets):
    """The row of the pair table for every token of a sequence: a hash of the token before and the token; `buckets` for the first."""
    return [buckets if i == 0 else (int(tokens[i - 1]) * mul_prev + int(t) * mul_cur) % buckets for i, t in enumerate(tokens)]


def embedding(tokens, table, pairs, mul_prev, mul_cur):
    return table[torch.as_tensor(list(tokens), dtype=torch.long)] + pairs[torch.tensor(pair_rows(tokens, mul_prev, mul_cur, pairs.shape[0] - 1))]


def rotate_half_split(x, base):
    """x [T, heads, r]: the pair (i, i + r/2) at position p is turned by p * base^(-2i/r)."""
    T, _, r = x.shape
    f = torch.tensor([float(base) ** (-2.0 * i / r) for i in range(r // 2)], dtype=torch.float64)
    a = torch.arange(T, dtype=torch.float64)[:, None] * f[None, :]
    cos, sin = torch.cos(a).to(x.dtype)[:, None, :], torch.sin(a).to(x.dtype)[:, None, :]
    u, v = x[..., :r // 2], x[..., r // 2:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin], dim=-1)


def window_mask(T, window):
    """[T, T] True where row i sees column j: 0 <= i - j < window (None: every j <= i)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    return seen if window is None else seen & (i - j < window)


def sink_softmax(scores, seen, sinks):
    """scores [H, T, T], sinks [H]: exp(score) over the keys a row sees, divided by their sum + exp(sink)."""
    scores = scores.masked_fill(~seen[None], float("-inf"))
    top = torch.maximum(scores.amax(dim=-1, keepdim=True), sinks[:, None, None])
    e = torch.exp(scores - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sinks[:, None, None] - top))


def latent_attention(h, w, m, eps, store=same):
    """m: the layer's `mixer` entry of config.json; w: its tensors by their short names."""
    T = h.shape[0]
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w["q"].T).view(T, H, d + r)
    down = h @ w["dkv"].T
    c = store(rms_norm(down[:, :rank], w["dkv.norm"], eps))
    k_rot = store(rotate_half_split(down[:, None, rank:], m["rot"]["base"]))[:, 0]
    q_plain, q_rot = store(q[..., :d]), store(rotate_half_split(q[..., d:], m["rot"]["base"]))
    seen = window_mask(T, m["mask"]["size"] if m.get("mask") else None)
    rotated = torch.einsum("thr,sr->hts", q_rot, k_rot)
    if store is same:
        k = (c @ w["uk"].T).view(T, H, d)
        v = (c @ w["uv"].T).view(T, H, dv)
        p = sink_softmax((torch.einsum("thd,shd->hts", q_plain, k) + rotated) * m["scale"], seen, w["sink"])
        o = torch.einsum("hts,shd->thd", p, v).reshape(T, H * dv)
    else:       # the same with W_uk folded into the queries and W_uv applied behind the sum over keys, which is where an engine that caches c alone rounds
        folded = store(torch.einsum("thd,hdc->thc", q_plain, w["uk"].view(H, d, rank)))
        p = sink_softmax((torch.einsum("thc,sc->hts", folded, c) + rotated) * m["scale"], seen, w["sink"])
        attended = store(torch.einsum("hts,sc->thc", store(p), c))
        o = torch.einsum("thc,hvc->thv", attended, w["uv"].view(H, dv, rank)).reshape(T, H * dv)
    return store(o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def short_conv_silu(x, taps):
    """x [T, channels], taps [channels, n]: y_t = silu(sum_j taps[:, j] x_(t - (n-1) + j)), zeros before the start."""
    n = taps.shape[1]
    padded = torch.cat([x.new_zeros(n - 1, x.shape[1]), x], dim=0)
    return silu(sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n)))


def channel_delta_rule(q, k, v, beta, g):
    """One head.  q, k, g [T, dk] (g: the decays of the memory's rows), v [T, dv], beta [T].  The memory starts at zero; a token lets
    its rows decay, moves what it holds along the key towards the value by beta, and is read with the query."""
    S = q.new_zeros(q.shape[1], v.shape[1])
    out = []
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out.append(S.T @ q[t])
    return torch.stack(out)


def channel_decays(pre, A_log, dt_bias, heads, dim):
    """pre [T, heads*dim] -> the decays [T, heads, dim]."""
    z = softplus(pre + dt_bias).view(-1, heads, dim)
    return torch.exp(-torch.exp(A_log)[None, :, None] * z)


def channel_delta(h, w, m, eps, store=same):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv_silu(h @ w["q"].T, w["q.conv"]).view(T, G, dk)
    k = short_conv_silu(h @ w["k"].T, w["k.conv"]).view(T, G, dk)
    v = short_conv_silu(h @ w["v"].T, w["v.conv"]).view(T, H, dv)
    unit = lambda x: x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)
    q, k = unit(q) * dk ** -0.5, unit(k)
    beta = torch.sigmoid(h @ w["b"].T)
    g = channel_decays(store(h @ w["a1"].T) @ w["a2"].T, w["A_log"], w["dt_bias"], H, dk)
    gate = torch.sigmoid(store(h @ w["g1"].T) @ w["g2"].T).view(T, H, dv)
    heads = []
    for i in range(H):
        j = i // (H // G)
        o = channel_delta_rule(q[:, j], k[:, j], v[:, i], beta[:, i], g[:, i])
        heads.append(rms_norm(o, w["norm"], eps) * gate[:, i])
    return store(torch.cat(heads, dim=-1)) @ w["o"].T


def route(h, router, correction, top, scale):
    """(expert numbers [T, top], weights [T, top]): softmax scores; score + correction chooses, the scores alone weigh."""
    s = torch.softmax(h @ router.T, dim=-1)
    ids = torch.topk(s + correction, top, dim=-1).indices
    chosen = torch.gather(s, 1, ids)
    return ids, chosen / (chosen.sum(dim=-1, keepdim=True) + 1e-20) * scale


def expert(h, gate, up, down, store=same):
    return store(silu(h @ gate.T) * (h @ up.T)) @ down.T


def experts(h, w, m, store=same):
    """m: the layer's `mlp` entry of config.json; w: its tensors by their short names.  The last `identity` numbers that the router
    gives are no experts: a row that chooses one gets its own h, weighed."""
    r = m["router"]
    ids, weights = route(h, w["router"], w["correction"], r["top"], r["scale"])
    out = torch.zeros_like(h)
    for e in range(r["experts"] + r["identity"]):
        mine = (weights * (ids == e)).sum(dim=-1, keepdim=True)
        rows = (ids == e).any(dim=-1)
        if rows.any():
            y = h[rows] if e >= r["experts"] else expert(h[rows], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], store)
            out[rows] += mine[rows] * y
    return out


def layer_runs(config):
    """[(layer, number of the walk that begins here, or None)] in running order."""
    n, loop = len(config["layers"]), config.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def forward(config, tensors, tokens, dtype=torch.float64, layer_outputs=None, store=same):
    """Logits [T, vocab] of a whole sequence.  config: config.json as a dict; tensors: by name.  layer_outputs: a list that
    gets the residual stream after every layer run."""
    t = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps, bigram = config["norm"]["eps"], (config.get("embedding") or {}).get("bigram")
    x0 = t["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] if bigram is None else embedding(tokens, t["embed"], t["bigram"], bigram["mul_prev"], bigram["mul_cur"])
    x = x0
    short = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}
    parts = [(short(f"l{i}.mix."), short(f"l{i}.mlp.")) for i in range(len(config["layers"]))]
    for i, walk in layer_runs(config):
        if walk is not None:
            x = x + (x0 if walk > 0 else 0) + t["loop.step"][walk]
        layer, p = config["layers"][i], f"l{i}."
        h = store(layer_norm(x, t[p + "norm1"], t[p + "norm1.b"], eps))
        mixer = {"latent_attention": latent_attention, "channel_delta": channel_delta}[layer["type"]]
        y = mixer(h, parts[i][0], layer["mixer"], eps, store)
        if layer.get("mlp") is not None:
            y = y + experts(h, parts[i][1], layer["mlp"], store)
        x = x + y
        if layer_outputs is not None:
            layer_outputs.append(x)
    return store(layer_norm(x, t["final.norm"], t["final.norm.b"], eps)) @ t["head"].T


def greedy(config, tensors, prompt, n, dtype=torch.float64):
    """The n tokens that follow `prompt` when the likeliest is taken every time (the lowest index on ties)."""
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(torch.argmax(forward(config, tensors, tokens, dtype)[-1])))
    return tokens[len(prompt):]
