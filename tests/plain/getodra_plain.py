"""A plain, slow Getodra decoder: whole sequences, no cache, one function per mechanism.

This module is the oracle the engine's Getodra model is compared with.  It shares no code with the
product package: it does not import it, keeps no pages or state slots, uses no kernels, and walks
every sequence from its first token.  Everything takes a dict of tensors keyed by checkpoint name and
the plain dict of config.json, so the same functions serve any size.  `dtype` is the working
precision (float64 or float32).

The design in this module's own notation (x: residual stream [T, width]):

    N_g(x) = g x / sqrt(mean(x^2) + eps)                      (g: one number for all features)
    C_w(x)_t = x_t + sum_b w[:, taps - 1 - b] * x_{t - b}     (b = 0 .. taps - 1, zeros before the first token)
    x0 = E[tok_t] + P[t]                                      (P: a learned row per position)
    per layer:   x <- x + N_norm1(mixer(C_canon1(x)));   x <- x + N_norm2(ff(C_canon2(x)))   (if it has a feed-forward)
    logits = W_head N_final(x)

A layer may borrow another's tensors.  The mixer is latent attention (keys and values of all heads are products of
one normed vector per token, one rotated key part shared by the heads, frequencies stretched for longer contexts,
each head's output gated by one number) or linear attention with a fixed decay per head.  The feed-forward is
W_down (gelu_tanh(W_gate h) * W_up h).
"""

from __future__ import annotations

import math

import torch

# See tests/plain/danonex_plain.py: with STORAGE set, products read and write values rounded to it;
# with JITTER = (generator, size) their sums are moved at random by that relative size first.
STORAGE = None
JITTER = None


def stored(x: torch.Tensor) -> torch.Tensor:
    return x if STORAGE is None else x.to(STORAGE).to(x.dtype)


def product(h: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    y = stored(h) @ weight.T
    if JITTER is not None:
        y = y * (1.0 + JITTER[1] * torch.randn(y.shape, generator=JITTER[0], dtype=y.dtype))
    return stored(y)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """`weight` is one number for all features or one per feature."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * weight


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# --------------------------------------------------------------------------- what the layers are made of


def embed(W: dict, tokens, dtype) -> torch.Tensor:
    ids = torch.as_tensor(list(tokens), dtype=torch.long)
    return W["embed"].to(dtype)[ids] + W["pos"].to(dtype)[: len(ids)]


def owner_of(cfg: dict, index: int) -> int:
    """The layer whose tensors layer `index` uses: its own, or those of the layer it names (and so on)."""
    while cfg["layers"][index].get("weights_of") is not None:
        index = int(cfg["layers"][index]["weights_of"])
    return index


def with_its_past(x: torch.Tensor, filters: torch.Tensor) -> torch.Tensor:
    """x [T, width] plus a causal convolution of itself: channel c of token t gains sum_b filters[c, taps-1-b] x[t-b, c]."""
    T, taps = x.shape[0], filters.shape[1]
    out = x.clone()
    for b in range(min(taps, T)):
        out[b:] = out[b:] + filters[:, taps - 1 - b] * x[:T - b]
    return out


# --------------------------------------------------------------------------- latent attention


def stretched_frequencies(rot: dict):
    """(frequency of each rotated pair, float64; multiplier of cosines and sines): base^(-2i/dims), blended with a
    `factor`-th of itself by a ramp over the pair's index between the indices that turn `fast` and `slow` times
    over the original context."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
    scaling = rot.get("scaling")
    if not scaling:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])
    place = lambda turns: dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    low = max(math.floor(place(float(scaling["fast"]))), 0)
    high = min(math.ceil(place(float(scaling["slow"]))), dims - 1)
    out = f.clone()
    for i in range(f.numel()):
        ramp = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
        out[i] = f[i] / factor * ramp + f[i] * (1.0 - ramp)
    return out, 0.1 * math.log(factor) + 1.0


def rotate_halves(x: torch.Tensor, freq: torch.Tensor, magnitude: float, angle_dtype=None) -> torch.Tensor:
    """x [T, heads, dim]: features (i, i + n), i < n = len(freq), of the token at place t turn by t * freq_i and are
    multiplied by `magnitude`; the features behind pass."""
    T, n = x.shape[0], freq.numel()
    if angle_dtype is not None:  # the angle as a product of two numbers of that type
        angle = (torch.arange(T, dtype=angle_dtype)[:, None] * freq.to(angle_dtype)[None, :]).to(torch.float64)
    else:
        angle = torch.arange(T, dtype=torch.float64)[:, None] * freq[None, :]
    c = (magnitude * torch.cos(angle)).to(x.dtype)[:, None, :]
    s = (magnitude * torch.sin(angle)).to(x.dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., :n], x[..., n:2 * n]
    out[..., :n] = u * c - v * s
    out[..., n:2 * n] = v * c + u * s
    return out


def causal_softmax(q, k, v, scale: float) -> torch.Tensor:
    """q [T, D], k [T, D], v [T, V] of one head, query by query: the query at i sees the keys j <= i."""
    out = torch.zeros((q.shape[0], v.shape[1]), dtype=q.dtype)
    for i in range(q.shape[0]):
        s = (k[:i + 1] @ q[i]) * scale
        e = torch.exp(s - s.max())
        out[i] = (e[:, None] * v[:i + 1]).sum(0) / e.sum()
    return out


def latent_attention(W: dict, prefix: str, m: dict, h: torch.Tensor, eps: float, dtype, angle_dtype=None) -> torch.Tensor:
    H, D, R, V, C = (int(m[key]) for key in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    T = h.shape[0]
    w = lambda name: W[prefix + name].to(dtype)
    q = product(h, w("q")).view(T, H, D + R)
    down = product(h, w("dkv"))
    latent = stored(rms_norm(down[:, :C], w("dkv.norm"), eps))
    shared = down[:, C:].view(T, 1, R)
    k_plain = product(latent, w("uk")).view(T, H, D)
    v = product(latent, w("uv")).view(T, H, V)
    freq, magnitude = stretched_frequencies(m["rot"])
    q_turned = stored(rotate_halves(q[..., D:], freq, magnitude, angle_dtype))
    k_turned = stored(rotate_halves(shared, freq, magnitude, angle_dtype))[:, 0]
    gate = sigmoid(product(h, w("g")))
    heads = []
    for j in range(H):
        qj = torch.cat([q[:, j, :D], q_turned[:, j]], dim=-1)
        kj = torch.cat([k_plain[:, j], k_turned], dim=-1)
        heads.append(gate[:, j:j + 1] * causal_softmax(qj, kj, v[:, j], float(m["scale"])))
    return product(stored(torch.cat(heads, dim=-1)), w("o"))


# --------------------------------------------------------------------------- linear attention with a fixed decay


def decaying_readout(q, k, v, decay: float) -> torch.Tensor:
    """One head, token by token from an empty state S [D, V]: S <- decay S + k_t v_t^T; o_t = S^T q_t."""
    S = torch.zeros((q.shape[1], v.shape[1]), dtype=q.dtype)
    out = torch.zeros((q.shape[0], v.shape[1]), dtype=q.dtype)
    for t in range(q.shape[0]):
        S = decay * S + k[t][:, None] * v[t][None, :]
        out[t] = S.T @ q[t]
    return out


def lightning(W: dict, prefix: str, m: dict, h: torch.Tensor, eps: float, dtype) -> torch.Tensor:
    H, D, V = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    w = lambda name: W[prefix + name].to(dtype)
    q = silu(product(h, w("q"))).view(T, H, D)
    k = silu(product(h, w("k"))).view(T, H, D)
    v = silu(product(h, w("v"))).view(T, H, V)
    o = torch.cat([decaying_readout(q[:, j], k[:, j], v[:, j], float(m["decay"][j])) for j in range(H)], dim=-1)
    o = rms_norm(o, w("norm"), eps) * sigmoid(product(h, w("g")))
    return product(stored(o), w("o"))


# --------------------------------------------------------------------------- the model


def feed_forward(W: dict, prefix: str, mlp: dict, h: torch.Tensor, dtype) -> torch.Tensor:
    if mlp["kind"] != "dense":
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    act = stored(gelu_tanh(product(h, W[prefix + "gate"].to(dtype))) * product(h, W[prefix + "up"].to(dtype)))
    return product(act, W[prefix + "down"].to(dtype))


def forward(W: dict, cfg: dict, tokens, dtype=torch.float64, taps=None, angle_dtype=None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence.  `taps`, a list, receives the stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = embed(W, tokens, dtype)
    for i, layer in enumerate(cfg["layers"]):
        at = f"l{owner_of(cfg, i)}."
        h = with_its_past(x, W[at + "canon1"].to(dtype))
        if layer["type"] == "latent_attention":
            y = latent_attention(W, at + "mix.", layer["mixer"], h, eps, dtype, angle_dtype)
        elif layer["type"] == "lightning":
            y = lightning(W, at + "mix.", layer["mixer"], h, eps, dtype)
        else:
            raise ValueError(f"unknown layer type {layer['type']!r}")
        x = x + rms_norm(y, W[at + "norm1"].to(dtype), eps)
        if layer.get("mlp") is not None:
            h = with_its_past(x, W[at + "canon2"].to(dtype))
            x = x + rms_norm(feed_forward(W, at + "mlp.", layer["mlp"], h, dtype), W[at + "norm2"].to(dtype), eps)
        if taps is not None:
            taps.append(x.clone())
    return product(rms_norm(x, W["final.norm"].to(dtype), eps), W["head"].to(dtype))


def greedy_generate(W: dict, cfg: dict, prompt, count: int, dtype=torch.float64):
    """(the `count` tokens that follow `prompt` greedily, the logits each was chosen from [count, vocab])."""
    tokens, rows = list(prompt), []
    for _ in range(count):
        rows.append(forward(W, cfg, tokens, dtype)[-1])
        tokens.append(int(rows[-1].argmax()))
    return tokens[len(prompt):], torch.stack(rows)
