"""A plain, slow Mulenex decoder: whole sequences, no cache, one function per mechanism.

This module is the oracle the engine's Mulenex model is compared with.  It shares no code with the
product package: it does not import it, keeps no pages or state slots, uses no kernels, and walks
every sequence from its first token.  Everything takes a dict of tensors keyed by checkpoint name and
the plain dict of config.json, so the same functions serve any size.  `dtype` is the working
precision (float64 or float32).

The design in this module's own notation (x: residual stream [T, width]):

    N_w(x) = (1 + w) x / sqrt(mean(x^2) + eps)
    x0_t = E[tok_t] + P(t),   P(t)_2i = sin(t 10000^(-2i/width)),  P(t)_(2i+1) = cos(the same)
    per layer:   x <- x + N_norm1b(mixer(N_norm1(x)));   x <- x + N_norm2b(ff(N_norm2(x)))   (if it has a feed-forward)
    logits = W_head N_final(x)

The mixer is softmax attention (a norm per query and key head, a temperature on the query that grows with the
position, capped scores, values mixed with those of the first such layer, a gate per head) or a matrix memory with
exponential gates.  The feed-forward is dense with biases and a squared ReLU, or experts weighted by the softmax
over the chosen logits, beside an expert that every token uses, times a gate of its own.
"""

from __future__ import annotations

import math

import torch

POSITION_BASE = 10000.0
READOUT_FLOOR = 1e-6
# With STORAGE set to a type, products read and write values rounded to it, and so does what a cache would hold;
# with JITTER = (generator, size) their sums are moved at random by that relative size first: what rounding alone does.
STORAGE = None
JITTER = None


def stored(x: torch.Tensor) -> torch.Tensor:
    return x if STORAGE is None else x.to(STORAGE).to(x.dtype)


def product(h: torch.Tensor, weight: torch.Tensor, bias=None) -> torch.Tensor:
    y = stored(h) @ weight.T
    if JITTER is not None:
        y = y * (1.0 + JITTER[1] * torch.randn(y.shape, generator=JITTER[0], dtype=y.dtype))
    return stored(y if bias is None else y + bias)


def over_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def offset_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return over_rms(x, eps) * (1.0 + weight)


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


def relu_squared(z: torch.Tensor) -> torch.Tensor:
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-z.abs()))


def soft_cap(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


# --------------------------------------------------------------------------- embedding


def position_vectors(count: int, width: int) -> torch.Tensor:
    """float64 [count, width]: sines and cosines in turn."""
    out = torch.zeros((count, width), dtype=torch.float64)
    for i in range((width + 1) // 2):
        angle = torch.arange(count, dtype=torch.float64) * POSITION_BASE ** (-2.0 * i / width)
        out[:, 2 * i] = torch.sin(angle)
        if 2 * i + 1 < width:
            out[:, 2 * i + 1] = torch.cos(angle)
    return out


def embed(W: dict, tokens, dtype) -> torch.Tensor:
    ids = torch.as_tensor(list(tokens), dtype=torch.long)
    rows = W["embed"].to(dtype)[ids]
    return rows + position_vectors(len(ids), rows.shape[1]).to(dtype)


# --------------------------------------------------------------------------- attention


def query_temperature(count: int, temp) -> torch.Tensor:
    """float64 [count]: what the query at each position is multiplied by (ones without `temp`)."""
    if not temp:
        return torch.ones(count, dtype=torch.float64)
    coef, every = float(temp["coef"]), int(temp["every"])
    return torch.tensor([1.0 + coef * math.log((p + 1) // every + 1) for p in range(count)], dtype=torch.float64)


def first_mixing_layer(cfg: dict):
    for i, layer in enumerate(cfg["layers"]):
        if layer["type"] == "attention" and layer["mixer"].get("v_mix"):
            return i
    return None


def mix_values(own: torch.Tensor, first: torch.Tensor, share) -> torch.Tensor:
    return (1.0 - share) * own + share * first


def capped_softmax_attend(q, k, v, scale: float, cap) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, V] of one sequence -> [T, H, V], query by query: the query at i sees the
    keys j <= i, with scores capped by cap tanh(s / cap) (`cap` None: as they are)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros((T, H, v.shape[-1]), dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            s = (k[:i + 1, g] @ q[i, h]) * scale
            if cap:
                s = soft_cap(s, float(cap))
            e = torch.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[:i + 1, g]
    return out


def attention(W: dict, prefix: str, m: dict, h: torch.Tensor, eps: float, dtype, first_values=None):
    """(output [T, width], the layer's own values [T, G, V] before any mixing).  `first_values`: the first mixing
    layer's values, in the layers that mix them in."""
    T = h.shape[0]
    H, G, D, V = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    get = lambda name: W[prefix + name].to(dtype)
    q = product(h, get("q")).view(T, H, D)
    k = product(h, get("k")).view(T, G, D)
    own = v = product(h, get("v")).view(T, G, V)
    q = over_rms(q, eps) * get("q.norm") * query_temperature(T, m.get("q_temp")).to(dtype)[:, None, None]
    k = over_rms(k, eps) * get("k.norm")
    if first_values is not None:
        v = mix_values(v, first_values, get("vmix"))
    o = capped_softmax_attend(stored(q), stored(k), stored(v), float(m["scale"]), m.get("softcap"))
    o = o * sigmoid(product(h, get("g")))[:, :, None]
    return product(o.reshape(T, H * V), get("o")), own


# --------------------------------------------------------------------------- matrix memory


def matrix_memory_recurrence(q, k, v, log_in, log_keep):
    """q, k [T, H, D], v [T, H, V], log_in and log_keep [T, H] -> read-outs [T, H, V].  The memory S [D, V], the key sum
    n [D] and the running maximum m all start at zero; every head is walked token by token."""
    T, H, D = q.shape
    V = v.shape[-1]
    S = torch.zeros((H, D, V), dtype=q.dtype)
    n = torch.zeros((H, D), dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    out = torch.zeros((T, H, V), dtype=q.dtype)
    for t in range(T):
        m_new = torch.maximum(log_keep[t] + m, log_in[t])
        keep, take = torch.exp(log_keep[t] + m - m_new), torch.exp(log_in[t] - m_new)
        S = keep[:, None, None] * S + take[:, None, None] * (k[t][:, :, None] * v[t][:, None, :])
        n = keep[:, None] * n + take[:, None] * k[t]
        m = m_new
        denom = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + READOUT_FLOOR
        out[t] = (S * q[t][:, :, None]).sum(1) / denom[:, None]
    return out


def matrix_memory(W: dict, prefix: str, m: dict, h: torch.Tensor, eps: float, dtype) -> torch.Tensor:
    T = h.shape[0]
    H, D, V, cap = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"])
    get = lambda name: W[prefix + name].to(dtype)
    q = product(h, get("q")).view(T, H, D) * D ** -0.5
    k = product(h, get("k")).view(T, H, D)
    v = product(h, get("v")).view(T, H, V)
    # the gates' logarithms add up over a sequence: their sums do not pass the storage type
    log_in = soft_cap(stored(h) @ get("i").T + get("i.b"), cap)
    log_keep = log_sigmoid(soft_cap(stored(h) @ get("f").T + get("f.b"), cap))
    o = over_rms(matrix_memory_recurrence(q, k, v, log_in, log_keep), eps)
    return product(o.reshape(T, H * V) * get("norm") * sigmoid(product(h, get("g"))), get("o"))


# --------------------------------------------------------------------------- feed-forwards


def dense(W: dict, prefix: str, h: torch.Tensor, dtype) -> torch.Tensor:
    get = lambda name: W[prefix + name].to(dtype)
    return product(relu_squared(stored(h) @ get("up").T + get("up.b")), get("down"), get("down.b"))


def route(z: torch.Tensor, top: int, margins=None):
    """z [T, E] router logits -> (chosen experts [T, top], their weights [T, top]: the softmax over the chosen logits
    alone).  `margins`, a list, receives [T]: the gap between the last expert chosen and the first one passed over."""
    ranked = z.sort(dim=-1, descending=True, stable=True)
    chosen = ranked.indices[:, :top]
    if margins is not None:
        gap = torch.full((z.shape[0],), float("inf"), dtype=z.dtype)
        if top < z.shape[1]:
            gap = ranked.values[:, top - 1] - ranked.values[:, top]
        margins.append(gap)
    return chosen, chosen_softmax(z, chosen)


def chosen_softmax(z: torch.Tensor, chosen: torch.Tensor) -> torch.Tensor:
    picked = z.gather(1, chosen)
    e = torch.exp(picked - picked.max(dim=-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def expert(W: dict, prefix: str, h: torch.Tensor, dtype) -> torch.Tensor:
    act = stored(silu(stored(h) @ W[prefix + "gate"].to(dtype).T) * (stored(h) @ W[prefix + "up"].to(dtype).T))
    return product(act, W[prefix + "down"].to(dtype))


def mixture(W: dict, prefix: str, mlp: dict, h: torch.Tensor, dtype, margins=None, forced=None) -> torch.Tensor:
    """`forced` [T, top]: experts to use instead of the ones `route` chooses (their weights are still this function's
    own), for comparing with an implementation in reduced precision, where a choice between two nearly equal
    logits may fall the other way."""
    z = stored(h) @ W[prefix + "router"].to(dtype).T + W[prefix + "router.b"].to(dtype)
    chosen, weights = route(z, int(mlp["router"]["top"]), margins)
    if forced is not None:
        chosen = torch.as_tensor(forced, dtype=torch.long)
        weights = chosen_softmax(z, chosen)
    out = torch.zeros_like(h)
    for e in range(int(mlp["router"]["experts"])):
        for t, place in (chosen == e).nonzero().tolist():
            out[t] = out[t] + weights[t, place] * expert(W, f"{prefix}e{e}.", h[t:t + 1], dtype)[0]
    if mlp.get("shared"):
        share = sigmoid(stored(h) @ W[prefix + "shared.sg"].to(dtype).T)
        out = out + share * expert(W, prefix + "shared.", h, dtype)
    return out


# --------------------------------------------------------------------------- the model


def forward(W: dict, cfg: dict, tokens, dtype=torch.float64, taps=None, margins=None, routing=None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence.  `taps`, a list, receives the stream after every layer;
    `margins`, a list, every routed feed-forward's margins [T] (see `route`); `routing` {layer: experts
    [T, top]} forces those layers' choices (see `mixture`)."""
    eps = float(cfg["norm"]["eps"])
    x = embed(W, tokens, dtype)
    source, first_values = first_mixing_layer(cfg), None
    for i, layer in enumerate(cfg["layers"]):
        at, m = f"l{i}.", layer["mixer"]
        norm = lambda name, y: offset_norm(y, W[at + name].to(dtype), eps)
        h = norm("norm1", x)
        if layer["type"] == "attention":
            y, own = attention(W, at + "mix.", m, h, eps, dtype, first_values if m.get("v_mix") else None)
            if i == source:
                first_values = own
        elif layer["type"] == "mlstm":
            y = matrix_memory(W, at + "mix.", m, h, eps, dtype)
        else:
            raise ValueError(f"unknown layer type {layer['type']!r}")
        x = x + norm("norm1b", y)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = norm("norm2", x)
            if mlp["kind"] == "dense":
                y = dense(W, at + "mlp.", h, dtype)
            else:
                y = mixture(W, at + "mlp.", mlp, h, dtype, margins, None if routing is None else routing.get(i))
            x = x + norm("norm2b", y)
        if taps is not None:
            taps.append(x.clone())
    return product(offset_norm(x, W["final.norm"].to(dtype), eps), W["head"].to(dtype))


def greedy_generate(W: dict, cfg: dict, prompt, count: int, dtype=torch.float64):
    """(the `count` tokens that follow `prompt` greedily, the logits each was chosen from [count, vocab])."""
    tokens, rows = list(prompt), []
    for _ in range(count):
        rows.append(forward(W, cfg, tokens, dtype)[-1])
        tokens.append(int(rows[-1].argmax()))
    return tokens[len(prompt):], torch.stack(rows)
