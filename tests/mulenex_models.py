"""Small Mulenex configurations for the tests, their random weights, and tokens to replay.

The configurations differ from one another in every size and constant and in the order of their layers: grouped,
ungrouped and single key/value heads, value widths above and below the key width and equal to it, score caps and none,
temperatures that grow every token, every few and never, values mixed in layers that follow the first one directly, after
other layers and not at all, matrix memories with one head and with several, dense and routed feed-forwards and none,
one expert chosen, several and all, with a shared expert narrower than the routed ones, as wide, and wider by a piece that
is not whole, widths the few-row product kernels take and widths they do not.
Weights are drawn so that no mechanism hides: query and key weights about one, shares of a half, gates and their
biases spread, norm weights (stored around zero) a fifth wide, router biases half a logit wide.
"""

from __future__ import annotations

import json
import os

import torch


def attention(heads, kv_heads, dim, vdim, scale, softcap=None, temp=None, v_mix=False):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap is not None:
        mixer["softcap"] = softcap
    if temp is not None:
        mixer["q_temp"] = {"coef": temp[0], "every": temp[1]}
    if v_mix:
        mixer["v_mix"] = True
    return {"type": "attention", "mixer": mixer}


def memory(heads, dim, vdim, cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp=None):
    return dict(mixer, mlp=mlp)


# P: everything at once; a shared expert of two pieces, the second not whole; a layer between the two that mix values
P = {"architecture": "Mulenex", "vocab": 300, "width": 64, "norm": {"eps": 2e-6}, "layers": [
        layer(attention(4, 2, 16, 24, 0.3, softcap=5.0, temp=(0.5, 7), v_mix=True), moe(24, 6, 2, shared=40)),
        layer(memory(2, 16, 24, 8.0), dense(88)),
        layer(attention(6, 2, 8, 24, 0.5, v_mix=True), moe(16, 5, 3)),
        layer(attention(4, 4, 16, 8, 0.4, softcap=3.0, temp=(0.2, 16))),
     ]}
# Q: a memory first, a width the few-row products do not take, one key/value head, every expert chosen, a narrow shared expert
Q = {"architecture": "Mulenex", "vocab": 211, "width": 100, "norm": {"eps": 1e-4}, "layers": [
        layer(memory(3, 20, 36, 15.0), moe(30, 4, 4, shared=12)),
        layer(attention(3, 1, 20, 28, 0.25, temp=(1.5, 1)), dense(120)),
        layer(attention(5, 1, 12, 28, 0.3, softcap=30.0, v_mix=True), moe(20, 9, 1, shared=20)),
        layer(memory(1, 40, 12, 4.0)),
        layer(attention(2, 1, 32, 28, 0.2, softcap=8.0, temp=(0.3, 50), v_mix=True), dense(60)),
        layer(attention(2, 1, 10, 28, 0.3, v_mix=True), moe(20, 3, 2)),
     ]}
# R: shapes the matrix-core kernels take (heads and values of 64 and 32, pages of 16, experts in multiples of 32)
R = {"architecture": "Mulenex", "vocab": 400, "width": 128, "norm": {"eps": 1e-5}, "layers": [
        layer(attention(8, 2, 64, 64, 0.18, softcap=10.0, temp=(0.25, 32), v_mix=True), moe(64, 8, 2, shared=128)),
        layer(memory(4, 32, 32, 10.0), moe(32, 4, 2, shared=32)),
        layer(attention(4, 4, 32, 32, 0.25, softcap=6.0, temp=(0.4, 64)), dense(256)),
        layer(memory(2, 64, 64, 12.0), dense(192)),
        layer(attention(6, 2, 64, 64, 0.15, v_mix=True), moe(64, 8, 3, shared=64)),
        layer(attention(2, 2, 32, 64, 0.3, softcap=12.0, v_mix=True), moe(32, 16, 4)),
     ]}
# S: nothing is a multiple of four; values mixed by nobody else; a cap that bends every score; one expert in all
S = {"architecture": "Mulenex", "vocab": 97, "width": 90, "norm": {"eps": 1e-5}, "layers": [
        layer(attention(3, 3, 22, 22, 0.8, softcap=1.0, temp=(0.7, 3), v_mix=True), moe(14, 1, 1, shared=15)),
        layer(memory(3, 10, 14, 6.0), dense(50)),
        layer(attention(6, 3, 10, 14, 0.35), moe(10, 7, 2, shared=5)),
     ]}
# V: recurrent mixers alone (no pages), a memory whose keys take the shorter chunks
V = {"architecture": "Mulenex", "vocab": 150, "width": 48, "norm": {"eps": 1e-6}, "layers": [
        layer(memory(1, 136, 40, 9.0), dense(64)),
        layer(memory(2, 24, 8, 5.0), moe(32, 3, 2, shared=64)),
     ]}
CONFIGS = {"P": P, "Q": Q, "R": R, "S": S, "V": V}
SEEDS = {"P": 61, "Q": 62, "R": 63, "S": 64, "V": 65}

STD = {"": 0.1, "embed": 0.7, "router": 0.15, ".b": 0.5, "vmix": 0.5, "norm1": 0.2, "norm1b": 0.2, "norm2": 0.2, "norm2b": 0.2,
       "final.norm": 0.2, "mix.i": 0.2, "mix.f": 0.2, "mix.g": 0.2, "shared.sg": 0.2}


def make_folder(tmp, name: str, cfg=None, std=None) -> str:
    """Write model `name` (or the given config under that name) with the product's random-weights mode."""
    import paged_attention_engine_amd as pae

    out = os.path.join(str(tmp), f"mulenex_{name}")
    pae.write_model_folder(pae.read_config_dict(cfg or CONFIGS[name]), SEEDS.get(name, 5), out, std=std or STD, norm_std=0.2)
    return out


def read_folder(folder: str):
    """(config dict, tensors by name) read without the product's loader."""
    from safetensors import safe_open

    with open(os.path.join(folder, "config.json")) as handle:
        cfg = json.load(handle)
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), "pt") as handle:
        for key in handle.keys():
            tensors[key] = handle.get_tensor(key)
    return cfg, tensors


def tokens_for(name: str, length: int, salt: int = 0):
    gen = torch.Generator().manual_seed(1000 * SEEDS.get(name, 5) + length + salt)
    return torch.randint(0, CONFIGS[name]["vocab"], (length,), generator=gen).tolist()
