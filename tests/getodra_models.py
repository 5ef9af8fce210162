"""Small Getodra configurations for the tests, their random weights, and tokens to replay.

The configurations differ from one another in every size and constant and in the order of their layers: either mixer
first, several of a kind in a row, layers that borrow an earlier layer's tensors (also one that itself borrows, and one of
each kind), layers without a feed-forward, convolutions of one to six taps, one head and several (more than a column
tile of the matrix cores holds), key widths that take the recurrence in chunks of either length, value widths above and
below the key width, decays close to one, one, one half and near zero, latents the matrix-core kernel takes and latents
it does not, heads whose keys and values long runs form and heads whose they do not, stretched frequencies (where some pairs keep theirs, some are blended and some divided) and plain ones,
widths the few-row product kernels take and widths they do not.  Weights are drawn so that no mechanism hides: filters
a third of a unit wide, the latent norms and the lightning norms a fifth about one, the norms' single numbers spread
about one, gates wide enough to open and shut, queries and keys wide enough that attention is peaked.
"""

from __future__ import annotations

import json
import os

import torch


def lightning(heads, dim, vdim, decay):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=10000.0, scaling=None):
    rot = {"base": base, "dims": rot_dim}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                                                  "scale": scale, "rot": rot}}


def layer(mixer, ff=None, weights_of=None):
    out = {**mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


_P_LATENT = latent(4, 16, 8, 24, 40, 0.3, base=500.0, scaling=(8.0, 64, 8.0, 1.0))
_P_LIGHT = lightning(2, 16, 24, (0.6, 0.995))
P = {"architecture": "Getodra", "vocab": 300, "width": 64, "max_positions": 256, "norm": {"eps": 2e-6}, "canon": {"taps": 4},
     "layers": [layer(_P_LIGHT, 40), layer(_P_LATENT, 72), layer(_P_LATENT, 72, weights_of=1), layer(_P_LIGHT, 40, weights_of=0),
                layer(lightning(3, 40, 8, (0.05, 1.0, 0.9)))]}
# a width the few-row products do not take, three taps, key widths of both chunk lengths, a borrower of a borrower
_Q_LATENT = latent(3, 20, 12, 36, 28, 0.25, base=50.0)
Q = {"architecture": "Getodra", "vocab": 211, "width": 100, "max_positions": 200, "norm": {"eps": 1e-5}, "canon": {"taps": 3},
     "layers": [layer(_Q_LATENT), layer(lightning(2, 144, 20, (0.98, 0.5)), 60), layer(_Q_LATENT, weights_of=0),
                layer(lightning(1, 72, 100, (0.999,)), 30), layer(_Q_LATENT, weights_of=2)]}
# latents the matrix-core kernel takes, with more heads than one column tile holds and with fewer; two taps
R = {"architecture": "Getodra", "vocab": 400, "width": 128, "max_positions": 512, "norm": {"eps": 1e-5}, "canon": {"taps": 2},
     "layers": [layer(latent(18, 16, 32, 16, 64, 0.2, base=3000.0, scaling=(4.0, 128, 16.0, 2.0)), 256),
                layer(lightning(4, 32, 32, (0.5, 0.9, 0.99, 0.9999)), 128), layer(latent(6, 32, 32, 32, 128, 0.2, base=100.0), 96),
                layer(lightning(2, 128, 64, (0.7, 0.97)), 64)]}
# nothing is a multiple of four; more taps than the register path holds
S = {"architecture": "Getodra", "vocab": 97, "width": 90, "max_positions": 160, "norm": {"eps": 1e-5}, "canon": {"taps": 6},
     "layers": [layer(lightning(3, 10, 14, (0.8, 0.3, 0.96)), 50), layer(latent(5, 18, 10, 22, 30, 0.35, base=70.0), 34)]}
# one tap (nothing is kept), latent attention alone
U = {"architecture": "Getodra", "vocab": 120, "width": 48, "max_positions": 192, "norm": {"eps": 1e-6}, "canon": {"taps": 1},
     "layers": [layer(latent(2, 8, 4, 12, 20, 0.5, base=200.0, scaling=(2.0, 32, 4.0, 1.0)), 56)]}
CONFIGS = {"P": P, "Q": Q, "R": R, "S": S, "U": U}
SEEDS = {"P": 41, "Q": 42, "R": 43, "S": 44, "U": 45}

STD = {"": 0.08, "embed": 0.5, "pos": 0.3, "canon1": 0.35, "canon2": 0.35, "mix.q": 0.15, "dkv": 0.15, "uk": 0.25, "mix.g": 0.3}


def make_folder(tmp, name: str, cfg=None, std=None) -> str:
    """Write model `name` (or the given config under that name) with the product's random-weights mode."""
    import paged_attention_engine_amd as pae

    out = os.path.join(str(tmp), f"getodra_{name}")
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
