"""Getodra: a decoder whose layers are listed one by one in config.json, with a norm on every sublayer's output and a
short convolution over time in front of every sublayer; some layers borrow an earlier layer's tensors.

config.json keys (every size and every constant that may differ between models is read from here):

    architecture      "Getodra"
    vocab, width      vocabulary and residual width
    max_positions     rows of the table `pos` of learned positions
    norm.eps          eps of every RMS norm of the model (inside the root)
    canon.taps        taps of the convolutions in front of the sublayers
    layers[i]         type: "latent_attention" | "lightning"; mixer: the mixer's sizes; mlp: {kind: "dense", ff} | null;
                      weights_of: j (optional): the layer has no tensors of its own and uses layer j's
      latent_attention  heads, dim (unrotated), rot_dim (rotated), vdim, kv_rank, scale,
                        rot {base, dims, scaling {factor, original, fast, slow} (optional)}
      lightning         heads, dim, vdim, decay [heads]

Fixed by the design, so constants of this file: x <- x + norm1(mixer(c1(x))), then x <- x + norm2(mlp(c2(x))), where
c(x) = x + conv(x) per channel and a norm's weight is a single number; the embedding's row plus the position's row,
neither scaled.  Latent attention: keys and values of the heads are products of one normed latent per token, one rotated
key part is shared by the heads; pairs (i, i + dims / 2); with rot.scaling the frequencies are stretched by a ramp and
cosines and sines are multiplied by 0.1 ln(factor) + 1; each head's output is gated by the sigmoid of one number.
Lightning attention: SiLU on q, k and v, a fixed decay per head, a norm over all heads together, a sigmoid gate.
Feed-forwards are W_down (gelu_tanh(W_gate h) * W_up h).
Tensor names: `embed`, `pos`, `final.norm`, `head`, and below `l<i>.`: `norm1`, `norm2` (single numbers), `canon1`,
`canon2` [width, taps], `mix.q|dkv|dkv.norm|uk|uv|g|o` (latent), `mix.q|k|v|g|o|norm` (lightning), `mlp.gate|up|down`.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple

from ..config.model_config import (ConfigError, FeedForwardSpec, FixedDecaySpec, FrequencyRamp, InputConvSpec,
                                   LatentMixerSpec, LayerSpec, ModelPlan, NormSpec, PositionSpec, ScheduleEntry, positive,
                                   require)
from ..config.registry import register_architecture

ARCHITECTURE = "Getodra"
FEED_FORWARD_ACTIVATION = "gelu_tanh"
LATENT, LIGHTNING = "latent_attention", "lightning"
_SIZES = {LATENT: ("heads", "dim", "rot_dim", "vdim", "kv_rank"), LIGHTNING: ("heads", "dim", "vdim")}


def _section(cfg: Mapping[str, Any], key: str, where: str) -> Mapping[str, Any]:
    value = cfg.get(key)
    if not isinstance(value, Mapping):
        raise ConfigError(f"{where} lacks the section '{key}'")
    return value


@dataclass(frozen=True)
class GetodraRotation:
    base: float
    dims: int
    ramp: Optional[FrequencyRamp]   # None: plain frequencies


@dataclass(frozen=True)
class GetodraLayer:
    type: str
    heads: int
    dim: int                                      # query/key width of a head (latent attention: the unrotated part)
    vdim: int
    ff: Optional[int]                             # None: the layer has no feed-forward
    weights_of: Optional[int] = None              # the layer whose tensors this one uses
    rot_dim: int = 0                              # latent attention: the rotated part of a head
    kv_rank: int = 0
    scale: float = 1.0
    rotation: Optional[GetodraRotation] = None
    decay: Tuple[float, ...] = ()                 # lightning: one per head


def _read_layer(layer: Mapping[str, Any], where: str) -> GetodraLayer:
    kind = layer.get("type")
    if kind not in _SIZES:
        raise ConfigError(f"{where}: unknown layer type {kind!r} (known: {', '.join(_SIZES)})")
    mixer = _section(layer, "mixer", where)
    keys = {}
    for key in _SIZES[kind]:
        if mixer.get(key) is None:
            raise ConfigError(f"{where}.mixer lacks the key '{key}'")
        keys[key] = int(mixer[key])
    if kind == LATENT:
        keys["scale"] = require(mixer, "scale", float)
        if keys["rot_dim"]:
            rot = _section(mixer, "rot", f"{where}.mixer")
            scaling, ramp = rot.get("scaling"), None
            if scaling:
                ramp = FrequencyRamp(**{key: require(scaling, key, float) for key in ("factor", "original", "fast", "slow")})
            keys["rotation"] = GetodraRotation(require(rot, "base", float), int(rot.get("dims", keys["rot_dim"])), ramp)
    else:
        decay = mixer.get("decay")
        if not isinstance(decay, (list, tuple)):
            raise ConfigError(f"{where}.mixer lacks the list 'decay'")
        keys["decay"] = tuple(float(d) for d in decay)
    mlp, ff = layer.get("mlp"), None
    if mlp is not None:
        if mlp.get("kind") != "dense":
            raise ConfigError(f"{where}.mlp: unknown kind {mlp.get('kind')!r} (known: dense)")
        ff = require(mlp, "ff")
    weights_of = layer.get("weights_of")
    return GetodraLayer(type=kind, ff=ff, weights_of=None if weights_of is None else int(weights_of), **keys)


@dataclass(frozen=True)
class GetodraConfig:
    vocab: int
    width: int
    max_positions: int
    eps: float
    taps: int
    layers: Tuple[GetodraLayer, ...]
    torch_dtype: str = "bfloat16"

    @classmethod
    def from_dict(cls, cfg: Mapping[str, Any]) -> "GetodraConfig":
        layers = cfg.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("config.json lacks the list 'layers'")
        out = cls(vocab=require(cfg, "vocab"), width=require(cfg, "width"), max_positions=require(cfg, "max_positions"),
                  eps=require(_section(cfg, "norm", "config.json"), "eps", float),
                  taps=require(_section(cfg, "canon", "config.json"), "taps"),
                  layers=tuple(_read_layer(layer, f"layers[{i}]") for i, layer in enumerate(layers)),
                  torch_dtype=str(cfg.get("torch_dtype", cfg.get("dtype", "bfloat16"))))
        out.validate()
        return out

    def validate(self) -> None:
        for name in ("vocab", "width", "max_positions"):
            positive(name, getattr(self, name))
        positive("canon.taps", self.taps)
        if not self.eps > 0:
            raise ConfigError(f"norm.eps must be positive, got {self.eps}")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            for key in _SIZES[layer.type]:
                if key != "rot_dim":
                    positive(f"{where}.mixer.{key}", getattr(layer, key))
            if layer.ff is not None:
                positive(f"{where}.mlp.ff", layer.ff)
            if layer.type == LIGHTNING and len(layer.decay) != layer.heads:
                raise ConfigError(f"{where}.mixer.decay: {len(layer.decay)} decays for {layer.heads} heads")
            if layer.rot_dim < 0:
                raise ConfigError(f"{where}.mixer.rot_dim must not be negative, got {layer.rot_dim}")
            if layer.rotation is not None:
                rot = layer.rotation
                if rot.dims % 2 or not 0 < rot.dims <= layer.rot_dim:
                    raise ConfigError(f"{where}: rot.dims {rot.dims} must be even and at most rot_dim {layer.rot_dim}")
                if not rot.base > 0:
                    raise ConfigError(f"{where}: rot.base must be positive")
                for key in ("factor", "original", "fast", "slow"):
                    if rot.ramp is not None and not getattr(rot.ramp, key) > 0:
                        raise ConfigError(f"{where}: rot.scaling.{key} must be positive")
            if layer.weights_of is not None:
                if not 0 <= layer.weights_of < len(self.layers) or layer.weights_of == i:
                    raise ConfigError(f"{where}.weights_of: no other layer {layer.weights_of}")
                owner = self.layers[self.owner_of(i)]
                if GetodraLayer(**{**layer.__dict__, "weights_of": None}) != owner:
                    raise ConfigError(f"{where}.weights_of: the layer differs from layer {self.owner_of(i)}, whose tensors it uses")

    def owner_of(self, index: int) -> int:
        """The layer whose tensors layer `index` uses: itself, or the one it names (and so on)."""
        seen = set()
        while self.layers[index].weights_of is not None:
            if index in seen:
                raise ConfigError(f"layers[{index}].weights_of: the layers borrow from each other in a circle")
            seen.add(index)
            index = self.layers[index].weights_of
            if not 0 <= index < len(self.layers):
                raise ConfigError(f"weights_of: no layer {index}")
        return index

    def to_json_dict(self) -> dict:
        layers = []
        for layer in self.layers:
            mixer = {key: getattr(layer, key) for key in _SIZES[layer.type]}
            if layer.type == LATENT:
                mixer["scale"] = layer.scale
                if layer.rotation is not None:
                    mixer["rot"] = {"base": layer.rotation.base, "dims": layer.rotation.dims}
                    if layer.rotation.ramp is not None:
                        mixer["rot"]["scaling"] = dict(layer.rotation.ramp.__dict__)
            else:
                mixer["decay"] = list(layer.decay)
            entry = {"type": layer.type, "mixer": mixer, "mlp": None if layer.ff is None else {"kind": "dense", "ff": layer.ff}}
            if layer.weights_of is not None:
                entry["weights_of"] = layer.weights_of
            layers.append(entry)
        return {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "max_positions": self.max_positions,
                "norm": {"eps": self.eps}, "canon": {"taps": self.taps}, "torch_dtype": self.torch_dtype, "layers": layers}

    # ------------------------------------------------------------------ specs
    def _mixer_spec(self, layer: GetodraLayer):
        if layer.type == LIGHTNING:
            return FixedDecaySpec(hidden_size=self.width, num_heads=layer.heads, key_dim=layer.dim, value_dim=layer.vdim,
                                  decays=layer.decay, norm_eps=self.eps)
        rot, position = layer.rotation, None
        if rot is not None:
            position = PositionSpec(kind="neox_rope", rotary_dim=rot.dims, theta=rot.base, ramp=rot.ramp)
        return LatentMixerSpec(hidden_size=self.width, num_heads=layer.heads, nope_dim=layer.dim, rope_dim=layer.rot_dim,
                               value_dim=layer.vdim, kv_rank=layer.kv_rank, scale=layer.scale, position=position,
                               norm_eps=self.eps, gate_name="g")

    def plan(self) -> ModelPlan:
        norm = lambda name: NormSpec(size=self.width, eps=self.eps, weight_name=name, one_weight=True)
        layers, index_of, optional = [], {}, []
        for i, layer in enumerate(self.layers):
            if layer.weights_of is not None:
                continue
            ffn = None
            if layer.ff is not None:
                ffn = FeedForwardSpec(hidden_size=self.width, intermediate_size=layer.ff, activation=FEED_FORWARD_ACTIVATION,
                                      gate_name="gate", up_name="up", down_name="down", weight_suffix="")
            else:  # a checkpoint may still hold what stands around the feed-forward the layer does not have
                optional += [f"l{i}.norm2", f"l{i}.canon2"]
            index_of[i] = len(layers)
            layers.append(LayerSpec(prefix=f"l{i}.", mixer=self._mixer_spec(layer), feed_forward=ffn, mixer_norm=norm("norm1"),
                                    feed_forward_norm=norm("norm2") if ffn is not None else None, mixer_prefix="mix.",
                                    feed_forward_prefix="mlp.", mixer_norm_prefix="", feed_forward_norm_prefix="",
                                    arrangement="branchnorm", input_conv=InputConvSpec(self.taps, ("canon1", "canon2"))))
        # a layer that borrows tensors is a second stop at the same layer, with a cache and state of its own
        schedule = tuple(ScheduleEntry(layer=index_of[self.owner_of(i)]) for i in range(len(self.layers)))
        return ModelPlan(
            architecture=ARCHITECTURE, hidden_size=self.width, vocab_size=self.vocab, layers=tuple(layers), schedule=schedule,
            final_norm=norm("final.norm"), embedding_name="embed", head_name="head", final_norm_prefix="",
            max_positions=self.max_positions, optional_names=tuple(optional), position_table_name="pos")


register_architecture(ARCHITECTURE, GetodraConfig.from_dict)
