"""Mulenex: a decoder whose layers are listed one by one in config.json, each with a norm before and after every
sublayer, softmax attention or a matrix memory, and a dense or routed feed-forward.

config.json keys (every size and every constant that may differ between models is read from here):

    architecture      "Mulenex"
    vocab, width      vocabulary and residual width
    norm.eps          eps of every RMS norm of the model (inside the root)
    layers[i]         type: "attention" | "mlstm"; mixer: the mixer's sizes;
                      mlp: {kind: "dense", ff} | {kind: "moe", expert {ff}, router {experts, top}, shared {ff}} | null
      attention       heads, kv_heads, dim (query/key width), vdim (value width), scale, softcap (or null),
                      q_temp {coef, every} (or null), v_mix (or false)
      mlstm           heads, dim, vdim, gate_cap

Fixed by the design, so constants of this file: x <- x + norm1b(mixer(norm1(x))), then x <- x + norm2b(mlp(norm2(x))),
with norm weights stored around zero (the weight is 1 + w); the embedding's row plus sines and cosines of the position
(base 10000), neither scaled.  Attention: an RMS norm of every query and key head with a plain weight that the heads
share, no rotation, queries times 1 + coef ln(floor((p + 1) / every) + 1), scores capped by softcap tanh(s / softcap),
every earlier key visible, the values of all layers with v_mix but the first of them mixed with that first one's, each
head's output gated by the sigmoid of one number, no biases.  Matrix memory: exponential gates capped by
gate_cap tanh(z / gate_cap), q times dim^-1/2, 1e-6 added to the read-out's denominator, a norm per head without eps of
its own, a weight per head and feature, a sigmoid output gate.  Dense feed-forwards: W_down relu(W_up h + b)^2 + b.
Routed ones: experts W_down (silu(W_gate h) * W_up h) weighted by the softmax over the chosen logits, the router with a
bias, and a shared expert of the same form times the sigmoid of one number per token.
Tensor names: `embed`, `final.norm`, `head`, and below `l<i>.`: `norm1`, `norm1b`, `norm2`, `norm2b`,
`mix.q|k|v|g|o`, `mix.q.norm`, `mix.k.norm`, `mix.vmix` (attention), `mix.q|k|v|g|o|norm`, `mix.i|f` with `.b` (mlstm),
`mlp.up|down` with `.b` (dense), `mlp.router`, `mlp.router.b`, `mlp.e<j>.gate|up|down`, `mlp.shared.gate|up|down|sg` (moe).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple

from ..config.model_config import (ConfigError, ExpertsSpec, FeedForwardSpec, LayerSpec, MatrixMemorySpec, MixerSpec,
                                   ModelPlan, NormSpec, QueryTemperature, ScheduleEntry, SharedExpertSpec, positive, require)
from ..config.registry import register_architecture

ARCHITECTURE = "Mulenex"
ATTENTION, MEMORY = "attention", "mlstm"
POSITION_BASE = 10000.0
READOUT_FLOOR = 1e-6
_SIZES = {ATTENTION: ("heads", "kv_heads", "dim", "vdim"), MEMORY: ("heads", "dim", "vdim")}


def _section(cfg: Mapping[str, Any], key: str, where: str) -> Mapping[str, Any]:
    value = cfg.get(key)
    if not isinstance(value, Mapping):
        raise ConfigError(f"{where} lacks the section '{key}'")
    return value


def _needed(cfg: Mapping[str, Any], key: str, where: str, kind=int):
    if cfg.get(key) is None:
        raise ConfigError(f"{where} lacks the key '{key}'")
    try:
        return kind(cfg[key])
    except (TypeError, ValueError) as err:
        raise ConfigError(f"{where}.{key} = {cfg[key]!r} is not {kind.__name__}") from err


@dataclass(frozen=True)
class MulenexLayer:
    type: str
    heads: int
    dim: int
    vdim: int
    # attention
    kv_heads: int = 0
    scale: float = 1.0
    softcap: Optional[float] = None
    q_temp: Optional[QueryTemperature] = None
    v_mix: bool = False
    # mlstm
    gate_cap: float = 0.0
    # feed-forward: dense with `ff`, routed with `experts`, or neither
    ff: Optional[int] = None
    experts: Optional[int] = None
    top: int = 0
    expert_ff: int = 0
    shared_ff: Optional[int] = None


def _read_layer(layer: Mapping[str, Any], where: str) -> MulenexLayer:
    kind = layer.get("type")
    if kind not in _SIZES:
        raise ConfigError(f"{where}: unknown layer type {kind!r} (known: {', '.join(_SIZES)})")
    mixer, at = _section(layer, "mixer", where), f"{where}.mixer"
    keys = {key: _needed(mixer, key, at) for key in _SIZES[kind]}
    if kind == ATTENTION:
        keys["scale"] = _needed(mixer, "scale", at, float)
        keys["softcap"] = float(mixer["softcap"]) if mixer.get("softcap") else None
        keys["v_mix"] = bool(mixer.get("v_mix", False))
        if mixer.get("q_temp"):
            temp = _section(mixer, "q_temp", at)
            keys["q_temp"] = QueryTemperature(_needed(temp, "coef", at + ".q_temp", float), _needed(temp, "every", at + ".q_temp"))
    else:
        keys["gate_cap"] = _needed(mixer, "gate_cap", at, float)
    mlp, at = layer.get("mlp"), f"{where}.mlp"
    if mlp is not None:
        if mlp.get("kind") == "dense":
            keys["ff"] = _needed(mlp, "ff", at)
        elif mlp.get("kind") == "moe":
            router = _section(mlp, "router", at)
            keys["experts"], keys["top"] = _needed(router, "experts", at + ".router"), _needed(router, "top", at + ".router")
            keys["expert_ff"] = _needed(_section(mlp, "expert", at), "ff", at + ".expert")
            if mlp.get("shared"):
                keys["shared_ff"] = _needed(_section(mlp, "shared", at), "ff", at + ".shared")
        else:
            raise ConfigError(f"{at}: unknown kind {mlp.get('kind')!r} (known: dense, moe)")
    return MulenexLayer(type=kind, **keys)


@dataclass(frozen=True)
class MulenexConfig:
    vocab: int
    width: int
    eps: float
    layers: Tuple[MulenexLayer, ...]
    torch_dtype: str = "bfloat16"

    @classmethod
    def from_dict(cls, cfg: Mapping[str, Any]) -> "MulenexConfig":
        layers = cfg.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("config.json lacks the list 'layers'")
        out = cls(vocab=require(cfg, "vocab"), width=require(cfg, "width"),
                  eps=require(_section(cfg, "norm", "config.json"), "eps", float),
                  layers=tuple(_read_layer(layer, f"layers[{i}]") for i, layer in enumerate(layers)),
                  torch_dtype=str(cfg.get("torch_dtype", cfg.get("dtype", "bfloat16"))))
        out.validate()
        return out

    def validate(self) -> None:
        positive("vocab", self.vocab)
        positive("width", self.width)
        if not self.eps > 0:
            raise ConfigError(f"norm.eps must be positive, got {self.eps}")
        source = self.value_source
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            for key in _SIZES[layer.type]:
                positive(f"{where}.mixer.{key}", getattr(layer, key))
            if layer.type == ATTENTION:
                if layer.heads % layer.kv_heads:
                    raise ConfigError(f"{where}: {layer.heads} heads are not a multiple of {layer.kv_heads} kv_heads")
                if layer.softcap is not None and not layer.softcap > 0:
                    raise ConfigError(f"{where}.mixer.softcap must be positive, got {layer.softcap}")
                if layer.q_temp is not None:
                    positive(f"{where}.mixer.q_temp.every", layer.q_temp.every)
                if layer.v_mix:
                    first = self.layers[source]
                    if (layer.kv_heads, layer.vdim) != (first.kv_heads, first.vdim):
                        raise ConfigError(f"{where}: {layer.kv_heads} value heads of {layer.vdim} cannot be mixed with layer "
                                          f"{source}'s {first.kv_heads} of {first.vdim}")
            elif not layer.gate_cap > 0:
                raise ConfigError(f"{where}.mixer.gate_cap must be positive, got {layer.gate_cap}")
            if layer.ff is not None:
                positive(f"{where}.mlp.ff", layer.ff)
            if layer.experts is not None:
                positive(f"{where}.mlp.router.experts", layer.experts)
                positive(f"{where}.mlp.expert.ff", layer.expert_ff)
                if not 0 < layer.top <= layer.experts:
                    raise ConfigError(f"{where}.mlp.router: top {layer.top} of {layer.experts} experts")
                if layer.shared_ff is not None:
                    positive(f"{where}.mlp.shared.ff", layer.shared_ff)

    @property
    def value_source(self) -> Optional[int]:
        """The first layer with v_mix, whose values the later ones mix in."""
        return next((i for i, layer in enumerate(self.layers) if layer.v_mix), None)

    def to_json_dict(self) -> dict:
        layers = []
        for layer in self.layers:
            mixer = {key: getattr(layer, key) for key in _SIZES[layer.type]}
            if layer.type == ATTENTION:
                mixer.update(scale=layer.scale, softcap=layer.softcap, v_mix=layer.v_mix,
                             q_temp=None if layer.q_temp is None else dict(layer.q_temp.__dict__))
            else:
                mixer["gate_cap"] = layer.gate_cap
            mlp = None
            if layer.ff is not None:
                mlp = {"kind": "dense", "ff": layer.ff}
            elif layer.experts is not None:
                mlp = {"kind": "moe", "expert": {"ff": layer.expert_ff}, "router": {"experts": layer.experts, "top": layer.top}}
                if layer.shared_ff is not None:
                    mlp["shared"] = {"ff": layer.shared_ff}
            layers.append({"type": layer.type, "mixer": mixer, "mlp": mlp})
        return {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
                "torch_dtype": self.torch_dtype, "layers": layers}

    # ------------------------------------------------------------------ specs
    def _mixer_spec(self, index: int):
        layer = self.layers[index]
        if layer.type == MEMORY:
            return MatrixMemorySpec(hidden_size=self.width, num_heads=layer.heads, key_dim=layer.dim, value_dim=layer.vdim,
                                    gate_cap=layer.gate_cap, norm_eps=self.eps, readout_floor=READOUT_FLOOR)
        mix = None
        if layer.v_mix:
            mix = "source" if index == self.value_source else "mixed"
        return MixerSpec(hidden_size=self.width, num_heads=layer.heads, num_kv_heads=layer.kv_heads, head_dim=layer.dim,
                         value_dim=layer.vdim, scale=layer.scale, softcap=layer.softcap, qkv_bias=False, out_bias=False,
                         qk_norm="per_head", qk_norm_eps=self.eps, q_norm_name="q.norm", k_norm_name="k.norm",
                         temperature=layer.q_temp, value_mix=mix, value_mix_name="vmix", head_gate_name="g", q_name="q",
                         k_name="k", v_name="v", o_name="o", weight_suffix="")

    def _feed_forward_spec(self, layer: MulenexLayer):
        if layer.ff is not None:
            return FeedForwardSpec(kind="dense", hidden_size=self.width, intermediate_size=layer.ff, activation="relu2",
                                   up_name="up", down_name="down", weight_suffix="", bias=True, bias_suffix=".b")
        if layer.experts is not None:
            return ExpertsSpec(hidden_size=self.width, intermediate_size=layer.expert_ff, num_experts=layer.experts,
                               top=layer.top, activation="silu", router_bias_name="router.b", weights_over="chosen",
                               shared=None if layer.shared_ff is None else SharedExpertSpec(layer.shared_ff))
        return None

    def plan(self) -> ModelPlan:
        norm = lambda name: NormSpec(size=self.width, eps=self.eps, weight_name=name, weight_offset=1.0)
        layers, optional = [], []
        for i, layer in enumerate(self.layers):
            ffn, mixer = self._feed_forward_spec(layer), self._mixer_spec(i)
            if ffn is None:  # a checkpoint may still hold the norms around the feed-forward the layer does not have
                optional += [f"l{i}.norm2", f"l{i}.norm2b"]
            if layer.type == ATTENTION and mixer.value_mix != "mixed":  # a share that is not used
                optional.append(f"l{i}.mix.vmix")
            layers.append(LayerSpec(prefix=f"l{i}.", mixer=mixer, feed_forward=ffn, mixer_norm=norm("norm1"),
                                    feed_forward_norm=norm("norm2") if ffn is not None else None,
                                    mixer_out_norm=norm("norm1b"),
                                    feed_forward_out_norm=norm("norm2b") if ffn is not None else None, mixer_prefix="mix.",
                                    feed_forward_prefix="mlp.", mixer_norm_prefix="", feed_forward_norm_prefix="",
                                    arrangement="sandwich"))
        return ModelPlan(
            architecture=ARCHITECTURE, hidden_size=self.width, vocab_size=self.vocab, layers=tuple(layers),
            schedule=tuple(ScheduleEntry(layer=i) for i in range(len(layers))), final_norm=norm("final.norm"),
            embedding_name="embed", head_name="head", final_norm_prefix="", optional_names=tuple(optional),
            sinusoid_base=POSITION_BASE)


register_architecture(ARCHITECTURE, MulenexConfig.from_dict)
