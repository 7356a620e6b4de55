"""Typed configuration of the Bipazen decoder, read from its config.json.

A Bipazen model is a list of pre-norm layers whose two results are scaled column by column before they are added,
x += ls1 * mixer(norm1(x)), x += ls2 * ff(norm2(x)), each with one of three mixers and a routed feed-forward (or none):

    mamba2              a selective state space layer in its dual form behind a short causal convolution
    rglru               a recurrent block with a real-gated linear recurrent unit behind a short causal convolution
    latent_attention    keys and values made from a cached latent, a rotated key part shared by the heads (halves paired),
                        queries straight from the input, a gate on every number of the heads' results

    moe                 sigmoid router without a correction or groups; a chosen expert, W_down (silu(W_gate h) * (W_up h)), is
                        given its input times its score

config.json names the architecture under `architecture` and gives every size and every constant that differs between
models; tensors are `embed` (the output head too), `final.norm` and, for layer i, `l<i>.norm1`, `l<i>.norm2`, `l<i>.ls1`,
`l<i>.ls2`, `l<i>.mix.*`, `l<i>.mlp.*`.  A layer with `weights_of: j` is layer j run once more, with a cache or state of its
own.  Keys that are not implemented are refused, never ignored.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Tuple

from .rerizen import _float, _get, _int, _only
from .specs import (ConfigError, EmbeddingSpec, GatedRecurrenceSpec, HeadSpec, LatentAttentionSpec, LayerRun, LayerScaleSpec, LayerSpec,
                    ModelSpec, NoPositionSpec, RMSNormSpec, RopeSpec, RoutedMLPSpec, SSDSpec)

ARCHITECTURE = "Bipazen"
MAX_POSITION = 1 << 20      # the engine's own bound on a context (block tables are made for it); the design has none
RECURRENCE_FACTOR = 8.0     # of the linear recurrent unit's logarithm of a
MIXERS = ("mamba2", "rglru", "latent_attention")


@dataclass(frozen=True)
class BipazenConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[dict, ...]                    # as config.json gives them (checked)
    max_position: int = MAX_POSITION

    @classmethod
    def from_dict(cls, d: dict) -> "BipazenConfig":
        _only(d, ("architecture", "architectures", "vocab", "width", "norm", "layers", "max_position", "torch_dtype"), "")
        layers = _get(d, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json layers: expected a list with at least one layer")
        norm = _get(d, "norm", "")
        _only(norm, ("eps",), "norm.")
        eps = _float(norm, "eps", "norm.")
        if not eps >= 0:
            raise ConfigError(f"config.json norm.eps: must be >= 0, got {eps}")
        cfg = cls(vocab=_int(d, "vocab", ""), width=_int(d, "width", ""), norm_eps=eps, layers=tuple(copy.deepcopy(layers)),
                  max_position=_int(d, "max_position", "") if "max_position" in d else MAX_POSITION)
        cfg.model_spec()        # checks every layer
        return cfg

    def to_dict(self) -> dict:
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
             "layers": copy.deepcopy(list(self.layers))}
        if self.max_position != MAX_POSITION:
            d["max_position"] = self.max_position
        return d

    # -- parts ---------------------------------------------------------------------------------
    def _mamba2(self, prefix: str, m: dict, where: str):
        _only(m, ("heads", "vdim", "state", "groups", "conv", "norm_groups"), where)
        return SSDSpec(hidden_size=self.width, num_heads=_int(m, "heads", where), head_dim=_int(m, "vdim", where),
                       state_size=_int(m, "state", where), groups=_int(m, "groups", where), conv_taps=_int(m, "conv", where),
                       norm_groups=_int(m, "norm_groups", where), norm_eps=self.norm_eps, prefix=prefix)

    def _rglru(self, prefix: str, m: dict, where: str):
        _only(m, ("width", "blocks", "conv"), where)
        return GatedRecurrenceSpec(hidden_size=self.width, width=_int(m, "width", where), blocks=_int(m, "blocks", where),
                                   conv_taps=_int(m, "conv", where), factor=RECURRENCE_FACTOR, prefix=prefix)

    def _latent(self, prefix: str, m: dict, where: str):
        _only(m, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot"), where)
        rot_dim = _int(m, "rot_dim", where, 0)
        position = NoPositionSpec()
        if rot_dim > 0:
            rot, at = _get(m, "rot", where), where + "rot."
            _only(rot, ("base", "dims"), at)
            dims = _int(rot, "dims", at)
            if dims > rot_dim:
                raise ConfigError(f"config.json {at}dims: {dims} exceeds rot_dim {rot_dim}")
            position = RopeSpec(head_dim=rot_dim, theta=_float(rot, "base", at), rotary_dim=dims)
        return LatentAttentionSpec(
            hidden_size=self.width, num_heads=_int(m, "heads", where), head_dim=_int(m, "dim", where), rot_dim=rot_dim,
            v_head_dim=_int(m, "vdim", where), q_rank=None, kv_rank=_int(m, "kv_rank", where), scale=_float(m, "scale", where),
            norm_eps=self.norm_eps, position=position, gate_each=True, prefix=prefix,
            names=("", "", "q", "dkv", "dkv.norm", "uk", "uv", "g", "o"))

    def _feed_forward(self, i: int, layer: dict):
        mlp = layer.get("mlp")
        if mlp is None:
            return None
        where = f"layers[{i}].mlp."
        kind = _get(mlp, "kind", where)
        if kind != "moe":
            raise ConfigError(f"config.json {where}kind: {kind!r} is not a feed-forward of this design (moe)")
        _only(mlp, ("kind", "expert", "router"), where)
        router, expert = _get(mlp, "router", where), _get(mlp, "expert", where)
        _only(router, ("experts", "top"), where + "router.")
        _only(expert, ("ff",), where + "expert.")
        return RoutedMLPSpec(hidden_size=self.width, experts=_int(router, "experts", where + "router."),
                             top=_int(router, "top", where + "router."), expert_size=_int(expert, "ff", where + "expert."),
                             activation="silu", prefix=f"l{i}.mlp.", router="sigmoid", renormalize=False, gate_name="gate", weigh_input=True)

    def _norm(self, name: str) -> RMSNormSpec:
        return RMSNormSpec(self.width, self.norm_eps, name, name="")

    def _layer(self, i: int, layer: dict) -> LayerSpec:
        where = f"layers[{i}]."
        kind = _get(layer, "type", where)
        m = _get(layer, "mixer", where)
        if not isinstance(m, dict):
            raise ConfigError(f"config.json {where}mixer: expected an object")
        if kind not in MIXERS:
            raise ConfigError(f"config.json {where}type: {kind!r} is not a mixer of this design ({', '.join(MIXERS)})")
        make = {"mamba2": self._mamba2, "rglru": self._rglru, "latent_attention": self._latent}[kind]
        parts = [("mixer_norm", self._norm(f"l{i}.norm1")), ("mixer", make(f"l{i}.mix.", m, where + "mixer.")),
                 ("mixer_scale", LayerScaleSpec(self.width, f"l{i}.ls1", name=""))]
        ffn = self._feed_forward(i, layer)
        if ffn is not None:
            parts += [("ffn_norm", self._norm(f"l{i}.norm2")), ("ffn", ffn), ("ffn_scale", LayerScaleSpec(self.width, f"l{i}.ls2", name=""))]
        return LayerSpec(parts=tuple(parts), block="scaled_pre_norm" if ffn is not None else "scaled_pre_norm_mixer")

    def model_spec(self) -> ModelSpec:
        layers, order = [], []
        runs_of = []            # entry of config.json's list -> index into `layers`
        for i, layer in enumerate(self.layers):
            if not isinstance(layer, dict):
                raise ConfigError(f"config.json layers[{i}]: expected an object")
            where = f"layers[{i}]."
            _only(layer, ("type", "mixer", "mlp", "weights_of"), where)
            if layer.get("weights_of") is None:
                runs_of.append(len(layers))
                layers.append(self._layer(i, layer))
            else:
                # the other layer once more: its tensors, a cache or state of this run's own
                source = _int(layer, "weights_of", where, 0)
                if source >= i:
                    raise ConfigError(f"config.json {where}weights_of: layer {source} is not an earlier layer")
                theirs = self.layers[source]
                for key in ("type", "mixer", "mlp"):
                    if key in layer and layer[key] != theirs.get(key):
                        raise ConfigError(f"config.json {where}{key}: differs from layer {source}'s, whose tensors it uses")
                runs_of.append(runs_of[source])
            order.append(LayerRun(runs_of[i]))
        return ModelSpec(
            architecture=ARCHITECTURE, hidden_size=self.width, vocab_size=self.vocab, max_position=self.max_position,
            embedding=EmbeddingSpec(self.vocab, self.width, prefix="embed", name=""),
            layers=tuple(layers), order=tuple(order), final_norm=self._norm("final.norm"),
            head=HeadSpec(self.vocab, self.width, tied=True))
