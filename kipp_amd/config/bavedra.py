"""Typed configuration of the Bavedra decoder, read from its config.json.

A Bavedra model scales the embedding's rows and is a list of pre-norm layers, x += mixer(norm1(x)), x += ff(norm2(x)), each
with one of three mixers and a dense or routed feed-forward (or none):

    rglru       a recurrent block with a real-gated linear recurrent unit behind a short causal convolution
    parallel    two mixers side by side on the same input, each result normed over the model's width, half their sum:
                grouped-query attention whose values are its keys before the rotation (neighbours paired), with a sliding
                window and one added to the softmax's denominator (`left`), and a selective state space layer in its dual form
                behind a short causal convolution, with a state of fixed size (`right`)
    delta       the gated delta rule behind short causal convolutions

    dense       W_down relu(W_up h)^2
    moe         softmax router with a correction of the choice, groups of experts of which the best stay (a group's score is
                its largest), identity experts among the choices, gated experts W_down (silu(W_gate h) * (W_up h)), a shared
                expert with a gate of its own

config.json names the architecture under `architecture` and gives every size and every constant that differs between
models; tensors are `embed`, `head`, `final.norm` and, for layer i, `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.*`, `l<i>.mlp.*`.
A layer with `weights_of: j` is layer j run once more, with a cache or state of its own.  Keys that are not implemented are
refused, never ignored.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Optional, Tuple

from .rerizen import _float, _get, _int, _only
from .specs import (AttentionSpec, ConfigError, DenseMLPSpec, EmbeddingSpec, GatedDeltaSpec, GatedRecurrenceSpec, HeadSpec, LayerRun,
                    LayerSpec, ModelSpec, ParallelMixerSpec, RMSNormSpec, RopeSpec, RoutedMLPSpec, SSDSpec)

ARCHITECTURE = "Bavedra"
MAX_POSITION = 1 << 20      # the engine's own bound on a context (block tables are made for it); the design has none
RECURRENCE_FACTOR = 8.0     # of the linear recurrent unit's logarithm of a
UNIT_EPS = 1e-6             # inside the root of the delta rule's unit norms
SIDE_SCALE = 0.5            # of each of the two results of a parallel mixer
MIXERS = ("rglru", "parallel", "delta")


def _window(m: dict, where: str) -> Optional[int]:
    """The length of the window; None (every earlier position is seen) where the mixer names none."""
    mask = m.get("mask")
    if mask is None:
        return None
    _only(mask, ("size",), where + "mask.")
    return _int(mask, "size", where + "mask.") if mask.get("size") is not None else None


@dataclass(frozen=True)
class BavedraConfig:
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    layers: Tuple[dict, ...]                    # as config.json gives them (checked)
    max_position: int = MAX_POSITION

    @classmethod
    def from_dict(cls, d: dict) -> "BavedraConfig":
        _only(d, ("architecture", "architectures", "vocab", "width", "embedding", "norm", "layers", "max_position", "torch_dtype"), "")
        layers = _get(d, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json layers: expected a list with at least one layer")
        embedding, norm = _get(d, "embedding", ""), _get(d, "norm", "")
        _only(embedding, ("scale",), "embedding.")
        _only(norm, ("eps",), "norm.")
        eps = _float(norm, "eps", "norm.")
        if not eps >= 0:
            raise ConfigError(f"config.json norm.eps: must be >= 0, got {eps}")
        cfg = cls(vocab=_int(d, "vocab", ""), width=_int(d, "width", ""), embedding_scale=_float(embedding, "scale", "embedding."),
                  norm_eps=eps, layers=tuple(copy.deepcopy(layers)),
                  max_position=_int(d, "max_position", "") if "max_position" in d else MAX_POSITION)
        cfg.model_spec()        # checks every layer
        return cfg

    def to_dict(self) -> dict:
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "embedding": {"scale": self.embedding_scale},
             "norm": {"eps": self.norm_eps}, "layers": copy.deepcopy(list(self.layers))}
        if self.max_position != MAX_POSITION:
            d["max_position"] = self.max_position
        return d

    # -- mixers --------------------------------------------------------------------------------
    def _rglru(self, prefix: str, m: dict, where: str):
        _only(m, ("width", "blocks", "conv"), where)
        return GatedRecurrenceSpec(hidden_size=self.width, width=_int(m, "width", where), blocks=_int(m, "blocks", where),
                                   conv_taps=_int(m, "conv", where), factor=RECURRENCE_FACTOR, prefix=prefix)

    def _attention(self, prefix: str, m: dict, where: str):
        _only(m, ("heads", "kv_heads", "dim", "vdim", "scale", "mask", "rot"), where)
        d, dv = _int(m, "dim", where), _int(m, "vdim", where)
        if dv != d:
            raise ConfigError(f"config.json {where}vdim: {dv} differs from dim {d}, but the values are the keys")
        rot, at = _get(m, "rot", where), where + "rot."
        _only(rot, ("base", "dims"), at)
        position = RopeSpec(head_dim=d, theta=_float(rot, "base", at), rotary_dim=_int(rot, "dims", at, 2), pairing="interleaved")
        return AttentionSpec(
            hidden_size=self.width, num_heads=_int(m, "heads", where), num_kv_heads=_int(m, "kv_heads", where), head_dim=d,
            position=position, window=_window(m, where), scale=_float(m, "scale", where), prefix=prefix,
            names=("q", "k", "", "o", "", ""), sink=True, keys_as_values=True)

    def _ssd(self, prefix: str, m: dict, where: str):
        _only(m, ("heads", "vdim", "state", "groups", "conv", "norm_groups"), where)
        return SSDSpec(hidden_size=self.width, num_heads=_int(m, "heads", where), head_dim=_int(m, "vdim", where),
                       state_size=_int(m, "state", where), groups=_int(m, "groups", where), conv_taps=_int(m, "conv", where),
                       norm_groups=_int(m, "norm_groups", where), norm_eps=self.norm_eps, prefix=prefix)

    def _parallel(self, prefix: str, m: dict, where: str):
        _only(m, ("left", "right"), where)
        return ParallelMixerSpec(left=self._attention(prefix + "left.", _get(m, "left", where), where + "left."),
                                 right=self._ssd(prefix + "right.", _get(m, "right", where), where + "right."),
                                 left_scale=SIDE_SCALE, right_scale=SIDE_SCALE,
                                 left_norm=self._norm(prefix + "left.out"), right_norm=self._norm(prefix + "right.out"))

    def _delta(self, prefix: str, m: dict, where: str):
        _only(m, ("heads", "kv_heads", "dim", "vdim", "conv"), where)
        return GatedDeltaSpec(hidden_size=self.width, num_heads=_int(m, "heads", where), num_kv_heads=_int(m, "kv_heads", where),
                              head_dim=_int(m, "dim", where), v_head_dim=_int(m, "vdim", where), conv_taps=_int(m, "conv", where),
                              norm_eps=self.norm_eps, unit_eps=UNIT_EPS, prefix=prefix)

    # -- feed-forwards ---------------------------------------------------------------------------
    def _feed_forward(self, i: int, layer: dict):
        mlp = layer.get("mlp")
        if mlp is None:
            return None
        where, prefix = f"layers[{i}].mlp.", f"l{i}.mlp."
        kind = _get(mlp, "kind", where)
        if kind == "dense":
            _only(mlp, ("kind", "ff"), where)
            return DenseMLPSpec(self.width, _int(mlp, "ff", where), "relu2", prefix)
        if kind != "moe":
            raise ConfigError(f"config.json {where}kind: {kind!r} is not a feed-forward of this design (dense, moe)")
        _only(mlp, ("kind", "expert", "router", "shared"), where)
        router, expert = _get(mlp, "router", where), _get(mlp, "expert", where)
        _only(router, ("experts", "top", "groups", "identity"), where + "router.")
        _only(expert, ("ff",), where + "expert.")
        groups = None
        if router.get("groups") is not None:
            _only(router["groups"], ("count", "keep"), where + "router.groups.")
            groups = tuple(_int(router["groups"], key, where + "router.groups.") for key in ("count", "keep"))
        shared = None
        if mlp.get("shared") is not None:
            _only(mlp["shared"], ("ff",), where + "shared.")
            shared = _int(mlp["shared"], "ff", where + "shared.")
        return RoutedMLPSpec(
            hidden_size=self.width, experts=_int(router, "experts", where + "router."), top=_int(router, "top", where + "router."),
            expert_size=_int(expert, "ff", where + "expert."), shared_size=shared, activation="silu", prefix=prefix, router="softmax",
            correction_name="correction", groups=groups, group_score="top1", gate_name="gate",
            identity=_int(router, "identity", where + "router.", 0) if router.get("identity") is not None else 0,
            shared_gate_name="shared.sg" if shared is not None else None)

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
        make = {"rglru": self._rglru, "parallel": self._parallel, "delta": self._delta}[kind]
        parts = [("mixer_norm", self._norm(f"l{i}.norm1")), ("mixer", make(f"l{i}.mix.", m, where + "mixer."))]
        ffn = self._feed_forward(i, layer)
        if ffn is not None:
            parts += [("ffn_norm", self._norm(f"l{i}.norm2")), ("ffn", ffn)]
        return LayerSpec(parts=tuple(parts), block="pre_norm" if ffn is not None else "pre_norm_mixer")

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
            embedding=EmbeddingSpec(self.vocab, self.width, prefix="embed", name="", scale=self.embedding_scale),
            layers=tuple(layers), order=tuple(order), final_norm=self._norm("final.norm"),
            head=HeadSpec(self.vocab, self.width, tied=False, prefix="head", name=""))
