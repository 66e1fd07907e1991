"""The Netovik decoder: its config.json and the parts it is made of.

config.json names everything that can differ between models of the design:

    architecture "Netovik", vocab, width, norm {eps, groups}, embedding {scale}, and `layers`, one entry a layer: `type`
    ("wkv" | "attention"), `mixer` (its sizes) and `mlp` (or null).

    wkv mixer: heads, dim.
    attention mixer: heads, kv_heads (heads if left out), dim, vdim (the values are the keys, so it is dim), scale,
    softcap (none if left out), bias_max, mask {size, keep_first} (everything is seen if left out).
    mlp: {"kind": "dense", "ff"} or {"kind": "moe", "router" {experts, top}, "expert" {ff}}.

Tensors: `embed`, `final.norm`; layer i under `l<i>.`: `norm1`, `norm2`, `dwa`, `mix.*`, `mlp.gate|up|down` or
`mlp.router`, `mlp.e<e>.gate|up|down`. Linear weights are [out, in]. The head is the embedding table. Two sizes are not
in config.json: the rank of the projection that a wkv mixer's decay goes through (the rows of `l<i>.mix.w1`) and the
rows of an attention layer's table of distance biases (`l<i>.mix.rel`). With a model folder at hand they come from the
tensors (`with_tensor_shapes`); a configuration without a folder (random weights) names them as `rank` and
`bias_rows` in the mixer. Nothing here fixes a size.

What the design fixes, and where it stands: norms in groups behind the sub-layers only and a weighted average over the
depth (`depth_averaged_branch_norm`); attention without rotation, with normed heads, values that are the keys, a
bias by the distance, scores mixed between the heads and a sink of score zero; experts weighted by the softmax over
all of them, not renormalised.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .model_config import ConfigError, LayerCall, LayerSpec, ModelSpec, PartSpec
from .musutar_config import DEFAULT_MAX_POSITIONS, _need


@dataclass(frozen=True)
class NetovikConfig:
    data: Mapping[str, Any]
    max_positions: int = DEFAULT_MAX_POSITIONS

    architecture = "Netovik"

    @property
    def vocab_size(self) -> int:
        return int(self.data["vocab"])

    @property
    def hidden_size(self) -> int:
        return int(self.data["width"])

    @property
    def num_layers(self) -> int:
        return len(self.data["layers"])

    @classmethod
    def from_dict(cls, data: Mapping[str, Any]) -> "NetovikConfig":
        vocab, width = _need(data, "vocab", int, "the model"), _need(data, "width", int, "the model")
        if vocab < 1 or width < 1:
            raise ConfigError("vocab and width must be >= 1")
        norm = data.get("norm") or {}
        _need(norm, "eps", float, "norm")
        if norm.get("groups") is not None:
            groups = _need(norm, "groups", int, "norm")
            if groups < 1 or width % groups:
                raise ConfigError("norm.groups must divide the width")
        if (data.get("embedding") or {}).get("scale") is not None:
            _need(data["embedding"], "scale", float, "embedding")
        layers = data.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("config.json lacks 'layers'")
        for i, layer in enumerate(layers):
            where = f"layer {i}"
            kind = _need(layer, "type", str, where)
            mixer = layer.get("mixer")
            if not isinstance(mixer, Mapping):
                raise ConfigError(f"config.json: {where} lacks 'mixer'")
            heads, dim = _need(mixer, "heads", int, where), _need(mixer, "dim", int, where)
            if heads < 1 or dim < 1:
                raise ConfigError(f"{where}: heads and dim must be >= 1")
            if kind == "attention":
                if mixer.get("kv_heads") is not None:
                    kv_heads = _need(mixer, "kv_heads", int, where)
                    if kv_heads < 1 or heads % kv_heads:
                        raise ConfigError(f"{where}: heads must be a positive multiple of kv_heads")
                if mixer.get("vdim") is not None and _need(mixer, "vdim", int, where) != dim:
                    raise ConfigError(f"{where}: the values are the keys, so vdim must be dim")
                if not _need(mixer, "scale", float, where) > 0:
                    raise ConfigError(f"{where}: scale must be positive")
                if mixer.get("softcap") is not None and not _need(mixer, "softcap", float, where) > 0:
                    raise ConfigError(f"{where}: softcap must be positive")
                if not _need(mixer, "bias_max", float, where) > 0:
                    raise ConfigError(f"{where}: bias_max must be positive")
                mask = mixer.get("mask")
                if mask:
                    if _need(mask, "size", int, where + " mask") < 1:
                        raise ConfigError(f"{where}: mask.size must be >= 1")
                    if mask.get("keep_first") is not None and _need(mask, "keep_first", int, where + " mask") < 0:
                        raise ConfigError(f"{where}: mask.keep_first must be >= 0")
            elif kind != "wkv":
                raise ConfigError(f"{where}: unknown layer type {kind!r}")
            mlp = layer.get("mlp")
            if mlp is None:
                continue
            mlp_kind = _need(mlp, "kind", str, where + " mlp")
            if mlp_kind == "dense":
                if _need(mlp, "ff", int, where + " mlp") < 1:
                    raise ConfigError(f"{where}: mlp.ff must be >= 1")
            elif mlp_kind == "moe":
                router = mlp.get("router")
                experts, top = _need(router, "experts", int, where + " router"), _need(router, "top", int, where + " router")
                if not 1 <= top <= experts:
                    raise ConfigError(f"{where}: router.top must be between 1 and router.experts")
                if _need(mlp.get("expert"), "ff", int, where + " expert") < 1:
                    raise ConfigError(f"{where}: expert.ff must be >= 1")
            else:
                raise ConfigError(f"{where}: unknown mlp kind {mlp_kind!r}")
        return cls(data=dict(data), max_positions=int(data.get("max_positions") or DEFAULT_MAX_POSITIONS))

    def to_dict(self) -> dict:
        return dict(self.data)

    def with_tensor_shapes(self, shapes: Mapping[str, tuple]) -> "NetovikConfig":
        """The sizes that only the tensors tell: the decays' rank and the rows of the tables of distance biases."""
        data, layers = dict(self.data), []
        for i, layer in enumerate(data["layers"]):
            name, key = (f"l{i}.mix.w1", "rank") if layer["type"] == "wkv" else (f"l{i}.mix.rel", "bias_rows")
            if name in shapes and len(shapes[name]) == 2:
                layer = dict(layer, mixer=dict(layer["mixer"], **{key: int(shapes[name][0])}))
            layers.append(layer)
        data["layers"] = layers
        return type(self)(data=data, max_positions=self.max_positions)

    @staticmethod
    def _from_tensor(mixer: Mapping[str, Any], key: str, what: str, layer: int) -> int:
        if mixer.get(key) is None:
            raise ConfigError(f"layer {layer}: {what} come from the tensors of a model folder, or from {key!r} in the "
                              f"layer's mixer")
        return int(mixer[key])

    def model_spec(self) -> ModelSpec:
        data = self.data
        width, eps = self.hidden_size, float(data["norm"]["eps"])
        groups = int(data["norm"].get("groups") or 1)
        norm = lambda base, name: PartSpec("group_rmsnorm", base, {"size": width, "eps": eps, "groups": groups,
                                                                   "weight_name": name})
        count = self.num_layers
        layers = []
        for i, layer in enumerate(data["layers"]):
            base = f"l{i}."
            m = layer["mixer"]
            if layer["type"] == "wkv":
                mixer = PartSpec("wkv", base + "mix.", {
                    "hidden_size": width, "num_heads": int(m["heads"]), "head_dim": int(m["dim"]), "eps": eps,
                    "decay_rank": self._from_tensor(m, "rank", "the rows of the decay's first projection", i)})
            else:
                mask = m.get("mask") or {}
                mixer = PartSpec("mixed_heads_attention", base + "mix.", {
                    "hidden_size": width, "num_heads": int(m["heads"]), "num_kv_heads": int(m.get("kv_heads") or m["heads"]),
                    "head_dim": int(m["dim"]), "scale": float(m["scale"]), "eps": eps, "bias": True,
                    "score_cap": None if m.get("softcap") is None else float(m["softcap"]),
                    "bias_rows": self._from_tensor(m, "bias_rows", "the rows of the distance biases", i),
                    "bias_max": float(m["bias_max"]), "sink_score": 0.0,
                    "window": None if mask.get("size") is None else int(mask["size"]),
                    "keep_first": int(mask.get("keep_first") or 0)})
            parts = {"mixer": mixer, "mixer_post_norm": norm(base, "norm1")}
            mlp = layer.get("mlp")
            if mlp is not None:
                if mlp["kind"] == "dense":
                    parts["feed_forward"] = PartSpec("swiglu", base + "mlp.", {
                        "hidden_size": width, "intermediate_size": int(mlp["ff"]),
                        "gate_name": "gate", "up_name": "up", "down_name": "down"})
                else:
                    parts["feed_forward"] = PartSpec("routed_experts", base + "mlp.", {
                        "hidden_size": width, "num_experts": int(mlp["router"]["experts"]),
                        "top": int(mlp["router"]["top"]), "expert_size": int(mlp["expert"]["ff"]), "router_bias": False,
                        "scoring": "softmax_all", "weight_on": "output", "route_in_hidden": True})
                parts["feed_forward_post_norm"] = norm(base, "norm2")
            layers.append(LayerSpec(PartSpec("depth_averaged_branch_norm", base, {"index": i, "layers": count}), parts))
        return ModelSpec(
            architecture=self.architecture,
            vocab_size=self.vocab_size,
            hidden_size=width,
            max_positions=self.max_positions,
            embedding=PartSpec("token_embedding", "", {
                "vocab_size": self.vocab_size, "hidden_size": width, "weight_name": "embed",
                "scale": float((data.get("embedding") or {}).get("scale") or 1.0)}),
            layers=tuple(layers),
            order=tuple(LayerCall(l) for l in range(count)),
            final_norm=norm("final.", "norm"),
            head=PartSpec("lm_head", "", {"vocab_size": self.vocab_size, "hidden_size": width, "tied_to": "embed",
                                          "weight_name": "head"}),
        )
