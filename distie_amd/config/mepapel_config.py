"""The Mepapel decoder: its config.json and the parts it is made of.

config.json names everything that can differ between models of the design:

    architecture "Mepapel", vocab, width, norm {eps}, residual_mult (what every sub-layer's normed result is multiplied by
    before it is added; one if left out), and `layers`, one entry a layer: `type` ("mamba2" | "delta" | "parallel"),
    `mixer` (its sizes) and `mlp` (or null).

    mamba2 mixer: heads, vdim, state, groups, conv (taps), norm_groups (groups and norm_groups are one if left out).
    delta mixer: heads, kv_heads (heads if left out), dim, vdim (dim if left out), conv (taps).
    parallel mixer: left {heads, kv_heads, dim, vdim, conv, rot {base, dims}, scale, mask {size}} (no convolution, rotation
    or mask where the key is left out) and right {heads, dim, vdim, rot, decay: one number a head}.
    mlp: {"kind": "dense", "ff", "limit"} or {"kind": "moe", "router" {experts, top, scale, groups {count, keep}},
    "expert" {ff}, "shared" {ff}} (scale one, one group, no shared expert where the key is left out).

Tensors: `embed`, `head`, `final.norm`; layer i under `l<i>.`: `norm1`, `norm2`, `mix.*` (a parallel layer's mixers under
`mix.left.*` and `mix.right.*`), `mlp.gate|up|down` or `mlp.router`, `mlp.correction`, `mlp.e<e>.gate|up|down`,
`mlp.shared.gate|up|down|sg`. Linear weights are [out, in]. Nothing here fixes a size.

What the design fixes, and where it stands: norms behind the sub-layers only (`branch_norm_residual`); in the left mixer
biases on all four projections, a norm on every head of q and k, rotation of neighbouring dimensions and chunks of positions
that see only themselves; in the right one rotation by halves; the constants of the clamped feed-forward below; experts
chosen by sigmoid scores with a correction and weighted by those scores' shares.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .model_config import ConfigError, LayerCall, LayerSpec, ModelSpec, PartSpec
from .musutar_config import DEFAULT_MAX_POSITIONS, _need

LAYER_TYPES = ("mamba2", "delta", "parallel")
DENSE_SLOPE = 1.702          # g * sigmoid(DENSE_SLOPE * g) * (u + DENSE_UP_SHIFT)
DENSE_UP_SHIFT = 1.0


def _sizes(data: Mapping[str, Any], keys, where: str, optional=()) -> None:
    for key in keys:
        if _need(data, key, int, where) < 1:
            raise ConfigError(f"{where}: {key} must be >= 1")
    for key in optional:
        if data.get(key) is not None and _need(data, key, int, where) < 1:
            raise ConfigError(f"{where}: {key} must be >= 1")


def _check_kv_heads(m: Mapping[str, Any], where: str) -> None:
    if int(m["heads"]) % int(m.get("kv_heads") or m["heads"]):
        raise ConfigError(f"{where}: heads must be a multiple of kv_heads")


def _check_rot(m: Mapping[str, Any], where: str) -> None:
    rot = m.get("rot")
    if not rot:
        return
    dims = _need(rot, "dims", int, where + " rot")
    if not _need(rot, "base", float, where + " rot") > 0:
        raise ConfigError(f"{where}: rot.base must be positive")
    if dims < 2 or dims % 2 or dims > int(m["dim"]):
        raise ConfigError(f"{where}: rot.dims must be even and at most dim")


@dataclass(frozen=True)
class MepapelConfig:
    data: Mapping[str, Any]
    max_positions: int = DEFAULT_MAX_POSITIONS

    architecture = "Mepapel"

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
    def from_dict(cls, data: Mapping[str, Any]) -> "MepapelConfig":
        vocab, width = _need(data, "vocab", int, "the model"), _need(data, "width", int, "the model")
        if vocab < 1 or width < 1:
            raise ConfigError("vocab and width must be >= 1")
        _need(data.get("norm") or {}, "eps", float, "norm")
        if data.get("residual_mult") is not None:
            _need(data, "residual_mult", float, "the model")
        layers = data.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("config.json lacks 'layers'")
        for i, layer in enumerate(layers):
            where = f"layer {i}"
            kind = _need(layer, "type", str, where)
            if kind not in LAYER_TYPES:
                raise ConfigError(f"{where}: unknown layer type {kind!r}")
            mixer = layer.get("mixer")
            if not isinstance(mixer, Mapping):
                raise ConfigError(f"config.json: {where} lacks 'mixer'")
            getattr(cls, f"_check_{kind}")(mixer, where)
            if layer.get("mlp") is not None:
                cls._check_mlp(layer["mlp"], where + " mlp")
        return cls(data=dict(data), max_positions=int(data.get("max_positions") or DEFAULT_MAX_POSITIONS))

    @staticmethod
    def _check_mamba2(m: Mapping[str, Any], where: str) -> None:
        _sizes(m, ("heads", "vdim", "state", "conv"), where, ("groups", "norm_groups"))
        if int(m["heads"]) % int(m.get("groups") or 1):
            raise ConfigError(f"{where}: heads must be a multiple of groups")
        if (int(m["heads"]) * int(m["vdim"])) % int(m.get("norm_groups") or 1):
            raise ConfigError(f"{where}: heads * vdim must be a multiple of norm_groups")

    @staticmethod
    def _check_delta(m: Mapping[str, Any], where: str) -> None:
        _sizes(m, ("heads", "dim", "conv"), where, ("kv_heads", "vdim"))
        _check_kv_heads(m, where)

    @staticmethod
    def _check_parallel(m: Mapping[str, Any], where: str) -> None:
        left, right = m.get("left"), m.get("right")
        if not isinstance(left, Mapping) or not isinstance(right, Mapping):
            raise ConfigError(f"config.json: {where} lacks 'left' or 'right'")
        _sizes(left, ("heads", "dim"), where + " left", ("kv_heads", "vdim", "conv"))
        _check_kv_heads(left, where + " left")
        _check_rot(left, where + " left")
        if not _need(left, "scale", float, where + " left") > 0:
            raise ConfigError(f"{where} left: scale must be positive")
        if left.get("mask"):
            _sizes(left["mask"], ("size",), where + " left mask")
        _sizes(right, ("heads", "dim"), where + " right", ("vdim",))
        _check_rot(right, where + " right")
        decay = right.get("decay")
        if not isinstance(decay, (list, tuple)) or len(decay) != int(right["heads"]):
            raise ConfigError(f"{where} right: decay must hold one value for each of the {right['heads']} heads")

    @staticmethod
    def _check_mlp(mlp: Mapping[str, Any], where: str) -> None:
        kind = _need(mlp, "kind", str, where)
        if kind == "dense":
            _sizes(mlp, ("ff",), where)
            if not _need(mlp, "limit", float, where) > 0:
                raise ConfigError(f"{where}: limit must be positive")
            return
        if kind != "moe":
            raise ConfigError(f"{where}: unknown mlp kind {kind!r}")
        router = mlp.get("router")
        _sizes(router, ("experts", "top"), where + " router")
        experts, top = int(router["experts"]), int(router["top"])
        if router.get("scale") is not None:
            _need(router, "scale", float, where + " router")
        groups = router.get("groups")
        open_experts = experts
        if groups:
            _sizes(groups, ("count", "keep"), where + " router.groups")
            if experts % int(groups["count"]) or int(groups["keep"]) > int(groups["count"]):
                raise ConfigError(f"{where}: router.groups.count must divide the experts and groups.keep be at most count")
            open_experts = experts // int(groups["count"]) * int(groups["keep"])
        if top > open_experts:
            raise ConfigError(f"{where}: router.top is more than the experts that can be chosen")
        _sizes(mlp.get("expert"), ("ff",), where + " expert")
        if mlp.get("shared"):
            _sizes(mlp["shared"], ("ff",), where + " shared")

    def to_dict(self) -> dict:
        return dict(self.data)

    @staticmethod
    def _position(m: Mapping[str, Any]):
        rot = m.get("rot")
        return PartSpec("rope_scaled", "", {"dims": int(rot["dims"]), "base": float(rot["base"])}) if rot else None

    def _mixer(self, kind: str, m: Mapping[str, Any], base: str) -> PartSpec:
        width, eps = self.hidden_size, float(self.data["norm"]["eps"])
        if kind == "mamba2":
            return PartSpec("state_space_duality", base, {
                "hidden_size": width, "num_heads": int(m["heads"]), "value_dim": int(m["vdim"]),
                "state_size": int(m["state"]), "groups": int(m.get("groups") or 1), "conv_taps": int(m["conv"]),
                "norm_groups": int(m.get("norm_groups") or 1), "eps": eps})
        if kind == "delta":
            return PartSpec("gated_delta_rule", base, {
                "hidden_size": width, "num_heads": int(m["heads"]), "num_kv_heads": int(m.get("kv_heads") or m["heads"]),
                "head_dim": int(m["dim"]), "value_dim": int(m.get("vdim") or m["dim"]), "conv_taps": int(m["conv"]),
                "eps": eps})
        left, right = m["left"], m["right"]
        size = (left.get("mask") or {}).get("size")
        mixers = {
            "left": PartSpec("conv_gated_attention", base + "left.", {
                "hidden_size": width, "num_heads": int(left["heads"]),
                "num_kv_heads": int(left.get("kv_heads") or left["heads"]), "head_dim": int(left["dim"]),
                "value_dim": int(left.get("vdim") or left["dim"]), "conv_taps": int(left.get("conv") or 0), "window": None,
                "chunk": None if size is None else int(size), "scale": float(left["scale"]), "output_gate": False,
                "bias": True, "out_bias": True, "qk_norm": {"eps": eps, "offset": 0.0}, "rotate": "neighbours",
                "position": self._position(left)}),
            "right": PartSpec("retention", base + "right.", {
                "hidden_size": width, "num_heads": int(right["heads"]), "head_dim": int(right["dim"]),
                "value_dim": int(right.get("vdim") or right["dim"]), "decay": tuple(float(d) for d in right["decay"]),
                "eps": eps, "rotate": "halves", "position": self._position(right)})}
        return PartSpec("parallel_mixers", base, {"hidden_size": width, "eps": eps, "mixers": mixers})

    def _feed_forward(self, mlp: Mapping[str, Any], base: str) -> PartSpec:
        width = self.hidden_size
        if mlp["kind"] == "dense":
            return PartSpec("swiglu", base, {
                "hidden_size": width, "intermediate_size": int(mlp["ff"]), "activation": "clamped_glu",
                "limit": float(mlp["limit"]), "slope": DENSE_SLOPE, "up_shift": DENSE_UP_SHIFT,
                "gate_name": "gate", "up_name": "up", "down_name": "down"})
        router, groups = mlp["router"], mlp["router"].get("groups") or {}
        scale = router.get("scale")
        return PartSpec("routed_experts", base, {
            "hidden_size": width, "num_experts": int(router["experts"]), "top": int(router["top"]),
            "expert_size": int(mlp["expert"]["ff"]), "router_bias": False, "scoring": "sigmoid_share", "correction": True,
            "groups": int(groups.get("count") or 1), "groups_kept": int(groups.get("keep") or 1),
            "weight_scale": 1.0 if scale is None else float(scale), "weight_on": "output", "route_in_hidden": True,
            "shared_size": int((mlp.get("shared") or {}).get("ff") or 0), "shared_gate": bool(mlp.get("shared"))})

    def model_spec(self) -> ModelSpec:
        data = self.data
        width, eps = self.hidden_size, float(data["norm"]["eps"])
        mult = 1.0 if data.get("residual_mult") is None else float(data["residual_mult"])
        norm = lambda base, name, gain=1.0: PartSpec("rmsnorm", base, {"size": width, "eps": eps, "weight_name": name,
                                                                       "gain": gain})
        layers = []
        for i, layer in enumerate(data["layers"]):
            base = f"l{i}."
            parts = {"mixer": self._mixer(layer["type"], layer["mixer"], base + "mix."),
                     "mixer_post_norm": norm(base, "norm1", mult)}
            if layer.get("mlp") is not None:
                parts["feed_forward"] = self._feed_forward(layer["mlp"], base + "mlp.")
                parts["feed_forward_post_norm"] = norm(base, "norm2", mult)
            layers.append(LayerSpec(PartSpec("branch_norm_residual", base, {}), parts))
        return ModelSpec(
            architecture=self.architecture,
            vocab_size=self.vocab_size,
            hidden_size=width,
            max_positions=self.max_positions,
            embedding=PartSpec("token_embedding", "", {"vocab_size": self.vocab_size, "hidden_size": width,
                                                       "weight_name": "embed"}),
            layers=tuple(layers),
            order=tuple(LayerCall(l) for l in range(len(layers))),
            final_norm=norm("final.", "norm"),
            head=PartSpec("lm_head", "", {"vocab_size": self.vocab_size, "hidden_size": width, "weight_name": "head"}),
        )
