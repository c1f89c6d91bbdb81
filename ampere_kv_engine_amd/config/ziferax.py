"""Typed configuration of the Ziferax decoder, read from the keys of its config.json.

A Ziferax model is a list of layers.  Every layer has ONE norm whose output both of its branches read - the mixer and a
feed-forward (or none) -, and their outputs are added to the residual sum together, times `residual_mult`.  The mixer:
  * `attention`: grouped-query attention whose values are its keys as they were projected, before the rotation; biases on
    the queries, the keys and the output; rotary positions over the first `rot.dims` dimensions of every head in
    interleaved pairs; a sliding window; a learned sink per head in the softmax's denominator.
The feed-forward is routed (`moe`): a softmax over all of the router's outputs scores them, the choice looks at score plus
a learned correction, the weights are the chosen scores over their sum; the last `router.identity` outputs hand the input
on as it is, the others are small feed-forwards with a clamped gate, and so is the expert that every token uses (`shared`).
A layer with `weights_of` has no tensors of its own: it runs the named layer's with a cache of its own.  The head is the
embedding table.  Every size and every constant that can differ between models is a key of config.json and travels from
here into the part specifications.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass

from .bolatar import GATE_SLOPE, VALUE_SHIFT
from .keranex import _get
from .qwen3 import ConfigError
from .specs import LayerSpec, ModelSpec, RunEntry, part

MIXER_TYPES = ("attention",)
MLP_KINDS = ("moe",)


@dataclass(frozen=True)
class ZiferaxConfig:
    raw: dict        # config.json as read (checked below; `to_dict` hands it back)

    architecture = "Ziferax"

    # ---- construction ---------------------------------------------------------------------------------
    @classmethod
    def from_dict(cls, raw: dict) -> "ZiferaxConfig":
        config = cls(raw=json.loads(json.dumps(raw)))
        config._check()
        return config

    @classmethod
    def from_folder(cls, folder: str) -> "ZiferaxConfig":
        with open(os.path.join(folder, "config.json")) as handle:
            return cls.from_dict(json.load(handle))

    def to_dict(self) -> dict:
        return json.loads(json.dumps(self.raw))

    @property
    def vocab_size(self) -> int:
        return self.raw["vocab"]

    @property
    def hidden_size(self) -> int:
        return self.raw["width"]

    @property
    def layers(self) -> list[dict]:
        return self.raw["layers"]

    def owner_of(self, index: int) -> int:
        """The layer whose tensors layer `index` runs: itself, or the one that `weights_of` leads to."""
        passed = []
        while self.layers[index].get("weights_of") is not None:
            passed.append(index)
            index = self.layers[index]["weights_of"]
            if not isinstance(index, int) or isinstance(index, bool) or not 0 <= index < len(self.layers):
                raise ConfigError(f"layers[{passed[-1]}].weights_of must name a layer of the model, got {index!r}")
            if index in passed:
                raise ConfigError(f"layers[{passed[0]}].weights_of leads back to itself")
        return index

    def _check(self) -> None:
        raw = self.raw
        _get(raw, "vocab"), _get(raw, "width"), _get(raw, "norm.eps", float), _get(raw, "residual_mult", float, positive=False)
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json key layers must be a non-empty list")
        for index, layer in enumerate(layers):
            where = f"layers[{index}]"
            kind = layer.get("type") if isinstance(layer, dict) else None
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{where}.type is {kind!r}; this design's mixers are {', '.join(MIXER_TYPES)}")
            mixer = layer.get("mixer")
            if not isinstance(mixer, dict):
                raise ConfigError(f"{where}.mixer must be an object")
            for key in ("heads", "kv_heads", "dim", "vdim"):
                _get(mixer, key)
            _get(mixer, "scale", float, positive=False)
            if mixer["heads"] % mixer["kv_heads"]:
                raise ConfigError(f"{where}.mixer.heads {mixer['heads']} is no multiple of kv_heads {mixer['kv_heads']}")
            if mixer["vdim"] != mixer["dim"]:
                raise ConfigError(f"{where}.mixer.vdim {mixer['vdim']} differs from dim {mixer['dim']}, but the values are the keys")
            if mixer.get("rot") is not None:
                dims = _get(mixer, "rot.dims")
                _get(mixer, "rot.base", float)
                if dims % 2 or dims > mixer["dim"]:
                    raise ConfigError(f"{where}.mixer.rot.dims must be even and at most dim {mixer['dim']}")
            if mixer.get("mask") is not None:
                _get(mixer, "mask.size")
            mlp = layer.get("mlp")
            if mlp is None:
                continue
            if not isinstance(mlp, dict) or mlp.get("kind") not in MLP_KINDS:
                raise ConfigError(f"{where}.mlp.kind must be {', '.join(MLP_KINDS)}")
            experts, top = _get(mlp, "router.experts"), _get(mlp, "router.top")
            identity = _get(mlp, "router.identity", positive=False) if mlp["router"].get("identity") is not None else 0
            if identity < 0:
                raise ConfigError(f"{where}.mlp.router.identity must not be negative")
            if top > experts + identity:
                raise ConfigError(f"{where}.mlp.router: {top} experts a token cannot be chosen from {experts} + {identity} outputs")
            for key in ("expert",) + (("shared",) if mlp.get("shared") is not None else ()):
                _get(mlp, f"{key}.ff"), _get(mlp, f"{key}.limit", float)
        for index, layer in enumerate(layers):
            owner = self.owner_of(index)
            if owner != index:
                rest, own = ({k: v for k, v in entry.items() if k != "weights_of"} for entry in (layer, layers[owner]))
                if rest != own:
                    raise ConfigError(f"layers[{index}] runs the tensors of layers[{owner}] but is described differently")

    # ---- the model this configuration describes -------------------------------------------------------
    def _owners(self) -> list[int]:
        """The layers with tensors of their own, in their order."""
        return [i for i in range(len(self.layers)) if self.owner_of(i) == i]

    def run_order(self) -> tuple[RunEntry, ...]:
        """The layers in their order; one that runs another's tensors is a further run of it, with a cache of its own."""
        place = {owner: i for i, owner in enumerate(self._owners())}
        runs: dict[int, int] = {}
        order = []
        for index in range(len(self.layers)):
            spot = place[self.owner_of(index)]
            order.append(RunEntry(spot, spot, cache_copy=runs.get(spot, 0)))
            runs[spot] = runs.get(spot, 0) + 1
        return tuple(order)

    @staticmethod
    def _attention(m: dict, hidden: int):
        mask, rot = m.get("mask"), m.get("rot")
        return part("gated_attention", hidden_size=hidden, q_heads=m["heads"], kv_heads=m["kv_heads"], head_dim=m["dim"],
                    value_dim=m["vdim"], values="keys", scale=float(m["scale"]), softcap=None, chunk=None,
                    window=mask["size"] if mask is not None else None, sink="learned", unit_norm_eps=None, head_gate=False,
                    position=part("rope_scaled", dims=rot["dims"], base=float(rot["base"]), layout="interleaved")
                    if rot is not None else None, bias_suffix=".b", out_bias_suffix=".b", name="mix")

    @staticmethod
    def _feed_forward(mlp: dict | None, hidden: int):
        if mlp is None:
            return part("none")
        router, shared = mlp["router"], mlp.get("shared")
        return part("routed_experts", hidden_size=hidden, expert_size=mlp["expert"]["ff"], experts=router["experts"],
                    top=router["top"], identity=router.get("identity") or 0, activation="clamped_gated",
                    limit=float(mlp["expert"]["limit"]), slope=GATE_SLOPE, shift=VALUE_SHIFT, weights="softmax_corrected",
                    shared_size=shared["ff"] if shared is not None else None,
                    shared_limit=float(shared["limit"]) if shared is not None else None, shared_gate=False, name="mlp")

    def to_model_spec(self) -> ModelSpec:
        raw = self.raw
        hidden, eps = raw["width"], float(raw["norm"]["eps"])
        norm = part("rmsnorm", size=hidden, eps=eps, single_rounding=True)
        layers = tuple(
            LayerSpec(block=part("shared_norm", hidden_size=hidden, norm=norm, residual_scale=float(raw["residual_mult"]), name="norm1"),
                      mixer=self._attention(self.layers[index]["mixer"], hidden),
                      feed_forward=self._feed_forward(self.layers[index].get("mlp"), hidden), prefix=f"l{index}.")
            for index in self._owners())
        return ModelSpec(
            architecture=self.architecture, vocab_size=raw["vocab"], hidden_size=hidden,
            embedding=part("embedding", vocab_size=raw["vocab"], hidden_size=hidden, name="embed"),
            layers=layers, run_order=self.run_order(),
            final_norm=part("rmsnorm", size=hidden, eps=eps, single_rounding=True, name="final.norm"),
            head=part("linear_head", vocab_size=raw["vocab"], hidden_size=hidden, name="head", tied_to="embed"),
            eos_token_ids=tuple(raw.get("eos", ())) if isinstance(raw.get("eos"), list) else (),
        )
