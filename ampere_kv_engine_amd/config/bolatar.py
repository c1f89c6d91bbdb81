"""Typed configuration of the Bolatar decoder, read from the keys of its config.json.

A Bolatar model is a list of layers, each with a mixer of its own kind and sizes and a dense gated feed-forward (or none)
whose gate and value are clamped at `limit`:
  * `delta`: the gated delta rule with a decay per head behind short convolutions, its state in the request's slot;
  * `parallel`: two mixers side by side that read the same input - `left`, grouped-query attention without rotation, its
    queries warmed by position (`q_temp`), its values normed per head, its scores lowered by the logarithm of the distance;
    `right`, time mixing with a decay per key channel and token and a bonus for the current one - whose outputs are normed
    over the model's width, each with a weight of its own, and averaged;
  * `mlstm`: a matrix memory with exponential gates per head under a running maximum.
Tokens' embeddings are scaled and meet a learned vector of their position; every norm of the layers has one number for all
coordinates; the logits pass a softcap.  Every size and every constant that can differ between models is a key of
config.json and travels from here into the part specifications; the rank of a time-mixing decay, which config.json need
not name (`right.rank`), is read from the shapes of the checkpoint's tensors.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass

from .keranex import _get
from .lirulix import UNIT_VECTOR_EPS, _checkpoint_shapes
from .qwen3 import ConfigError
from .specs import LayerSpec, ModelSpec, RunEntry, part

MIXER_TYPES = ("delta", "parallel", "mlstm")
READ_EPS = 1e-6                      # beside the denominator of the matrix memory's read-out: fixed by the design
GATE_SLOPE, VALUE_SHIFT = 1.702, 1.0     # of the feed-forward's activation: fixed by the design
BRANCH_SHARE = 0.5                   # of either side of a parallel mixer: fixed by the design


@dataclass(frozen=True)
class BolatarConfig:
    raw: dict        # config.json as read, with the decays' ranks filled in (checked below; `to_dict` hands it back)

    architecture = "Bolatar"

    # ---- construction ---------------------------------------------------------------------------------
    @classmethod
    def from_dict(cls, raw: dict, shapes: dict | None = None) -> "BolatarConfig":
        """`shapes`: tensor shapes of the checkpoint, from which a size that config.json does not name is taken."""
        raw = json.loads(json.dumps(raw))
        for index, layer in enumerate(raw.get("layers") or []):
            if not (isinstance(layer, dict) and layer.get("type") == "parallel" and isinstance(layer.get("mixer"), dict)
                    and isinstance(layer["mixer"].get("right"), dict)):
                continue
            right, tensor = layer["mixer"]["right"], f"l{index}.mix.right.w1"
            if shapes is not None and tensor in shapes:
                found = int(shapes[tensor][0])
                if right.setdefault("rank", found) != found:
                    raise ConfigError(f"layers[{index}].mixer.right.rank is {right['rank']}, the checkpoint's {tensor} has {found} rows")
        config = cls(raw=raw)
        config._check()
        return config

    @classmethod
    def from_folder(cls, folder: str) -> "BolatarConfig":
        with open(os.path.join(folder, "config.json")) as handle:
            return cls.from_dict(json.load(handle), _checkpoint_shapes(folder))

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

    def _check(self) -> None:
        raw = self.raw
        for key in ("vocab", "width", "max_positions"):
            _get(raw, key)
        _get(raw, "norm.eps", float), _get(raw, "embedding.scale", float, positive=False)
        if raw.get("logit_softcap") is not None:
            _get(raw, "logit_softcap", float)
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
            if kind == "delta":
                for key in ("heads", "kv_heads", "dim", "vdim", "conv"):
                    _get(mixer, key)
                self._check_groups(mixer, f"{where}.mixer")
            elif kind == "mlstm":
                for key in ("heads", "dim", "vdim"):
                    _get(mixer, key)
                _get(mixer, "gate_cap", float)
            else:
                for key in ("left.heads", "left.kv_heads", "left.dim", "left.vdim", "right.heads", "right.dim"):
                    _get(mixer, key)
                self._check_groups(mixer["left"], f"{where}.mixer.left")
                _get(mixer, "left.scale", float)
                if mixer["left"].get("q_temp") is not None:
                    _get(mixer, "left.q_temp.coef", float, positive=False), _get(mixer, "left.q_temp.every")
                if "rank" not in mixer["right"]:
                    raise ConfigError(f"{where}.mixer.right.rank is named neither by config.json nor by a checkpoint's tensors")
                _get(mixer, "right.rank")
            mlp = layer.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
                    raise ConfigError(f"{where}.mlp.kind must be dense")
                _get(mlp, "ff"), _get(mlp, "limit", float)

    @staticmethod
    def _check_groups(sizes: dict, where: str) -> None:
        if sizes["heads"] % sizes["kv_heads"]:
            raise ConfigError(f"{where}.heads {sizes['heads']} is no multiple of kv_heads {sizes['kv_heads']}")

    # ---- the model this configuration describes -------------------------------------------------------
    def _mixer(self, kind: str, m: dict):
        hidden, eps = self.raw["width"], float(self.raw["norm"]["eps"])
        if kind == "delta":
            return part("gated_delta_rule", hidden_size=hidden, heads=m["heads"], kv_heads=m["kv_heads"], head_dim=m["dim"],
                        value_dim=m["vdim"], taps=m["conv"], decay="per_head", unit_eps=UNIT_VECTOR_EPS, eps=eps, name="mix")
        if kind == "mlstm":
            return part("matrix_memory", hidden_size=hidden, heads=m["heads"], head_dim=m["dim"], value_dim=m["vdim"],
                        gate_cap=float(m["gate_cap"]), read_eps=READ_EPS, eps=eps, name="mix")
        left, right = m["left"], m["right"]
        temp = left.get("q_temp")
        attention = part("gated_attention", hidden_size=hidden, q_heads=left["heads"], kv_heads=left["kv_heads"],
                         head_dim=left["dim"], value_dim=left["vdim"], scale=float(left["scale"]), softcap=None, chunk=None,
                         window=None, sink=False, unit_norm_eps=None, head_gate=False, value_norm_eps=eps, distance_bias=True,
                         query_temperature=(float(temp["coef"]), int(temp["every"])) if temp is not None else None,
                         name="mix.left")
        mixing = part("time_mixing", hidden_size=hidden, heads=right["heads"], head_dim=right["dim"], decay_rank=right["rank"],
                      eps=eps, name="mix.right")
        return part("parallel", hidden_size=hidden, branches=((attention, BRANCH_SHARE), (mixing, BRANCH_SHARE)), out_norm_eps=eps)

    def to_model_spec(self) -> ModelSpec:
        raw = self.raw
        hidden, eps = raw["width"], float(raw["norm"]["eps"])
        norm = part("rmsnorm", size=hidden, eps=eps, single_rounding=True, scalar=True)
        layers = []
        for index, layer in enumerate(self.layers):
            mlp = layer.get("mlp")
            feed_forward = part("none") if mlp is None else part(
                "swiglu", hidden_size=hidden, intermediate_size=mlp["ff"], name="mlp", names=("gate", "up", "down"),
                activation="clamped", limit=float(mlp["limit"]), slope=GATE_SLOPE, shift=VALUE_SHIFT)
            layers.append(LayerSpec(
                block=part("scaled_prenorm", hidden_size=hidden, norm=norm, residual_scale=1.0, names=("norm1", "norm2")),
                mixer=self._mixer(layer["type"], layer["mixer"]), feed_forward=feed_forward, prefix=f"l{index}."))
        cap = raw.get("logit_softcap")
        return ModelSpec(
            architecture=self.architecture, vocab_size=raw["vocab"], hidden_size=hidden,
            embedding=part("positioned_embedding", vocab_size=raw["vocab"], hidden_size=hidden, name="embed",
                           scale=float(raw["embedding"]["scale"]), positions="pos", position_rows=raw["max_positions"]),
            layers=tuple(layers), run_order=tuple(RunEntry(i, i) for i in range(len(layers))),
            final_norm=part("rmsnorm", size=hidden, eps=eps, single_rounding=True, scalar=True, name="final.norm"),
            head=part("linear_head", vocab_size=raw["vocab"], hidden_size=hidden, name="head",
                      softcap=float(cap) if cap is not None else None),
            eos_token_ids=tuple(raw.get("eos", ())) if isinstance(raw.get("eos"), list) else (),
            max_position=raw["max_positions"],
        )
