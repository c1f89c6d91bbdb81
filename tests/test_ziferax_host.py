"""Ziferax on the host: its configuration, and the engine's side of it - registry, loading, caches of layers that run
another's tensors, windows, batching, the scheduler - with the torch double standing in for the HIP kernels, against the
plain implementation.  The HIP kernels meet the same cases in `test_ziferax_gpu.py`."""

import copy
import json
import math
import os

import pytest
import torch
from safetensors.torch import load_file

import schedules
import ziferax_cases as Z
from ampere_kv_engine_amd.cache.pages import RELEASED
from ampere_kv_engine_amd.config import ConfigError, RunEntry, ZiferaxConfig, load_config
from ampere_kv_engine_amd.engine.model import expected_tensors
from plain import ziferax_plain as plain
from torch_kernels import TorchKernels


@pytest.fixture(scope="module", params=["A", "B"])       # (the third configuration, of served sizes, meets the GPU alone)
def case(request, tmp_path_factory):
    return Z.make_case(request.param, str(tmp_path_factory.mktemp(f"ziferax_{request.param}")))


@pytest.fixture(scope="module")
def engine(case):
    return Z.make_engine(case, "float32", "cpu", kernels=TorchKernels())


@pytest.mark.parametrize("cutting", Z.CUTTINGS, ids=lambda f: f.__name__)
def test_cutting(engine, case, cutting):
    cutting(engine, case)


@pytest.mark.parametrize("mechanism", Z.MECHANISMS)
def test_one_mechanism_alone(mechanism, tmp_path):
    case = Z.make_case(mechanism, str(tmp_path), Z.alone(mechanism))
    engine = Z.make_engine(case, "float32", "cpu", kernels=TorchKernels())
    Z.case_whole(engine, case)
    Z.case_portions_down_to_two_tokens(engine, case)
    Z.case_mixed_with_pages_and_slots_used_again(engine, case)


# ---- the configuration -----------------------------------------------------------------------------------------------

def test_the_configuration_names_every_part_and_tensor(tmp_path):
    raw = copy.deepcopy(Z.ZIFERAX_A)
    folder = str(tmp_path)
    with open(os.path.join(folder, "config.json"), "w") as handle:
        json.dump(raw, handle)
    config = load_config(folder)                     # found through the key "architecture"
    assert isinstance(config, ZiferaxConfig) and config.to_dict() == raw
    spec = config.to_model_spec()
    assert [layer.prefix for layer in spec.layers] == ["l0.", "l1.", "l2."]        # (the other layers own no tensors)
    assert [layer.feed_forward.kind for layer in spec.layers] == ["routed_experts", "none", "routed_experts"]
    assert all(layer.block.kind == "shared_norm" and layer.block["residual_scale"] == 0.6 and layer.block["norm"]["single_rounding"]
               for layer in spec.layers)
    attention = spec.layers[0].mixer
    assert attention["values"] == "keys" and attention["window"] == 13 and attention["sink"] == "learned" and attention["scale"] == 0.3
    assert attention["position"]["layout"] == "interleaved" and attention["position"]["dims"] == 16 and attention["position"]["base"] == 100.0
    assert attention["bias_suffix"] == attention["out_bias_suffix"] == ".b"
    routed = spec.layers[0].feed_forward
    assert routed["weights"] == "softmax_corrected" and (routed["experts"], routed["identity"], routed["top"]) == (7, 3, 3)
    assert (routed["limit"], routed["shared_limit"], routed["slope"], routed["shift"]) == (0.9, 2.1, 1.702, 1.0)
    assert routed["shared_size"] == 28 and not routed["shared_gate"] and spec.layers[2].feed_forward["shared_size"] is None
    assert spec.head["tied_to"] == "embed"
    assert spec.run_order == (RunEntry(0, 0), RunEntry(1, 1), RunEntry(2, 2), RunEntry(0, 0, cache_copy=1), RunEntry(2, 2, cache_copy=1),
                              RunEntry(0, 0, cache_copy=2))
    assert len({spec.cache_key(entry) for entry in spec.run_order}) == 6
    names = {t.name: tuple(t.shape) for t in expected_tensors(spec) if not t.optional}
    assert names["embed"] == (211, 88) and names["final.norm"] == names["l0.norm1"] == (88,) and "head" not in names
    assert names["l0.mix.q"] == (144, 88) and names["l0.mix.q.b"] == (144,) and names["l0.mix.k"] == (48, 88) and names["l0.mix.k.b"] == (48,)
    assert names["l0.mix.o"] == (88, 144) and names["l0.mix.o.b"] == (88,) and names["l0.mix.sink"] == (6,) and "l0.mix.v" not in names
    assert names["l0.mlp.router"] == (10, 88) and names["l0.mlp.correction"] == (10,) and "l0.mlp.e7.up" not in names
    assert names["l0.mlp.e6.gate"] == names["l0.mlp.e6.up"] == (20, 88) and names["l0.mlp.e0.down"] == (88, 20)
    assert names["l0.mlp.shared.gate"] == (28, 88) and names["l0.mlp.shared.down"] == (88, 28)
    assert not any(name.startswith(("l3.", "l4.", "l5.", "l1.mlp")) for name in names) and "l2.mlp.shared.up" not in names


def test_layers_may_run_the_tensors_of_one_behind_them_and_of_one_that_runs_anothers():
    config = ZiferaxConfig.from_dict(Z.ZIFERAX_B)
    assert [config.owner_of(i) for i in range(6)] == [3, 1, 2, 3, 3, 5]
    spec = config.to_model_spec()
    assert [layer.prefix for layer in spec.layers] == ["l1.", "l2.", "l3.", "l5."]
    assert spec.run_order == (RunEntry(2, 2), RunEntry(0, 0), RunEntry(1, 1), RunEntry(2, 2, cache_copy=1), RunEntry(2, 2, cache_copy=2),
                              RunEntry(3, 3))
    assert spec.layers[3].mixer["position"] is None and spec.layers[2].mixer["window"] is None
    assert [plain.owner_of(Z.ZIFERAX_B["layers"], i) for i in range(6)] == [3, 1, 2, 3, 3, 5]


@pytest.mark.parametrize("change,message", [
    (lambda raw: raw["layers"][1].update(type="rglru"), "type"),
    (lambda raw: raw["layers"][1]["mixer"].update(kv_heads=2), "kv_heads"),
    (lambda raw: raw["layers"][1]["mixer"].update(vdim=16), "vdim"),
    (lambda raw: raw["layers"][1]["mixer"]["rot"].update(dims=7), "rot.dims"),
    (lambda raw: raw["layers"][1]["mixer"]["rot"].update(dims=22), "rot.dims"),
    (lambda raw: raw["layers"][1]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda raw: raw["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda raw: raw["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda raw: raw["layers"][0]["mlp"]["router"].update(top=11), "router"),
    (lambda raw: raw["layers"][0]["mlp"]["router"].update(identity=-1), "identity"),
    (lambda raw: raw["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda raw: raw["layers"][0]["mlp"]["shared"].update(limit=0), "limit"),
    (lambda raw: raw["layers"][3].update(weights_of=6), "weights_of"),
    (lambda raw: raw["layers"][0].update(weights_of=3), "leads back"),
    (lambda raw: raw["layers"][3].update(weights_of=2), "described differently"),
    (lambda raw: raw.pop("residual_mult"), "residual_mult"),
])
def test_configurations_the_design_does_not_allow_are_refused(change, message):
    raw = copy.deepcopy(Z.ZIFERAX_A)
    change(raw)
    with pytest.raises(ConfigError, match=message):
        ZiferaxConfig.from_dict(raw)


# ---- caches ------------------------------------------------------------------------------------------------------------

def test_every_run_of_a_layer_has_a_cache_of_its_own_and_windows_give_pages_back(case, engine):
    from ampere_kv_engine_amd.engine import StepEntry
    spec, page, layers = engine.spec, case["page_size"], case["raw"]["layers"]
    keys = [spec.cache_key(entry) for entry in spec.run_order]
    assert len(set(keys)) == len(keys) == len(engine.cache.layer_cache) == len(layers)
    for key, layer in zip(keys, layers):
        view, m = engine.cache.layer_cache[key], layer["mixer"]
        assert view.k.shape[1:] == (m["kv_heads"], page, m["dim"]) and view.v.shape[1:] == (m["kv_heads"], m["dim"], page)
    assert len({view.k.data_ptr() for view in engine.cache.layer_cache.values()}) == len(layers)
    seq = engine.open("w")
    engine.step([StepEntry(seq, case["requests"]["d"], [])])
    engine.step([StepEntry(seq, case["requests"]["a"][:1], [])])    # (what a window has passed is given back when tokens register)
    windowed = 0
    for table, group in zip(seq.tables, engine.cache.groups):
        if group.need.window is None:
            continue
        windowed += 1
        assert table.num_held <= (group.need.window + page - 1) // page + 1
        assert RELEASED in table.pages, "nothing behind the window was given back"
    assert windowed == len({(l["mixer"]["mask"]["size"], l["mixer"]["kv_heads"], l["mixer"]["dim"]) for l in layers if "mask" in l["mixer"]})
    # two runs of one layer write different keys: their inputs differ
    owners = [plain.owner_of(layers, i) for i in range(len(layers))]
    again = next(i for i in range(len(layers)) if owners[i] in owners[:i])
    first = owners.index(owners[again])
    assert not torch.equal(engine.cache.layer_cache[keys[first]].k, engine.cache.layer_cache[keys[again]].k)
    engine.close(seq)
    assert engine.cache.num_free_pages == [engine.config.num_pages] * len(engine.cache.groups)


def test_an_input_share_is_added_by_blocks_that_take_one_and_by_a_kernel_elsewhere(case):
    """The same feed-forward in a block that adds what identity experts hand on inside its norm, and where it has to add that
    itself: the same numbers."""
    from types import SimpleNamespace
    from ampere_kv_engine_amd.engine.batch import Arena
    from ampere_kv_engine_amd.parts.base import InputShare
    engine = Z.make_engine(case, "float32", "cpu", kernels=TorchKernels())
    index = next(i for i, layer in enumerate(engine.spec.layers) if layer.feed_forward.get("identity"))
    part = engine.model.blocks[index].feed_forward
    x = torch.randn(9, case["raw"]["width"])
    ctx = SimpleNamespace(arena=Arena("cpu", 1 << 20), takes_input_share=True)
    share = part.forward(x, ctx)
    assert isinstance(share, InputShare) and share.rows is x and share.weights[:, share.column].max() > 0
    want = share.delta + share.weights[:, share.column, None] * share.rows
    want = want.clone()
    ctx.arena.reset()
    ctx.takes_input_share = False
    torch.testing.assert_close(part.forward(x, ctx), want)


# ---- the plain implementation's own mechanisms, where a sentence of the design can be checked by hand -----------------

def test_plain_mechanisms_by_hand():
    assert plain.window_mask(4, 2).int().tolist() == [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]
    assert plain.window_mask(3, 1).int().tolist() == [[1, 0, 0], [0, 1, 0], [0, 0, 1]]
    assert plain.window_mask(3, None).int().tolist() == [[1, 0, 0], [1, 1, 0], [1, 1, 1]]
    # a sink of ln 2 beside one key of score 0: 1 / (1 + 2); beside two: 1 / (2 + 2) each
    weights = plain.softmax_with_sink(torch.zeros(2, 2), plain.window_mask(2, None), torch.tensor(math.log(2.0)))
    torch.testing.assert_close(weights, torch.tensor([[1 / 3, 0.0], [0.25, 0.25]]))
    # the pair (2, 3) turns a tenth as fast as (0, 1); dimensions beyond pass
    turned = plain.turn_pairs(torch.arange(6.0).view(1, 1, 6), torch.tensor([2]), 4, 100.0)[0, 0]
    want = [-math.sin(2.0), math.cos(2.0), 2 * math.cos(0.2) - 3 * math.sin(0.2), 3 * math.cos(0.2) + 2 * math.sin(0.2), 4.0, 5.0]
    torch.testing.assert_close(turned, torch.tensor(want))
    # scores (1/2, 1/4, 1/4): a correction brings the last in before the second, the weights know nothing of it
    router = torch.log(torch.tensor([[0.5], [0.25], [0.25]]))
    chosen, weights = plain.corrected_choice(torch.ones(1, 1), router, torch.tensor([0.0, 0.0, 0.1]), 2)
    assert chosen.tolist() == [[0, 2]]
    torch.testing.assert_close(weights, torch.tensor([[2 / 3, 1 / 3]]))
    chosen, weights = plain.corrected_choice(torch.ones(1, 1), router, torch.tensor([-0.6, 0.0, 0.0]), 1)
    assert chosen.tolist() == [[1]] and weights.tolist() == [[1.0]]       # (equal ones: the lower index)
    # gate 3 is held to 1 from above alone, up -5 to -1: (1 sigmoid(1.702)) (-1 + 1) = 0; gate -3 stays
    one = lambda value: torch.tensor([[value]])
    assert plain.clamped_expert(one(1.0), one(3.0), one(-5.0), one(1.0), 1.0).item() == 0.0
    got = plain.clamped_expert(one(1.0), one(-3.0), one(0.5), one(2.0), 1.0).item()
    assert got == pytest.approx(2.0 * -3.0 / (1.0 + math.exp(1.702 * 3.0)) * 1.5, rel=1e-6)
    assert plain.owner_of([{}, {"weights_of": 0}, {"weights_of": 1}], 2) == 0


def test_a_key_at_the_windows_edge_and_the_values_before_rotation_decide_the_output():
    """The plain attention with inputs made so that one key stands out: it is seen from exactly `size` positions, from
    everywhere without a window, hidden by a sink that outweighs it - and its value does not turn with its position."""
    n, size = 40, 7
    wide = lambda rows, cols, entries: torch.tensor([[entries.get((r, c), 0.0) for c in range(cols)] for r in range(rows)])

    def run(marked, mask=True, sink=-50.0):
        h = torch.zeros(n, 3)
        h[:, 0] = 1.0                      # every token: the same query direction
        h[marked, 1] = 1.0                 # one position: a key along the queries (beyond the rotated pair)
        m = dict(heads=1, kv_heads=1, dim=4, vdim=4, scale=40.0, rot=dict(dims=2, base=10000.0), **({"mask": dict(size=size)} if mask else {}))
        w = {"q": wide(4, 3, {(2, 0): 1.0}), "k": wide(4, 3, {(2, 1): 1.0, (0, 1): 1.0}), "q.b": torch.zeros(4), "k.b": torch.zeros(4),
             "sink": torch.tensor([sink]), "o": torch.eye(4), "o.b": torch.tensor([0.0, 0.0, 0.0, 9.0])}
        out = plain.attention(h, w, m)
        assert torch.equal(out[:, 3], torch.full((n,), 9.0)) and out[:, 1].abs().max() < 1e-6      # (no value has turned)
        return (out[:, 0] > 0.5).nonzero().flatten().tolist()

    assert run(9) == list(range(9, 9 + size))
    assert run(0) == list(range(size))
    assert run(3, mask=False) == list(range(3, n))
    assert run(9, sink=60.0) == []


MISTAKES = {
    "a window one key too wide": ("window_mask", lambda n, size, true: true(n, size + 1 if size is not None else None)),
    "a window one key too narrow": ("window_mask", lambda n, size, true: true(n, max(size - 1, 1) if size is not None else None)),
    "no sink": ("softmax_with_sink", lambda scores, seen, sink, true: true(scores, seen, torch.full_like(sink, -1e4))),
    "a sink of 1": ("softmax_with_sink", lambda scores, seen, sink, true: true(scores, seen, torch.zeros_like(sink))),
    "no biases": ("affine", lambda h, matrix, bias, true: h @ matrix.T),
    "pairs in halves": ("turn_pairs", lambda x, positions, dims, base, true: torch.cat((true(
        x[..., :dims].unflatten(-1, (2, dims // 2)).transpose(-1, -2).flatten(-2), positions, dims, base).unflatten(-1, (dims // 2, 2)).transpose(-1, -2).flatten(-2),
        x[..., dims:]), -1)),
    "positions one too large": ("turn_pairs", lambda x, positions, dims, base, true: true(x, positions * 1.05, dims, base)),
    "a choice without corrections": ("corrected_choice", lambda h, router, correction, top, true: true(h, router, 0.0 * correction, top)),
    "weights that are not divided by their sum": ("corrected_choice", lambda h, router, correction, top, true: (
        true(h, router, correction, top)[0], torch.gather(torch.softmax(h @ router.T, -1), 1, true(h, router, correction, top)[0]))),
    "limits that are all alike": ("clamped_expert", lambda h, gate, up, down, limit, true: true(h, gate, up, down, 1.5)),
    "no limits": ("clamped_expert", lambda h, gate, up, down, limit, true: true(h, gate, up, down, 1e9)),
}


@pytest.mark.parametrize("mistake", list(MISTAKES))
def test_a_mistake_in_any_mechanism_leaves_the_limits(case, mistake, monkeypatch):
    """The weights are sharp enough: a mistake planted in the plain implementation moves its logits out of the limits that
    the engine is held to, in both precisions."""
    name, wrong = MISTAKES[mistake]
    true = getattr(plain, name)
    monkeypatch.setattr(plain, name, lambda *args: wrong(*args, true))
    got = Z.plain_logits(case["folder"], case["requests"]["d"])
    for dtype in ("float32", "bfloat16"):
        position, by_max, by_rms = Z.errors(got, case["expected"]["d"], dtype)
        assert position is not None, f"{mistake} stays within the limits of {dtype}: {by_max:.2f}, {by_rms:.2f}"


def test_a_layer_with_another_layers_tensors_does_not_share_its_cache(case):
    """A decoded token's keys are taken from the run's own cache: with the caches of two runs exchanged the logits leave
    the limits."""
    engine = Z.make_engine(case, "float32", "cpu", kernels=TorchKernels())
    ids = {"d": case["requests"]["d"]}
    got, _ = schedules.run(engine, ids, schedules.last_one_by_one(ids, 20))
    Z.assert_close(got["d"], case["expected"]["d"], "float32")
    spec = engine.spec
    entries = [e for e in spec.run_order if e.layer == next(x.layer for x in spec.run_order if x.cache_copy == 1)][:2]
    caches = engine.cache.layer_cache
    original = dict(caches)
    for entry in entries:
        caches[spec.cache_key(entry)] = original[spec.cache_key(entries[0])]      # (both runs write and read one cache)
    got, _ = schedules.run(engine, ids, schedules.last_one_by_one(ids, 20))
    with pytest.raises(AssertionError, match="first wrong position"):
        Z.assert_close(got["d"], case["expected"]["d"], "float32")
