"""Bolatar on the host: its configuration, and the engine's side of it - registry, loading, caches and states, positions a
model does not know, batching, the scheduler - with the torch double standing in for the HIP kernels, against the plain
implementation.  The HIP kernels meet the same cases in `test_bolatar_gpu.py`."""

import copy
import json
import math
import os

import pytest
import torch
from safetensors.torch import load_file

import bolatar_cases as B
from ampere_kv_engine_amd.config import BolatarConfig, ConfigError, RunEntry, load_config
from ampere_kv_engine_amd.engine.model import expected_tensors
from plain import bolatar_plain as plain
from torch_kernels import TorchKernels


@pytest.fixture(scope="module", params=["A", "B"])       # (the third configuration, of served sizes, meets the GPU alone)
def case(request, tmp_path_factory):
    return B.make_case(request.param, str(tmp_path_factory.mktemp(f"bolatar_{request.param}")))


@pytest.fixture(scope="module")
def engine(case):
    return B.make_engine(case, "float32", "cpu", kernels=TorchKernels())


@pytest.mark.parametrize("cutting", B.CUTTINGS, ids=lambda f: f.__name__)
def test_cutting(engine, case, cutting):
    if cutting is B.case_long_decoding:
        cutting(engine, case, tokens=90)         # (the double steps through recurrences token by token on the host)
    else:
        cutting(engine, case)


@pytest.mark.parametrize("mechanism", B.MECHANISMS)
def test_one_mechanism_alone(mechanism, tmp_path):
    case = B.make_case(mechanism, str(tmp_path), B.alone(mechanism))
    engine = B.make_engine(case, "float32", "cpu", kernels=TorchKernels())
    B.case_whole(engine, case)
    B.case_portions_down_to_two_tokens(engine, case)
    B.case_mixed_with_pages_and_slots_used_again(engine, case)


def test_the_configuration_names_every_part_and_tensor(tmp_path):
    raw = copy.deepcopy(B.BOLATAR_A)
    folder = str(tmp_path)
    with open(os.path.join(folder, "config.json"), "w") as handle:
        json.dump(raw, handle)
    config = load_config(folder)                     # found through the key "architecture"
    assert isinstance(config, BolatarConfig) and config.to_dict() == raw
    spec = config.to_model_spec()
    assert [layer.mixer.kind for layer in spec.layers] == ["gated_delta_rule", "parallel", "matrix_memory", "matrix_memory"]
    assert [layer.feed_forward.kind for layer in spec.layers] == ["swiglu", "none", "swiglu", "none"]
    assert all(layer.block.kind == "scaled_prenorm" and layer.block["norm"]["scalar"] and layer.block["norm"]["single_rounding"]
               and layer.block["residual_scale"] == 1.0 for layer in spec.layers)
    delta, both, memory, _ = (layer.mixer for layer in spec.layers)
    assert delta["decay"] == "per_head" and delta["taps"] == 3 and delta["unit_eps"] == 1e-6 and delta["eps"] == 1e-6
    (left, left_share), (right, right_share) = both["branches"]
    assert left_share == right_share == 0.5 and both["out_norm_eps"] == 1e-6
    assert left["distance_bias"] and left["value_norm_eps"] == 1e-6 and left["query_temperature"] == (0.4, 19)
    assert left["scale"] == 0.3 and left["window"] is None and not left["sink"] and left.get("position") is None
    assert right.kind == "time_mixing" and right["decay_rank"] == 12 and right["head_dim"] == 20
    assert memory["gate_cap"] == 9.0 and memory["read_eps"] == 1e-6
    ff = spec.layers[0].feed_forward
    assert ff["activation"] == "clamped" and (ff["limit"], ff["slope"], ff["shift"]) == (0.8, 1.702, 1.0)
    assert spec.embedding.kind == "positioned_embedding" and spec.embedding["scale"] == 7.0 and spec.embedding["position_rows"] == 300
    assert spec.head["softcap"] == 6.0 and spec.head.get("tied_to") is None and spec.max_position == 300
    assert spec.run_order == tuple(RunEntry(i, i) for i in range(4))
    names = {t.name: tuple(t.shape) for t in expected_tensors(spec) if not t.optional}
    assert names["embed"] == names["head"] == (211, 96) and names["pos"] == (300, 96)
    assert names["final.norm"] == names["l0.norm1"] == names["l0.norm2"] == () and "l1.norm2" not in names
    assert names["l0.mix.q"] == names["l0.mix.k"] == (48, 96) and names["l0.mix.v"] == names["l0.mix.g"] == (120, 96)
    assert names["l0.mix.q.conv"] == (48, 3) and names["l0.mix.v.conv"] == (120, 3) and names["l0.mix.norm"] == (20,)
    assert names["l0.mix.a"] == names["l0.mix.b"] == (6, 96) and names["l0.mix.A_log"] == names["l0.mix.dt_bias"] == (6,)
    assert names["l1.mix.left.q"] == (144, 96) and names["l1.mix.left.v"] == (32, 96) and names["l1.mix.left.r1"] == (6,)
    assert names["l1.mix.left.o"] == (96, 96) and names["l1.mix.left.out"] == names["l1.mix.right.out"] == (96,)
    assert names["l1.mix.right.mu.w"] == (96,) and names["l1.mix.right.w1"] == (12, 96) and names["l1.mix.right.w2"] == (60, 12)
    assert names["l1.mix.right.u"] == (3, 20) and names["l1.mix.right.norm"] == (60,) and names["l1.mix.right.o"] == (96, 60)
    assert names["l2.mix.q"] == (72, 96) and names["l2.mix.g"] == (120, 96) and names["l2.mix.f.b"] == (3,) and names["l2.mix.i"] == (3, 96)
    assert names["l2.mlp.up"] == (56, 96) and names["l2.mlp.down"] == (96, 56)
    held = {t.name for t in expected_tensors(BolatarConfig.from_dict(B.BOLATAR_B).to_model_spec())}
    assert "l1.norm2" not in held and "l4.mlp.up" not in held and "l2.norm2" in held


def test_a_decays_rank_comes_from_the_checkpoint_where_the_configuration_does_not_name_it(tmp_path):
    folder = B.make_folder(str(tmp_path), B.BOLATAR_A, 3)
    path = os.path.join(folder, "config.json")
    with open(path) as handle:
        raw = json.load(handle)
    del raw["layers"][1]["mixer"]["right"]["rank"]
    with open(path, "w") as handle:
        json.dump(raw, handle)
    assert load_config(folder).layers[1]["mixer"]["right"]["rank"] == 12
    with pytest.raises(ConfigError, match="rank"):
        BolatarConfig.from_dict(raw)                 # neither named nor to be found
    raw["layers"][1]["mixer"]["right"]["rank"] = 9
    with open(path, "w") as handle:
        json.dump(raw, handle)
    with pytest.raises(ConfigError, match="12 rows"):
        load_config(folder)


@pytest.mark.parametrize("change,message", [
    (lambda raw: raw["layers"][0].update(type="rglru"), "type"),
    (lambda raw: raw["layers"][0]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda raw: raw["layers"][1]["mixer"]["left"].update(kv_heads=4), "kv_heads"),
    (lambda raw: raw["layers"][0]["mixer"].update(conv=0), "conv"),
    (lambda raw: raw["layers"][1]["mixer"].pop("right"), "right"),
    (lambda raw: raw["layers"][1]["mixer"]["left"]["q_temp"].update(every=0), "every"),
    (lambda raw: raw["layers"][1]["mixer"]["left"].pop("scale"), "scale"),
    (lambda raw: raw["layers"][2]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda raw: raw["layers"][2]["mlp"].update(kind="moe"), "kind"),
    (lambda raw: raw["layers"][2]["mlp"].pop("limit"), "limit"),
    (lambda raw: raw.update(logit_softcap=0), "logit_softcap"),
    (lambda raw: raw.pop("max_positions"), "max_positions"),
    (lambda raw: raw["embedding"].pop("scale"), "scale"),
])
def test_configurations_the_design_does_not_allow_are_refused(change, message):
    raw = copy.deepcopy(B.BOLATAR_A)
    change(raw)
    with pytest.raises(ConfigError, match=message):
        BolatarConfig.from_dict(raw)


def test_every_layer_keeps_what_its_mixer_asked_for(case, engine):
    from ampere_kv_engine_amd.engine import StepEntry
    layers, page, width = case["raw"]["layers"], case["page_size"], case["raw"]["width"]
    for index, layer in enumerate(layers):
        view, m = engine.cache.layer_cache[index], layer["mixer"]
        if layer["type"] == "delta":
            channels = 2 * m["kv_heads"] * m["dim"] + m["heads"] * m["vdim"]
            assert view.k is None and view.state.shape == (4, m["heads"] * m["dim"] * m["vdim"] + (m["conv"] - 1) * channels)
        elif layer["type"] == "mlstm":
            assert view.k is None and view.state.shape[1] >= m["heads"] * ((m["vdim"] + 1) * m["dim"] + 1)
        else:
            left, right = m["left"], m["right"]
            assert view.k.shape[1:] == (left["kv_heads"], page, left["dim"]) and view.v.shape[1:] == (left["kv_heads"], left["vdim"], page)
            assert view.state.shape == (4, right["heads"] * right["dim"] ** 2 + width)
    seq = engine.open("w")
    engine.step([StepEntry(seq, case["requests"]["d"], [])])
    states = [view.state for view in engine.cache.layer_cache.values() if view.state is not None]
    assert len(states) == len(layers) and all(state[seq.slot].any() for state in states)
    slot = seq.slot
    engine.close(seq)
    seq = engine.open("again")           # the slot comes round again: nothing of its predecessor is left
    assert seq.slot == slot and not any(state[slot].any() for state in states)
    engine.close(seq)
    assert engine.cache.num_free_pages == [engine.config.num_pages] * len(engine.cache.groups)


def test_a_request_cannot_outgrow_the_positions_the_model_knows(case):
    from ampere_kv_engine_amd.engine import StepEntry
    from ampere_kv_engine_amd.engine.scheduler import Scheduler
    engine = B.make_engine(case, "float32", "cpu", kernels=TorchKernels(), num_pages=400)
    known = case["raw"]["max_positions"]
    ids = B.random_ids(case["raw"]["vocab"], known, seed=8)
    seq = engine.open("w")
    engine.step([StepEntry(seq, ids[:200], [])])
    with pytest.raises(ValueError, match="positions"):
        engine.step([StepEntry(seq, ids[:known - 199], [])])
    assert seq.length == 200                                    # nothing of the step was registered
    engine.step([StepEntry(seq, ids[200:known - 1], [])])
    logits = engine.step([StepEntry(seq, ids[known - 1:], [0])])
    B.assert_close(logits, B.plain_logits(case["folder"], ids)[-1:], "float32", "the last known position")
    engine.close(seq)
    with pytest.raises(ValueError, match="positions"):
        Scheduler(engine).submit("r", ids[:known - 3], 5)
    Scheduler(engine).submit("r", ids[:known - 4], 5)


# ---- parts under a block that takes tensors only ------------------------------------------------------------------------

def test_mixers_side_by_side_norm_their_outputs_themselves_where_the_block_takes_tensors(case, engine):
    """The two branches are normed inside the next norm's kernel where the block says that it takes them so; for any other
    block the mixer returns the tensor of the same sum."""
    from types import SimpleNamespace
    from ampere_kv_engine_amd.engine import StepEntry
    from ampere_kv_engine_amd.engine.batch import Arena
    from ampere_kv_engine_amd.parts.base import NormedPair
    index = next(i for i, layer in enumerate(case["raw"]["layers"]) if layer["type"] == "parallel")
    mixer = engine.model.blocks[index].mixer
    torch.manual_seed(4)
    n, width = 11, case["raw"]["width"]
    x = torch.randn(n, width)
    results = {}
    for unsettled in (True, False):
        seq = engine.open("w")
        ctx, _ = engine.builder.build([StepEntry(seq, [1] * n, [])])
        engine.kernels.step_prologue(ctx)
        ctx.arena, ctx.takes_unsettled_branch = Arena("cpu"), unsettled
        got = mixer.forward(x, ctx, engine.cache.layer_cache[index])
        assert isinstance(got, NormedPair) == unsettled
        stream = torch.zeros(n, width)
        if unsettled:
            got.settle(stream)
        results[unsettled] = stream if unsettled else got
        engine.close(seq)
    torch.testing.assert_close(results[True], results[False], rtol=1e-5, atol=1e-6)
    weights = load_file(os.path.join(case["folder"], "model.safetensors"))
    want = plain.parallel(x, {k: v.float() for k, v in plain.sub_weights(weights, f"l{index}.mix.").items()},
                          case["raw"]["layers"][index]["mixer"], case["raw"]["norm"]["eps"])
    torch.testing.assert_close(results[True], want, rtol=1e-4, atol=1e-4)
    stream = torch.zeros(n, width)
    pair = NormedPair(torch.ones(n, width), torch.full((width,), 2.0), -torch.ones(n, width), torch.ones(width), 0.0, 0.5, engine.kernels)
    pair.times(3.0).settle(stream)
    torch.testing.assert_close(stream, torch.full((n, width), 1.5))       # 3 * 0.5 * (2 - 1)


# ---- the plain implementation's own mechanisms, where a sentence of the design can be checked by hand -----------------

def test_plain_mechanisms_by_hand():
    torch.testing.assert_close(plain.rms_norm(torch.tensor([[3.0, -3.0]]), torch.tensor(0.5), 0.0), torch.tensor([[0.5, -0.5]]))
    torch.testing.assert_close(plain.unit_rms(torch.tensor([[1.0, 7.0]]), 0.0), torch.tensor([[0.2, 1.4]]))
    assert plain.query_temperature(7, 2.0, 3).tolist() == pytest.approx(
        [1.0, 1.0] + [1 + 2 * math.log(2)] * 3 + [1 + 2 * math.log(3)] * 2)          # rises at p = 2 and p = 5
    bias = plain.distance_bias(3, torch.tensor(2.0), torch.tensor(0.5))
    torch.testing.assert_close(bias, torch.tensor([[0, 0, 0], [2 * math.log(1.5), 0, 0], [2 * math.log(2.0), 2 * math.log(1.5), 0]]))
    assert plain.shifted(torch.tensor([[1.0], [2.0], [3.0]])).tolist() == [[0.0], [1.0], [2.0]]
    assert plain.causal_convolution(torch.tensor([[1.0], [2.0], [3.0]]), torch.tensor([[10.0, 1.0]])).tolist() == [[1.0], [12.0], [23.0]]
    sig = lambda z: 1 / (1 + math.exp(-z))
    got = plain.limited_activation(torch.tensor([5.0, -3.0, 0.5]), torch.tensor([0.25, -9.0, 9.0]), 2.0)
    assert got.tolist() == pytest.approx([2 * sig(3.404) * 1.25, -3 * sig(-5.106) * -1.0, 0.5 * sig(0.851) * 3.0])
    torch.testing.assert_close(plain.softplus(torch.tensor([0.0, 30.0, -30.0])), torch.tensor([math.log(2), 30.0, math.exp(-30.0)]))
    torch.testing.assert_close(plain.embed(torch.tensor([1, 0]), torch.tensor([[1.0], [2.0]]), 3.0, torch.tensor([[0.5], [0.25], [9.0]])),
                               torch.tensor([[6.5], [3.25]]))


def _eye(lo, hi, width):
    return torch.eye(width)[lo:hi]


def test_delta_rule_by_hand():
    """One head of one key channel: a unit key is +-1, so S <- g S; S += beta (v k - S), o = S q; both writes and the decay."""
    h = torch.tensor([[4.0, 4.0, 6.0, 0.0, -50.0, 9.0], [4.0, 4.0, -2.0, 0.0, -50.0, 9.0], [4.0, 4.0, 3.0, -60.0, 0.0, 9.0]])
    w = {name: _eye(i, i + 1, 6) for i, name in enumerate(("q", "k", "v", "b", "a", "g"))}
    w.update({f"{n}.conv": torch.ones(1, 1) for n in "qkv"}, A_log=torch.tensor([0.0]), dt_bias=torch.tensor([0.0]), norm=torch.ones(1),
             o=torch.ones(1, 1))
    m = dict(heads=1, kv_heads=1, dim=1, vdim=1, conv=1)
    v = plain.silu(h[:, 2])
    gate = float(plain.silu(torch.tensor(9.0)))
    eps = 1.0                       # (inside the root of a single value's norm: its size stays visible)
    S0 = 0.5 * float(v[0])          # beta one half, nothing decays (softplus(-50) = 0)
    S1 = S0 + 0.5 * (float(v[1]) - S0)
    S2 = 0.5 * S1                   # no write (sigmoid(-60) = 0), and exp(-ln 2) of what was there
    want = [s / math.sqrt(s * s + eps) * gate for s in (S0, S1, S2)]
    got = plain.delta_rule(h, w, m, eps)[:, 0].tolist()
    assert got == pytest.approx(want, rel=1e-4)


def test_matrix_memory_by_hand():
    """One head of one channel.  The running maximum starts at zero: a first token with a small input gate is divided by
    exp(-m) = 1, not by its own weight; later a large gate takes the memory over."""
    h = torch.tensor([[1.0, 2.0, 3.0, 0.0, -4.0, 2.0], [1.0, 1.0, 5.0, 0.0, 6.0, 2.0]])
    w = {name: _eye(i, i + 1, 6) for i, name in enumerate(("q", "k", "v", "g", "i", "f"))}
    w.update({"i.b": torch.zeros(1), "f.b": torch.zeros(1), "norm": torch.ones(1), "o": torch.ones(1, 1)})
    cap, eps = 8.0, 1.0
    i0, i1, f = cap * math.tanh(-4 / cap), cap * math.tanh(6 / cap), -math.log(1 + math.exp(-cap * math.tanh(2 / cap)))
    m0 = max(f, i0)                                             # f > i0: the maximum comes from the gate that forgets zeros
    S0, n0 = math.exp(i0 - m0) * 6, math.exp(i0 - m0) * 2
    o0 = S0 / (max(n0, math.exp(-m0)) + 1e-6)
    m1 = max(f + m0, i1)
    S1, n1 = math.exp(f + m0 - m1) * S0 + math.exp(i1 - m1) * 5, math.exp(f + m0 - m1) * n0 + math.exp(i1 - m1)
    o1 = S1 / (max(n1, math.exp(-m1)) + 1e-6)
    want = [o / math.sqrt(o * o + eps) * 0.5 for o in (o0, o1)]
    got = plain.matrix_memory(h, w, dict(heads=1, dim=1, vdim=1, gate_cap=cap), eps)[:, 0].tolist()
    assert m0 == f and m1 == i1 and got == pytest.approx(want, rel=1e-4)


def test_time_mixing_by_hand():
    """One head of one channel, every mix half of the row and half of the row before: the current token enters through its
    bonus, and its write only the next read-out."""
    h = torch.tensor([[2.0, 1.0, 3.0, 0.0, 1.0], [4.0, 3.0, 1.0, 0.0, 0.0]])
    w = {name: _eye(i, i + 1, 5) for i, name in enumerate(("r", "k", "v", "g"))}
    w.update({f"mu.{s}": torch.full((5,), 0.5) for s in "rkvgw"}, w1=torch.zeros(1, 5), w2=torch.zeros(1, 1), w0=torch.tensor([math.log(math.log(2.0))]),
             u=torch.tensor([[3.0]]), norm=torch.ones(1), o=torch.ones(1, 1))
    w["g"] = torch.zeros(1, 5)
    w["g"][0, 4] = 40.0                                           # the gate reads the last column's mix: 0.5, then 0.5
    gate = 20.0
    eps = 1.0
    r, k, v = (1.0, 3.0), (0.5, 2.0), (1.5, 2.0)                  # mixes with zeros before the first row
    o = [3 * k[0] * v[0] * r[0], (k[0] * v[0] + 3 * k[1] * v[1]) * r[1]]
    got = plain.time_mixing(h, w, dict(heads=1, dim=1), eps)[:, 0].tolist()
    assert got == pytest.approx([x / math.sqrt(x * x + eps) * gate for x in o], rel=1e-4)
    three = torch.cat((h, torch.zeros(1, 5)))
    S = 0.5 * k[0] * v[0] + k[1] * v[1]                           # the decay is one half
    x = (S + 3 * 1.5 * 0.5) * 2.0
    assert plain.time_mixing(three, w, dict(heads=1, dim=1), eps)[2, 0] == pytest.approx(0.0)      # (its gate is shut: the mix is zero)
    w["g"][0, 4], w["g"][0, 0] = 0.0, 10.0
    assert plain.time_mixing(three, w, dict(heads=1, dim=1), eps)[2, 0] == pytest.approx(x / math.sqrt(x * x + eps) * 20.0, rel=1e-4)


def test_a_far_key_decides_the_output_as_far_as_its_distance_allows():
    """The plain attention with one key that stands out: without a bias it is seen from everywhere behind it; with one the
    score falls by r1 ln(1 + r2 d) until the other keys outweigh it; the temperature brings it back."""
    n, marked = 60, 5

    def run(r1, r2, temp=None):
        h = torch.zeros(n, 3)
        h[:, 0] = 1.0
        h[marked, 1] = 1.0
        w = {"q": torch.tensor([[1.0, 0, 0], [0, 0, 0]]), "k": torch.tensor([[0, 1.0, 0], [0, 0, 0]]), "v": torch.tensor([[0, 1.0, 0], [1.0, -1.0, 0]]),
             "r1": torch.tensor([r1]), "r2": torch.tensor([r2]), "o": torch.eye(2)}
        m = dict(heads=1, kv_heads=1, dim=2, vdim=2, scale=12.0, **({"q_temp": temp} if temp else {}))
        # values are normed: the marked key's is (sqrt 2, 0), every other one (0, sqrt 2)
        return (plain.biased_attention(h, w, m, 1e-12)[:, 0] > 0.5 * math.sqrt(2.0)).nonzero().flatten().tolist()

    assert run(0.0, 1.0) == list(range(marked, n))
    seen = run(4.0, 1.0)
    assert seen[0] == marked and seen == list(range(marked, seen[-1] + 1)) and 10 < len(seen) < n - marked
    assert run(4.0, 1.0, dict(coef=3.0, every=20))[-1] == n - 1
