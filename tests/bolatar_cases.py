"""Shared by the Bolatar tests on the GPU and, with the torch double of the kernel set, on the host: small
configurations whose sizes differ from each other in every respect, model folders with random weights made sharp
enough that a fault shows, the expectation from the plain implementation, and the check of a schedule."""

import json
import os

import torch
from safetensors.torch import load_file, save_file

import keranex_cases as K
import schedules
import tukevik_cases as T
from conftest import random_ids
from plain import bolatar_plain as plain

DELTA = lambda heads, kv, dim, vdim, conv: dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv)
MLSTM = lambda heads, dim, vdim, cap: dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap)
LEFT = lambda heads, kv, dim, vdim, scale, coef=None, every=None: dict(
    heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale, **({"q_temp": dict(coef=coef, every=every)} if every else {}))
RIGHT = lambda heads, dim, rank: dict(heads=heads, dim=dim, rank=rank)
PARALLEL = lambda left, right: dict(left=left, right=right)
DENSE = lambda ff, limit: dict(kind="dense", ff=ff, limit=limit)

# Keys, values and heads of every mixer of different widths, none a power of two; grouped heads; three taps; a temperature
# that rises every 19 positions; a layer without a feed-forward; limits that clamp many values; widths no multiple of 16.
BOLATAR_A = dict(
    architecture="Bolatar", vocab=211, width=96, max_positions=300, norm=dict(eps=1e-6), embedding=dict(scale=7.0), logit_softcap=6.0,
    layers=[
        dict(type="delta", mixer=DELTA(6, 2, 24, 20, 3), mlp=DENSE(72, 0.8)),
        dict(type="parallel", mixer=PARALLEL(LEFT(6, 2, 24, 16, 0.3, 0.4, 19), RIGHT(3, 20, 12)), mlp=None),
        dict(type="mlstm", mixer=MLSTM(3, 24, 40, 9.0), mlp=DENSE(56, 2.5)),
        dict(type="mlstm", mixer=MLSTM(1, 12, 8, 3.0), mlp=None),
    ])
# One tap (no convolution at all) and five; as many key heads as heads, and one for all; no temperature, and one at every
# position; no softcap; the embedding as it is; heads of six value channels; a low rank that is no multiple of eight.
BOLATAR_B = dict(
    architecture="Bolatar", vocab=130, width=64, max_positions=257, norm=dict(eps=1e-5), embedding=dict(scale=1.0),
    layers=[
        dict(type="parallel", mixer=PARALLEL(LEFT(4, 4, 8, 24, 0.5), RIGHT(5, 8, 5)), mlp=DENSE(48, 1.0)),
        dict(type="delta", mixer=DELTA(2, 2, 40, 8, 1), mlp=None),
        dict(type="mlstm", mixer=MLSTM(4, 8, 6, 14.0), mlp=DENSE(40, 0.5)),
        dict(type="delta", mixer=DELTA(3, 1, 5, 12, 5), mlp=DENSE(24, 1.5)),
        dict(type="parallel", mixer=PARALLEL(LEFT(2, 1, 12, 4, 0.4, -0.2, 1), RIGHT(1, 36, 16)), mlp=None),
    ])
# Sizes in multiples of 32 and 64 and pages of 16 - where the prompts' attention runs on the matrix cores in bfloat16.
BOLATAR_C = dict(
    architecture="Bolatar", vocab=300, width=128, max_positions=400, norm=dict(eps=1e-5), embedding=dict(scale=9.0), logit_softcap=20.0,
    layers=[
        dict(type="parallel", mixer=PARALLEL(LEFT(8, 2, 64, 32, 0.125, 0.5, 40), RIGHT(2, 64, 32)), mlp=DENSE(192, 1.0)),
        dict(type="mlstm", mixer=MLSTM(2, 128, 64, 12.0), mlp=DENSE(160, 3.0)),
        dict(type="delta", mixer=DELTA(4, 2, 64, 128, 4), mlp=DENSE(128, 1.2)),
        dict(type="parallel", mixer=PARALLEL(LEFT(2, 1, 128, 64, 0.1, 0.25, 64), RIGHT(4, 32, 8)), mlp=None),
    ])
BOLATAR = {"A": (BOLATAR_A, 81, 4), "B": (BOLATAR_B, 84, 8), "C": (BOLATAR_C, 83, 16)}        # config, weight seed, page size

LENGTHS, PROMPTS, POOL_TOKENS = K.LENGTHS, K.PROMPTS, K.POOL_TOKENS
# float32: a few hundred float32 operations and recurrences over two hundred tokens; measured up to 4e-6 (1e-4 in a
# drawn configuration whose softmaxes are very sharp).  bfloat16: as served,
# against the plain float32 logits: positions lie within 0.04 (median 0.003 to 0.008) - except where a head's read-out is
# almost zero before it is normed (a first token whose query and key are nearly at right angles: its sign and size are then
# rounding; the torch double, which rounds where the kernels round, shows the same): a twentieth of a request's positions may
# lie beyond.
LIMITS = {"float32": dict(max=3e-4, rms=3e-4), "bfloat16": dict(max=0.06, rms=0.08)}
BEYOND = {"float32": 0.0, "bfloat16": 0.05}


def sharpen(folder: str, raw: dict, seed: int = 0) -> None:
    """Random tensors of N(0, 0.02) hide faults: softmaxes are flat, a state's k v^T vanishes beside anything else, every
    decay is the same and every gate stands at one half.  Projections are scaled, and what sets decays, gates, mixes and the
    attention's bias is drawn over the range in which it matters: states that forget within a token and states that keep a
    hundred of them, heads with a steep and heads with a hardly noticeable distance bias."""
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    generator = torch.Generator().manual_seed(9000 + seed)

    def scale(name, factor):
        tensors[name] = (tensors[name].float() * factor).to(torch.bfloat16)

    def uniform(name, low, high):
        tensors[name] = (low + (high - low) * torch.rand(tensors[name].shape, generator=generator)).to(torch.bfloat16)

    scale("embed", 25.0), scale("pos", 40.0), scale("head", 4.0)
    for index, layer in enumerate(raw["layers"]):
        p = f"l{index}.mix."
        if layer["type"] == "delta":
            for name in ("q", "k", "v", "g", "b", "a"):
                scale(p + name, 12.0)
            for name in ("q.conv", "k.conv", "v.conv"):
                scale(p + name, 40.0)
            uniform(p + "A_log", -5.0, 0.5), uniform(p + "dt_bias", -2.0, 1.0)
        elif layer["type"] == "mlstm":
            for name, factor in (("q", 20.0), ("k", 20.0), ("v", 20.0), ("g", 20.0), ("i", 20.0), ("f", 15.0)):
                scale(p + name, factor)
            uniform(p + "i.b", -3.0, 3.0), uniform(p + "f.b", 0.0, 7.0)
        else:
            for name, factor in (("left.q", 20.0), ("left.k", 20.0), ("left.v", 5.0), ("right.r", 15.0), ("right.k", 15.0),
                                 ("right.v", 15.0), ("right.g", 20.0), ("right.w1", 15.0), ("right.w2", 30.0), ("right.u", 40.0)):
                scale(p + name, factor)
            uniform(p + "left.r1", 0.0, 1.2), uniform(p + "left.r2", 0.0, 1.5), uniform(p + "right.w0", -6.0, 0.5)
        if layer.get("mlp") is not None:
            for name in ("gate", "up", "down"):
                scale(f"l{index}.mlp.{name}", 8.0)
    save_file(tensors, path, metadata={"format": "pt"})


def make_folder(folder: str, raw: dict, seed: int) -> str:
    from ampere_kv_engine_amd.config import BolatarConfig
    from ampere_kv_engine_amd.weights import write_random_model
    write_random_model(folder, BolatarConfig.from_dict(raw), seed)
    sharpen(folder, raw, seed)
    return folder


def plain_logits(folder: str, ids: list[int]) -> torch.Tensor:
    with open(os.path.join(folder, "config.json")) as handle:
        raw = json.load(handle)
    return plain.forward(raw, load_file(os.path.join(folder, "model.safetensors")), ids)


def plain_greedy(folder: str, prompt: list[int], new_tokens: int) -> list[int]:
    ids, out = list(prompt), []
    for _ in range(new_tokens):
        out.append(int(plain_logits(folder, ids)[-1].argmax()))
        ids.append(out[-1])
    return out


def make_case(name: str, folder: str, config=None) -> dict:
    raw, seed, page_size = config if config is not None else BOLATAR[name]
    make_folder(folder, raw, seed)
    requests = {r: random_ids(raw["vocab"], n, seed=700 + i) for i, (r, n) in enumerate(LENGTHS.items())}
    expected = {r: plain_logits(folder, ids) for r, ids in requests.items()}
    return dict(name=name, folder=folder, page_size=page_size, requests=requests, expected=expected, raw=raw)


make_engine = K.make_engine


def errors(got, want, dtype):
    saved = K.LIMITS, K.BEYOND
    K.LIMITS, K.BEYOND = LIMITS, BEYOND
    try:
        return K.errors(got, want, dtype)
    finally:
        K.LIMITS, K.BEYOND = saved


def assert_close(got, want, dtype: str, what: str = ""):
    position, by_max, by_rms = errors(got, want, dtype)
    if position is not None:
        raise AssertionError(f"{what}: first wrong position {position} of {want.reshape(-1, want.shape[-1]).shape[0]}; "
                             f"worst max error {by_max:.2f} x its limit, worst rms error {by_rms:.2f} x its limit ({dtype})")
    return max(by_max, by_rms)


def check(engine, case, schedule):
    got, pages = schedules.run(engine, case["requests"], schedule)
    dtype = engine.config.dtype
    worst = 0.0
    for name, want in case["expected"].items():
        worst = max(worst, assert_close(got[name], want, dtype, f"{case['name']}/{dtype} request {name}"))
    assert engine.cache.num_free_pages == [engine.config.num_pages] * len(engine.cache.groups), "pages were lost"
    assert engine.cache.slots.num_free == engine.config.max_seqs, "slots were lost"
    print(f"[bolatar {case['name']} {dtype}] worst error {worst:.2f} of its limit")
    return pages


def spread(got: dict, case) -> tuple[float, float]:
    """(median, 90th percentile) over all requests' positions of the worst logit's error against the largest |logit|."""
    errors = [(got[name] - want).abs().amax(1) / want.abs().max() for name, want in case["expected"].items()]
    errors = torch.cat(errors)
    assert not torch.isnan(errors).any(), "NaN logits"
    return float(errors.median()), float(errors.quantile(0.9))


# ---- the cuttings (those of the other designs' cases, held to this design's limits) -----------------------------------

def _with_this_check(cutting):
    def run(engine, case, **more):
        saved = T.check, T.plain_logits, T.plain_greedy
        T.check, T.plain_logits, T.plain_greedy = check, plain_logits, plain_greedy
        try:
            return cutting(engine, case, **more)
        finally:
            T.check, T.plain_logits, T.plain_greedy = saved
    run.__name__ = cutting.__name__
    return run


case_whole = _with_this_check(T.case_whole)
case_prefill_then_token_by_token = _with_this_check(T.case_prefill_then_token_by_token)
case_token_by_token_from_the_first = _with_this_check(T.case_token_by_token_from_the_first)
case_portions_down_to_two_tokens = _with_this_check(T.case_portions_down_to_two_tokens)
case_mixed_with_pages_and_slots_used_again = _with_this_check(T.case_mixed_with_pages_and_slots_used_again)
case_first_tokens = _with_this_check(T.case_first_tokens)
case_long_decoding = _with_this_check(T.case_long_decoding)
case_greedy_generation = _with_this_check(T.case_greedy_generation)

CUTTINGS = [case_whole, case_prefill_then_token_by_token, case_token_by_token_from_the_first,
            case_portions_down_to_two_tokens, case_mixed_with_pages_and_slots_used_again, case_first_tokens,
            case_long_decoding, case_greedy_generation]


# ---- one mechanism alone: a small model in which nothing else contributes ----------------------------------------------

def alone(mechanism: str) -> tuple:
    """(config, weight seed, page size) of a small model in which one mechanism alone shapes the logits."""
    tiny = dict(type="mlstm", mixer=MLSTM(1, 8, 4, 5.0))
    layers = {
        "delta rule": dict(type="delta", mixer=DELTA(4, 2, 16, 28, 4), mlp=None),
        "attention beside time mixing": dict(type="parallel", mixer=PARALLEL(LEFT(4, 2, 16, 24, 0.35, 0.6, 11), RIGHT(2, 20, 8)), mlp=None),
        "matrix memory": dict(type="mlstm", mixer=MLSTM(3, 20, 12, 8.0), mlp=None),
        "dense feed-forward": dict(tiny, mlp=DENSE(56, 0.9)),
    }
    raw = dict(architecture="Bolatar", vocab=150, width=48, max_positions=240, norm=dict(eps=1e-6), embedding=dict(scale=3.0),
               logit_softcap=9.0, layers=[layers[mechanism]])
    return raw, 91 + sorted(layers).index(mechanism), 4


MECHANISMS = ("delta rule", "attention beside time mixing", "matrix memory", "dense feed-forward")
