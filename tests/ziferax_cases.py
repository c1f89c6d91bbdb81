"""Shared by the Ziferax tests on the GPU and, with the torch double of the kernel set, on the host: small
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
from plain import ziferax_plain as plain

ATTN = lambda heads, kv, dim, scale, window=None, dims=None, base=None: dict(
    heads=heads, kv_heads=kv, dim=dim, vdim=dim, scale=scale, **({"rot": dict(dims=dims, base=base)} if dims else {}),
    **({"mask": dict(size=window)} if window else {}))
MOE = lambda experts, identity, top, ff, limit, shared=None, shared_limit=None: dict(
    kind="moe", router=dict(experts=experts, identity=identity, top=top), expert=dict(ff=ff, limit=limit),
    **({"shared": dict(ff=shared, limit=shared_limit)} if shared else {}))
LAYER = lambda mixer, mlp, of=None: dict(type="attention", mixer=mixer, mlp=mlp, **({} if of is None else {"weights_of": of}))

WIDE, NARROW = ATTN(6, 2, 24, 0.3, 13, 16, 100.0), ATTN(3, 3, 20, 0.25, 29, 20, 1e4)
MANY, FEW = MOE(7, 3, 3, 20, 0.9, 28, 2.1), MOE(4, 1, 2, 36, 1.6)
# Windows that are no multiple of a page, rotations over a part of the head and over all of it, a layer without a
# feed-forward, one without a shared expert, limits that clamp many values and differ between the experts and the shared
# one; the first layer's tensors run three times, the third layer's twice; widths that are no multiple of 16.
ZIFERAX_A = dict(
    architecture="Ziferax", vocab=211, width=88, norm=dict(eps=1e-6), residual_mult=0.6,
    layers=[LAYER(WIDE, MANY), LAYER(NARROW, None), LAYER(NARROW, FEW), LAYER(WIDE, MANY, 0), LAYER(NARROW, FEW, 2),
            LAYER(WIDE, MANY, 0)])
# A layer that runs the tensors of one behind it, and one that names a layer which names another; no identity experts with
# every expert chosen, identity experts alone beside a single real one, one output a token; a window of one position and one
# of exactly two pages, no window, no rotation, a rotation over a single pair; one key head for all heads.
ONE, TWO, OPEN, BARE = ATTN(4, 4, 8, 0.5, 1, 8, 1e6), ATTN(5, 1, 40, 0.12, 16, 2, 50.0), ATTN(4, 2, 16, 0.4, None, 4, 300.0), ATTN(2, 1, 12, 0.35, 40)
ZIFERAX_B = dict(
    architecture="Ziferax", vocab=130, width=64, norm=dict(eps=1e-5), residual_mult=1.0,
    layers=[LAYER(OPEN, MOE(3, 0, 3, 40, 1.0, 16, 0.7), 3), LAYER(ONE, MOE(1, 6, 4, 48, 1.2, 8, 1.2)), LAYER(TWO, MOE(9, 2, 1, 8, 0.5)),
            LAYER(OPEN, MOE(3, 0, 3, 40, 1.0, 16, 0.7)), LAYER(OPEN, MOE(3, 0, 3, 40, 1.0, 16, 0.7), 0), LAYER(BARE, None)])
# Sizes in multiples of 32 and pages of 16 - where the prompts' attention runs on the matrix cores in bfloat16.
LARGE, SLIM = ATTN(8, 2, 64, 0.125, 50, 32, 1e5), ATTN(4, 4, 32, 0.18, 33, 32, 1e4)
ZIFERAX_C = dict(
    architecture="Ziferax", vocab=300, width=128, norm=dict(eps=1e-5), residual_mult=0.35,
    layers=[LAYER(LARGE, MOE(6, 2, 2, 64, 1.4, 96, 0.8)), LAYER(SLIM, MOE(12, 4, 4, 32, 1.1, 64, 3.0)), LAYER(LARGE, MOE(6, 2, 2, 64, 1.4, 96, 0.8), 0),
            LAYER(ATTN(2, 1, 128, 0.1, 70, 64, 1e4), MOE(5, 1, 3, 48, 0.9))])
ZIFERAX = {"A": (ZIFERAX_A, 101, 4), "B": (ZIFERAX_B, 102, 8), "C": (ZIFERAX_C, 103, 16)}        # config, weight seed, page size

LENGTHS, PROMPTS, POOL_TOKENS = K.LENGTHS, K.PROMPTS, K.POOL_TOKENS
# float32: a few hundred float32 operations a position.  bfloat16: as served, against the plain float32 logits: positions lie
# within 0.02 (median 0.004 to 0.01); a tenth of a request's positions may lie beyond, where a rounded activation turns a
# router's close call.
LIMITS = {"float32": dict(max=2e-4, rms=2e-4), "bfloat16": dict(max=0.045, rms=0.055)}
BEYOND = {"float32": 0.0, "bfloat16": 0.1}


def sharpen(folder: str, raw: dict, seed: int = 0) -> None:
    """Random tensors of N(0, 0.02) hide faults: softmaxes are flat and one key more or less hardly shows, a sink is one key
    among many, biases vanish, nothing reaches a limit, the router's scores are all alike and its corrections change no
    choice.  Projections, biases, routers and experts are scaled - to the same effect at any width -; sinks and corrections
    are drawn over the range in which they matter."""
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    generator = torch.Generator().manual_seed(9100 + seed)
    by_width = (88.0 / raw["width"]) ** 0.5

    def scale(name, factor):
        tensors[name] = (tensors[name].float() * factor).to(torch.bfloat16)

    def uniform(name, low, high):
        tensors[name] = (low + (high - low) * torch.rand(tensors[name].shape, generator=generator)).to(torch.bfloat16)

    scale("embed", 25.0)
    for name in list(tensors):
        if name.endswith((".mix.q", ".mix.k")):
            scale(name, 9.0 * by_width)
        elif name.endswith((".mix.q.b", ".mix.k.b", ".mix.o.b")):
            scale(name, 20.0)
        elif name.endswith(".mix.o"):
            scale(name, 6.0)
        elif name.endswith(".mix.sink"):
            uniform(name, -1.0, 4.0)
        elif name.endswith(".mlp.router"):
            scale(name, 12.0 * by_width)
        elif name.endswith(".mlp.correction"):
            uniform(name, -0.3, 0.3)
        elif ".mlp." in name and not name.endswith(".down"):
            scale(name, 7.0 * by_width)
        elif ".mlp." in name:
            scale(name, 7.0)
    save_file(tensors, path, metadata={"format": "pt"})


def make_folder(folder: str, raw: dict, seed: int) -> str:
    from ampere_kv_engine_amd.config import ZiferaxConfig
    from ampere_kv_engine_amd.weights import write_random_model
    write_random_model(folder, ZiferaxConfig.from_dict(raw), seed)
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
    raw, seed, page_size = config if config is not None else ZIFERAX[name]
    make_folder(folder, raw, seed)
    requests = {r: random_ids(raw["vocab"], n, seed=800 + i) for i, (r, n) in enumerate(LENGTHS.items())}
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
    print(f"[ziferax {case['name']} {dtype}] worst error {worst:.2f} of its limit")
    return pages


def check_spread(engine, case, schedule) -> None:
    """For drawn configurations as they are served: many experts and layers make many close calls, so not every position is
    held to the limit - the middle one is, and three quarters of them to twice that."""
    got, _ = schedules.run(engine, case["requests"], schedule)
    errors = torch.cat([(got[name] - want).abs().amax(1) / want.abs().max() for name, want in case["expected"].items()])
    assert not torch.isnan(errors).any(), "NaN logits"
    median, most, limit = float(errors.median()), float(errors.quantile(0.75)), LIMITS[engine.config.dtype]["max"]
    assert median < limit and most < 2 * limit, f"{case['name']}: median {median:.4f}, three quarters within {most:.4f}"
    print(f"[ziferax {case['name']} {engine.config.dtype}] median error {median:.4f}, three quarters within {most:.4f}")


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
    tiny, plain_attention, calm = ATTN(1, 1, 8, 0.3, 2, 4, 100.0), ATTN(4, 2, 16, 0.35), ATTN(4, 2, 16, 0.15, None, 8, 100.0)
    layers = {
        "windowed attention": [LAYER(ATTN(4, 2, 16, 0.35, 11, 12, 1000.0), None)],
        "attention without rotation or window": [LAYER(plain_attention, None)],
        "experts chosen by corrected scores": [LAYER(tiny, MOE(9, 0, 3, 12, 5.0))],
        "identity experts": [LAYER(tiny, MOE(2, 7, 4, 8, 5.0))],
        "shared expert": [LAYER(tiny, MOE(1, 0, 1, 8, 0.4, 36, 0.8))],
        "tensors run again": [LAYER(calm, None), LAYER(tiny, MOE(3, 1, 4, 8, 1.0)), LAYER(calm, None, 0), LAYER(calm, None, 0)],
    }
    raw = dict(architecture="Ziferax", vocab=150, width=48, norm=dict(eps=1e-6), residual_mult=0.8, layers=layers[mechanism])
    return raw, 111 + sorted(layers).index(mechanism), 4


MECHANISMS = ("windowed attention", "attention without rotation or window", "experts chosen by corrected scores", "identity experts",
              "shared expert", "tensors run again")
