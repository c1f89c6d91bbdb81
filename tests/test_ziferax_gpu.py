"""Ziferax on the GPU: every kernel of its own against the plain implementation's function of the same mechanism, and
the engine with the HIP kernels through the cuttings of `ziferax_cases` - float32 against tight limits, bfloat16 as
it is served."""

import json
import math
import os
import random
import subprocess
import sys
from types import SimpleNamespace

import pytest
import torch

import schedules
import ziferax_cases as Z
from conftest import ROOT, random_ids
from plain import ziferax_plain as plain
from test_mekuvik_gpu import _pages_for
from test_tukevik_gpu import _ctx

pytestmark = pytest.mark.gpu
DEVICE = "cuda:0"


@pytest.fixture(scope="module")
def hip():
    from ampere_kv_engine_amd.kernels.hip import HipKernels
    return HipKernels(DEVICE)


@pytest.fixture(scope="module", params=list(Z.ZIFERAX))
def case(request, tmp_path_factory):
    return Z.make_case(request.param, str(tmp_path_factory.mktemp(f"ziferax_{request.param}")))


@pytest.fixture(scope="module", params=["float32", "bfloat16"])
def engine(request, case):
    return Z.make_engine(case, request.param, DEVICE)


# ---- the engine through the cuttings -----------------------------------------------------------------------------------

@pytest.mark.filterwarnings("ignore:a bfloat16 matrix")
@pytest.mark.parametrize("cutting", Z.CUTTINGS, ids=lambda f: f.__name__)
def test_cutting(engine, case, cutting):
    if cutting is Z.case_greedy_generation and engine.config.dtype != "float32":
        pytest.skip("greedy tokens are compared with the plain float32 implementation's")
    cutting(engine, case)
    assert engine.kernels.parts_library_path.endswith("libakv_parts.so")


@pytest.mark.filterwarnings("ignore:a bfloat16 matrix")
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mechanism", Z.MECHANISMS)
def test_one_mechanism_alone(mechanism, dtype, tmp_path):
    case = Z.make_case(mechanism, str(tmp_path), Z.alone(mechanism))
    engine = Z.make_engine(case, dtype, DEVICE)
    Z.case_whole(engine, case)
    Z.case_prefill_then_token_by_token(engine, case)
    Z.case_portions_down_to_two_tokens(engine, case)
    Z.case_mixed_with_pages_and_slots_used_again(engine, case)


def test_steps_are_recorded_and_replayed(case):
    """Decode steps come again and again: the second is recorded, the later ones are replays; all agree with the plain
    implementation, and with an engine that records nothing to a few units in the last place."""
    ids = case["requests"]["d"]
    want = case["expected"]["d"]
    outs = {}
    for graphs in (True, False):
        engine = Z.make_engine(case, "float32", DEVICE, decode_graphs=graphs)
        got, _ = schedules.run(engine, {"d": ids}, schedules.last_one_by_one({"d": ids}, 60))
        Z.assert_close(got["d"], want, "float32", f"graphs {graphs}")
        outs[graphs] = got["d"]
        if graphs:
            assert any(g is not None for g in engine._graphs.values()), "nothing was recorded"
    torch.testing.assert_close(outs[True], outs[False], rtol=0, atol=2e-5 * float(want.abs().max()))


def test_trace_replay_of_a_random_model(case, tmp_path):
    """bin/trace_run on a configuration file and a seed: the mixed cutting, every position against the plain model."""
    from ampere_kv_engine_amd.config import ZiferaxConfig
    from ampere_kv_engine_amd.weights import write_random_model
    import numpy as np
    config_path = tmp_path / "config.json"
    config_path.write_text(json.dumps(case["raw"]))
    folder = write_random_model(str(tmp_path / "model"), ZiferaxConfig.from_dict(case["raw"]), 9)
    requests = {name: case["requests"][name] for name in ("a", "b", "e")}
    schedule = schedules.mixed(requests, Z.PROMPTS, 16, 64, seed=3)
    out = tmp_path / "out"
    lines = "\n".join(json.dumps(r) for r in schedules.to_trace(requests, schedule)) + "\n"
    done = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--random-config", str(config_path),
                           "--weights-seed", "9", "--dtype", "float32", "--out", str(out), "--max-tokens", "1024"],
                          input=lines, capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [l for l in done.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(len(schedule))]
    fed = {name: 0 for name in requests}
    for number, (entries, _) in enumerate(schedule):
        got = torch.from_numpy(np.fromfile(out / f"{number}.f32", dtype="<f4").reshape(-1, case["raw"]["vocab"]).copy())
        row = 0
        for name, count in entries:
            want = Z.plain_logits(folder, requests[name][:fed[name] + count])[fed[name]:]
            Z.assert_close(got[row:row + count], want, "float32", f"step {number} request {name}")
            fed[name] += count
            row += count


def test_the_command_line_generates_with_a_ziferax_model(case, tmp_path):
    """`python -m ampere_kv_engine_amd.runner` on a configuration file and a seed: one request, and several through the
    scheduler, greedy; the tokens of the plain implementation."""
    import re
    from ampere_kv_engine_amd.config import ZiferaxConfig
    from ampere_kv_engine_amd.weights import write_random_model
    config_path = tmp_path / "config.json"
    config_path.write_text(json.dumps(case["raw"]))
    folder = write_random_model(str(tmp_path / "model"), ZiferaxConfig.from_dict(case["raw"]), 5)
    prompts = [case["requests"]["a"][:19], case["requests"]["b"][:6], case["requests"]["c"][:31]]
    want = [Z.plain_greedy(folder, ids, 6) for ids in prompts]
    base = [sys.executable, "-m", "ampere_kv_engine_amd.runner", "--random-config", str(config_path), "--weights-seed", "5",
            "--max-new-tokens", "6", "--ignore-eos"]
    run = lambda more: subprocess.run(base + more, capture_output=True, text=True, timeout=600, cwd=ROOT)
    one = run(["--mode", "generate", "--dtype", "float32", "--prompt-ids", " ".join(map(str, prompts[0])), "--prefill-chunk", "8"])
    assert one.returncode == 0, one.stderr[-2000:]
    assert json.loads(re.search(r"generated_token_ids = (\[.*\])", one.stdout).group(1)) == want[0]
    prompts_file = tmp_path / "prompts.txt"
    prompts_file.write_text("\n".join(" ".join(map(str, ids)) for ids in prompts) + "\n")
    many = run(["--mode", "generate", "--dtype", "float32", "--prompts-file", str(prompts_file), "--max-seqs", "2",
                "--prefill-chunk", "5"])
    assert many.returncode == 0, many.stderr[-2000:]
    got = [json.loads(line)["generated_token_ids"] for line in many.stdout.splitlines() if line.startswith("{")]
    assert got == want, many.stdout
    check = run(["--mode", "check", "--prompt-len", "40"])
    assert check.returncode == 0, check.stdout[-1500:] + check.stderr[-1500:]


def random_configuration(seed: int) -> tuple:
    """Sizes, constants, the order of layers and whose tensors they run drawn from a seed: any head counts and groupings,
    keys and rotated dimensions of many widths (some no multiple of 8), windows from one position to longer than a request
    or none, any number of experts and identity experts of which one to all are chosen, with and without a shared one."""
    rng = random.Random(seed)
    layers = []
    for index in range(rng.choice((2, 3, 4, 6))):
        if index and rng.random() < 0.35:
            owner = rng.randrange(index)
            layers.append(dict({k: v for k, v in layers[owner].items() if k != "weights_of"}, weights_of=owner))
            continue
        kv, group = rng.choice((1, 2, 3)), rng.choice((1, 2, 4, 5))
        dim = rng.choice((8, 12, 32, 64, 72, 80, 128))
        dims = rng.choice((None,) + tuple(d for d in (2, 4, 8, 12, 32, 64) if d <= dim))
        window = rng.choice((None, 1, 2, 5, 16, 31, 64, 100, 500))
        experts, identity = rng.choice((1, 2, 5, 8, 17, 70)), rng.choice((0, 1, 2, 5))
        mlp = rng.choice((None,) + 4 * (Z.MOE(experts, identity, rng.randint(1, min(experts + identity, 6)), rng.choice((8, 20, 33, 64)),
                                              rng.choice((0.3, 1.0, 4.0)), rng.choice((None, 8, 48, 21)), rng.choice((0.5, 2.0))),))
        layers.append(Z.LAYER(Z.ATTN(kv * group, kv, dim, rng.uniform(0.1, 0.5), window, dims, rng.choice((100.0, 1e4, 1e6))), mlp))
    raw = dict(architecture="Ziferax", vocab=rng.choice((97, 260, 1000)), width=rng.choice((40, 72, 96, 120, 192, 100)),
               norm=dict(eps=rng.choice((1e-5, 1e-6))), residual_mult=rng.choice((0.2, 0.7, 1.0, 1.5)), layers=layers)
    return raw, seed, rng.choice((4, 8, 16, 32))


@pytest.mark.filterwarnings("ignore:a bfloat16 matrix")
@pytest.mark.parametrize("seed", range(900, 912))
def test_a_random_configuration_through_the_cuttings(seed, tmp_path):
    config = random_configuration(seed)
    print(f"seed {seed}: {config[0]}, pages of {config[2]}", flush=True)
    case = Z.make_case(f"random {seed}", str(tmp_path), config)
    for dtype in ("float32", "bfloat16"):
        engine = Z.make_engine(case, dtype, DEVICE)
        hold = Z.check if dtype == "float32" else Z.check_spread
        hold(engine, case, schedules.whole(case["requests"]))
        hold(engine, case, schedules.portions(case["requests"]))
        hold(engine, case, schedules.last_one_by_one(case["requests"], 32))
        hold(engine, case, schedules.mixed(case["requests"], Z.PROMPTS, case["page_size"], engine.config.num_pages, seed=seed))


LONG = {
    "no window": [Z.LAYER(Z.ATTN(4, 2, 32, 0.5, None, 16, 1e4), None)],
    "a long window": [Z.LAYER(Z.ATTN(6, 3, 24, 0.4, 200, 16, 1e5), None)],
    "tensors run again": [Z.LAYER(Z.ATTN(4, 1, 64, 0.2, 170, 32, 1e5), None), Z.LAYER(Z.ATTN(4, 1, 64, 0.2, 170, 32, 1e5), None, 0)],
}


@pytest.mark.filterwarnings("ignore:a bfloat16 matrix")
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mechanism", list(LONG))
def test_long_requests_whose_far_keys_count(mechanism, dtype, tmp_path):
    """Attention alone, made sharp, over requests of several hundred tokens in pages of 16: a query's few heavy keys lie
    anywhere in what it sees, so a page or a tile of keys that went missing far back moves the logits.  Whole, in portions of
    2 to 128 tokens, and with the last 40 tokens one by one - where a window passes over decoded tokens."""
    from ampere_kv_engine_amd.config import EngineConfig
    from ampere_kv_engine_amd.engine import Engine
    raw = dict(architecture="Ziferax", vocab=150, width=64, norm=dict(eps=1e-6), residual_mult=0.9, layers=LONG[mechanism])
    folder = Z.make_folder(str(tmp_path), raw, 121 + list(LONG).index(mechanism))
    requests = {"a": random_ids(150, 530, seed=1), "b": random_ids(150, 263, seed=2)}
    expected = {name: Z.plain_logits(folder, ids) for name, ids in requests.items()}
    engine = Engine.from_folder(folder, EngineConfig(dtype=dtype, page_size=16, num_pages=56, max_seqs=4, max_batched_tokens=640,
                                                     max_seq_len=640, device=DEVICE))
    for what, schedule in (("whole", schedules.whole(requests)),
                           ("portions", schedules.portions(requests, sizes=(2, 3, 37, 64, 5, 128, 2, 16, 90, 2))),
                           ("last tokens one by one", schedules.last_one_by_one(requests, 40))):
        got, _ = schedules.run(engine, requests, schedule)
        for name, want in expected.items():
            Z.assert_close(got[name], want, dtype, f"{mechanism}, {what}, request {name}")
    assert engine.cache.num_free_pages == [56] * len(engine.cache.groups)


# ---- the kernels one by one, against the plain functions ----------------------------------------------------------------

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv_heads,dim,dims,page,window", [
    (4, 2, 16, 12, 4, 11), (3, 1, 40, 40, 16, 64), (8, 2, 64, 32, 16, 72), (2, 1, 128, 64, 16, 200), (8, 8, 32, 2, 8, 20),
    (2, 2, 256, 128, 16, None), (6, 3, 64, 0, 32, 33), (5, 5, 24, 8, 8, 1)])
def test_attention_whose_values_are_its_keys_alone(hip, dtype, heads, kv_heads, dim, dims, page, window):
    """Two requests in two portions each and a last token alone, through the interleaved rotation with the cache write and
    the attention with its sinks, against the plain attention of the whole sequences.  Keys are made to stand out at position
    0, in the middle of the long request and at its window's far edge: each must count for exactly the queries that see it -
    just inside and just outside the window, in prompts and for the token that comes alone - and its value is the key as it
    was before the rotation."""
    torch.manual_seed(heads * 100 + dim)
    lengths = (75, 700 if dim <= 64 else 330)
    scale = 4.0 / math.sqrt(dim)
    q_size, k_size = heads * dim, kv_heads * dim
    width = q_size + k_size
    rows = [torch.randn(n, width) for n in lengths]
    # every query leans along one direction (beyond the rotated dimensions, where there are any); the marked keys lie along it
    lo = dims if dims < dim else 0
    along = torch.zeros(dim)
    along[lo:] = torch.randint(0, 2, (dim - lo,)).float() * 2 - 1
    for projected, n in zip(rows, lengths):
        projected[:, :q_size].view(n, heads, dim).add_(0.4 * along)
        for needle in {0, n // 2, max(n - 1 - (window or n), 0), max(n - (window or n), 0)}:
            projected[needle, q_size:].view(kv_heads, dim)[:, lo:] = along[lo:] * 3 / (1 + needle % 3)
    rows = [r.to(dtype).float() for r in rows]
    sinks = torch.linspace(-2.0, 6.0, heads)
    rotation = {}
    if dims:
        freqs = torch.tensor([1000.0 ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64).float()
        table = torch.empty(max(lengths) + page, dims // 2, 2, dtype=torch.float32, device=DEVICE)
        hip.rope_table(freqs.to(DEVICE), table)
        rotation = dict(table=table, rot_dims=dims, interleaved=True)
    k_pages, v_pages, block_table = _pages_for(lengths, page, kv_heads, dim, dim, dtype)
    got = [torch.zeros(n, heads * dim) for n in lengths]
    steps = [((0, 0), (41, 5)), ((41, 5), (lengths[0] - 42, lengths[1] - 6)), ((lengths[0] - 1, lengths[1] - 1), (1, 1))]
    for befores, counts in steps:
        ctx = _ctx(befores, counts)
        projected = torch.cat([rows[r][b:b + c] for r, (b, c) in enumerate(zip(befores, counts))]).to(dtype).to(DEVICE)
        slot_map = torch.tensor([int(block_table[r, p // page]) * page + p % page for r, (b, c) in enumerate(zip(befores, counts))
                                 for p in range(b, b + c)], dtype=torch.int32, device=DEVICE)
        meta = SimpleNamespace(block_table=block_table.to(DEVICE), rows=None, width=block_table.shape[1], slot_map=slot_map)
        q = torch.empty(ctx.num_tokens, q_size, dtype=dtype, device=DEVICE)
        out = torch.empty(ctx.num_tokens, heads * dim, dtype=dtype, device=DEVICE)
        more = dict(rotation, positions=ctx.positions) if dims else {}
        hip.unit_norm_write(projected, heads, kv_heads, dim, dim, None, slot_map, k_pages, v_pages, q, keyed_values=True, **more)
        hip.gated_attention(q, k_pages, v_pages, None, 0, ctx, meta, heads, kv_heads, dim, dim, scale, None, None, window, True,
                            out, sink_logits=sinks.to(DEVICE))
        at = 0
        for r, (b, c) in enumerate(zip(befores, counts)):
            got[r][b:b + c] = out[at:at + c].float().cpu()
            at += c
    for r, n in enumerate(lengths):         # the values in their pages: the keys as they were, position by position
        for p in (0, n // 2, n - 1):
            held = v_pages[int(block_table[r, p // page]), :, :, p % page].float().cpu()
            assert torch.equal(held, rows[r][p, q_size:].view(kv_heads, dim)), f"request {r}, position {p}"
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, scale=scale, **({"rot": dict(dims=dims, base=1000.0)} if dims else {}),
             **({"mask": dict(size=window)} if window else {}))
    eye = torch.eye(width)
    w = {"q": eye[:q_size], "k": eye[q_size:], "q.b": torch.zeros(q_size), "k.b": torch.zeros(k_size), "sink": sinks,
         "o": torch.eye(heads * dim), "o.b": torch.zeros(heads * dim)}
    for r, n in enumerate(lengths):
        want = plain.attention(rows[r], w, m)
        error = (got[r] - want).abs().max() / want.abs().max()
        assert error < (3e-5 if dtype == torch.float32 else 0.04), f"request {r}: {error:.2e}"


@pytest.mark.parametrize("tokens,experts,identity,top,shared", [
    (5, 7, 3, 3, True), (40, 16, 0, 1, True), (3, 2, 2, 4, False), (130, 8, 8, 8, True), (1, 1, 0, 1, False), (9, 70, 130, 6, True),
    (300, 256, 64, 70, True), (17, 1, 63, 5, False)])
def test_routing_by_corrected_scores(hip, tokens, experts, identity, top, shared):
    torch.manual_seed(tokens + experts)
    outputs = experts + identity
    logits, correction = torch.randn(tokens, outputs) * 2, torch.randn(outputs) * 0.3
    if outputs > 2:
        correction[1] = correction[0]
        logits[0, :2] = 3.0                                # equal choice scores: the lower index goes first
    if tokens > 2:
        logits[2] = -200.0
        logits[2, -1] = 100.0                              # one score of 1, the others zero: a chosen one may weigh nothing
        logits[1] += 5000.0
    gates = torch.full((tokens, experts + (1 if shared else 0) + (1 if identity else 0)), 7.0, device=DEVICE)
    hip.route_corrected(logits.to(DEVICE), correction.to(DEVICE), gates, experts, top, shared=shared)
    chosen, weights = plain.corrected_choice(logits, torch.eye(outputs), correction, top)
    want = torch.zeros(tokens, outputs).scatter_(1, chosen, weights)
    got = gates.cpu()
    torch.testing.assert_close(got[:, :experts], want[:, :experts], rtol=2e-5, atol=1e-7)
    if shared:
        assert got[:, experts].eq(1).all()
    if identity:
        torch.testing.assert_close(got[:, -1], want[:, experts:].sum(1), rtol=2e-5, atol=1e-7)
    total = got[:, :experts].sum(1) + (got[:, -1] if identity else 0.0)
    assert total[3:].sub(1).abs().max() < 1e-5 if tokens > 3 else True
    again = torch.zeros_like(gates)                        # a token's gates do not depend on what else is in the step
    hip.route_corrected(logits[-1:].to(DEVICE).contiguous(), correction.to(DEVICE), again[:1], experts, top, shared=shared)
    assert torch.equal(again[0], gates[-1])
    with pytest.raises(Exception, match="gates"):
        hip.route_corrected(logits.to(DEVICE), correction.to(DEVICE), torch.zeros(tokens, experts + 5, device=DEVICE), experts, top, shared=shared)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("tokens,experts,ff,shared,extra", [(5, 7, 12, 20, 1), (40, 16, 64, 128, 0), (3, 2, 33, 0, 1), (130, 8, 8, 8, 1), (1, 5, 7, 3, 0)])
def test_the_clamped_gate_of_experts(hip, dtype, tokens, experts, ff, shared, extra):
    """Limits of their own for the experts and for the one every token uses, exact zeros where the gate is zero, and the
    plain expert's activation everywhere else - values on, inside and outside the limits."""
    torch.manual_seed(tokens + ff)
    columns = experts * ff + shared
    gates = torch.rand(tokens, experts + (1 if shared else 0) + extra)
    gates[:, :experts] *= (torch.rand(tokens, experts) < 0.4)
    gate_up = (torch.randn(tokens, 2 * columns) * 2).to(dtype)
    gate_up[0, :4] = torch.tensor([0.75, -0.75, 3.0, -40.0]).to(dtype)
    gate_up[0, columns:columns + 4] = torch.tensor([0.75, -0.75, -3.0, 50.0]).to(dtype)
    gates[0, 0] = 1.0
    act = torch.full((tokens, columns), 9.0, dtype=dtype, device=DEVICE)
    hip.gate_clamped_mul(gate_up.to(DEVICE), gates.to(DEVICE), act, experts, ff, 0.75, plain.SIGMOID_SLOPE, 1.0, 2.5)
    g, u = gate_up[:, :columns].float(), gate_up[:, columns:].float()
    want = torch.empty(tokens, columns)
    for c in range(columns):
        inside = c < experts * ff
        one = torch.ones(1, 1)
        value = plain.clamped_expert(torch.stack((g[:, c], u[:, c]), 1), torch.tensor([[1.0, 0.0]]), torch.tensor([[0.0, 1.0]]), one,
                                     0.75 if inside else 2.5)
        want[:, c] = value[:, 0] * gates[:, c // ff if inside else experts]
    torch.testing.assert_close(act.float().cpu(), want.to(dtype).float(), rtol=2e-5 if dtype == torch.float32 else 1e-2, atol=1e-6)
    unused = gates[:, :experts].repeat_interleave(ff, dim=1) == 0
    assert act[:, :experts * ff].cpu()[unused].eq(0).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_share_of_the_input_meets_the_residual_sum(hip, dtype):
    """Two branches and a weighted share of the rows they read, added times a constant and normed in one kernel; the same
    share added to a branch by a kernel of its own."""
    torch.manual_seed(8)
    for tokens, hidden in ((5, 96), (3, 40), (2, 4100), (1, 10), (300, 2048), (4, 8200)):
        stream = torch.randn(tokens, hidden, device=DEVICE)
        a, b, rows = (torch.randn(tokens, hidden, device=DEVICE).to(dtype) for _ in range(3))
        weights = torch.rand(tokens, 7, device=DEVICE)
        weights[0, 4] = 0.0
        gain = 1 + 0.2 * torch.randn(hidden, device=DEVICE)
        out = torch.empty(tokens, hidden, dtype=dtype, device=DEVICE)
        share = weights[:, 4, None] * rows.float()
        for second in (None, b):
            mine = stream.clone()
            want_stream = stream + 0.6 * (a.float() + (second.float() if second is not None else 0.0) + share)
            more = dict(share=rows, share_weights=weights, share_at=4, **({"delta2": second} if second is not None else {}))
            hip.norm_add_norm(mine, a, None, 0.0, gain, 1e-5, out, delta_scale=0.6, **more)
            torch.testing.assert_close(mine, want_stream, rtol=1e-6, atol=2e-6)
            want = plain.rms_norm(want_stream, gain, 1e-5)
            torch.testing.assert_close(out.float(), want.to(dtype).float(), rtol=1e-5 if dtype == torch.float32 else 8e-3, atol=1e-5)
            settled = stream.clone()
            hip.norm_add_norm(settled, a, None, 0.0, None, 0.0, None, delta_scale=0.6, **more)
            assert torch.equal(settled, mine)
        total = b.clone()
        hip.add_weighted_rows(rows, weights, 4, total)
        torch.testing.assert_close(total.float(), (b.float() + share).to(dtype).float(), rtol=1e-6 if dtype == torch.float32 else 8e-3, atol=1e-6)
    with pytest.raises(Exception, match="share"):
        hip.norm_add_norm(stream, a, gain, 1e-5, None, 0.0, None, share=rows, share_weights=weights, share_at=4)
    with pytest.raises(Exception, match="weights"):
        hip.add_weighted_rows(rows, weights, 7, total)
