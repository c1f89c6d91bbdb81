"""Bolatar on the GPU: every kernel of its own against the plain implementation's function of the same mechanism, and the
engine with the HIP kernels through the cuttings of `bolatar_cases` - float32 against tight limits, bfloat16 as it is
served."""

import json
import math
import os
import random
import subprocess
import sys
from types import SimpleNamespace

import pytest
import torch

import bolatar_cases as B
import schedules
from conftest import ROOT
from plain import bolatar_plain as plain
from test_mekuvik_gpu import _pages_for
from test_tukevik_gpu import _ctx

pytestmark = pytest.mark.gpu
DEVICE = "cuda:0"


@pytest.fixture(scope="module")
def hip():
    from ampere_kv_engine_amd.kernels.hip import HipKernels
    return HipKernels(DEVICE)


@pytest.fixture(scope="module", params=list(B.BOLATAR))
def case(request, tmp_path_factory):
    return B.make_case(request.param, str(tmp_path_factory.mktemp(f"bolatar_{request.param}")))


@pytest.fixture(scope="module", params=["float32", "bfloat16"])
def engine(request, case):
    return B.make_engine(case, request.param, DEVICE)


@pytest.mark.filterwarnings("ignore:a bfloat16 matrix")
@pytest.mark.parametrize("cutting", B.CUTTINGS, ids=lambda f: f.__name__)
def test_cutting(engine, case, cutting):
    if cutting is B.case_greedy_generation and engine.config.dtype != "float32":
        pytest.skip("greedy tokens are compared with the plain float32 implementation's")
    cutting(engine, case)
    assert engine.kernels.parts_library_path.endswith("libakv_parts.so")


@pytest.mark.filterwarnings("ignore:a bfloat16 matrix")
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mechanism", B.MECHANISMS)
def test_one_mechanism_alone(mechanism, dtype, tmp_path):
    case = B.make_case(mechanism, str(tmp_path), B.alone(mechanism))
    engine = B.make_engine(case, dtype, DEVICE)
    B.case_whole(engine, case)
    B.case_prefill_then_token_by_token(engine, case)
    B.case_portions_down_to_two_tokens(engine, case)
    B.case_mixed_with_pages_and_slots_used_again(engine, case)


def test_steps_are_recorded_and_replayed(case):
    """Decode steps come again and again: the second is recorded, the later ones are replays; all agree with the plain
    implementation, and with an engine that records nothing to a few units in the last place."""
    ids = case["requests"]["d"]
    want = case["expected"]["d"]
    outs = {}
    for graphs in (True, False):
        engine = B.make_engine(case, "float32", DEVICE, decode_graphs=graphs)
        got, _ = schedules.run(engine, {"d": ids}, schedules.last_one_by_one({"d": ids}, 60))
        B.assert_close(got["d"], want, "float32", f"graphs {graphs}")
        outs[graphs] = got["d"]
        if graphs:
            assert any(g is not None for g in engine._graphs.values()), "nothing was recorded"
    torch.testing.assert_close(outs[True], outs[False], rtol=0, atol=2e-5 * float(want.abs().max()))


def test_trace_replay_of_a_random_model(case, tmp_path):
    """bin/trace_run on a configuration file and a seed: the mixed cutting, every position against the plain model."""
    from ampere_kv_engine_amd.config import BolatarConfig
    from ampere_kv_engine_amd.weights import write_random_model
    import numpy as np
    config_path = tmp_path / "config.json"
    config_path.write_text(json.dumps(case["raw"]))
    folder = write_random_model(str(tmp_path / "model"), BolatarConfig.from_dict(case["raw"]), 9)
    requests = {name: case["requests"][name] for name in ("a", "b", "e")}
    schedule = schedules.mixed(requests, B.PROMPTS, 16, 64, seed=3)
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
            want = B.plain_logits(folder, requests[name][:fed[name] + count])[fed[name]:]
            B.assert_close(got[row:row + count], want, "float32", f"step {number} request {name}")
            fed[name] += count
            row += count


def test_the_command_line_generates_with_a_bolatar_model(case, tmp_path):
    """`python -m ampere_kv_engine_amd.runner` on a configuration file and a seed: one request, and several through the
    scheduler, greedy; the tokens of the plain implementation."""
    import re
    from ampere_kv_engine_amd.config import BolatarConfig
    from ampere_kv_engine_amd.weights import write_random_model
    config_path = tmp_path / "config.json"
    config_path.write_text(json.dumps(case["raw"]))
    folder = write_random_model(str(tmp_path / "model"), BolatarConfig.from_dict(case["raw"]), 5)
    prompts = [case["requests"]["a"][:19], case["requests"]["b"][:6], case["requests"]["c"][:31]]
    want = [B.plain_greedy(folder, ids, 6) for ids in prompts]
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
    """Sizes, constants and the order of layers drawn from a seed: any head counts and groupings, keys and values of
    different widths (some no multiple of 4), one to six taps, temperatures from every position to never, layers without a
    feed-forward, low ranks that are no multiple of 8."""
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.choice((2, 3, 4, 5))):
        mlp = rng.choice((None, B.DENSE(rng.choice((40, 64, 100, 132)), rng.choice((0.5, 1.0, 7.0)))))
        kind = rng.choice(("delta", "parallel", "mlstm"))
        kv, group = rng.choice((1, 2, 3)), rng.choice((1, 2, 4, 5))
        dim, vdim = rng.choice((7, 8, 12, 32, 64, 80, 128)), rng.choice((4, 8, 24, 33, 64, 72))
        if kind == "delta":
            mixer = B.DELTA(kv * group, kv, dim, vdim, rng.choice((1, 2, 3, 4, 6)))
        elif kind == "mlstm":
            mixer = B.MLSTM(rng.choice((1, 2, 5)), dim, vdim, rng.choice((2.0, 7.5, 15.0)))
        else:
            left = B.LEFT(kv * group, kv, dim, vdim, rng.uniform(0.1, 0.5), *rng.choice(((None, None), (0.3, 1), (0.7, 13), (-0.1, 50))))
            mixer = B.PARALLEL(left, B.RIGHT(rng.choice((1, 2, 3, 7)), rng.choice((4, 9, 16, 32, 64)), rng.choice((3, 8, 24))))
        layers.append(dict(type=kind, mixer=mixer, mlp=mlp))
    raw = dict(architecture="Bolatar", vocab=rng.choice((97, 260, 1000)), width=rng.choice((40, 72, 96, 120, 192)), max_positions=320,
               norm=dict(eps=rng.choice((1e-5, 1e-6))), embedding=dict(scale=rng.choice((1.0, 5.0, 12.0))), layers=layers)
    if rng.random() < 0.7:
        raw["logit_softcap"] = rng.choice((3.0, 15.0, 30.0))
    return raw, seed, rng.choice((4, 8, 16, 32))


@pytest.mark.filterwarnings("ignore:a bfloat16 matrix")
@pytest.mark.parametrize("seed", range(800, 810))
def test_a_random_configuration_through_the_cuttings(seed, tmp_path):
    """float32 against the plain implementation, position by position.  In bfloat16 a drawn configuration may amplify rounding
    (softmaxes of a few keys, read-outs near zero that are normed): its errors are held to those of the torch double, which
    rounds where the kernels round."""
    from torch_kernels import TorchKernels
    config = random_configuration(seed)
    print(f"seed {seed}: {config[0]}, pages of {config[2]}", flush=True)
    case = B.make_case(f"random {seed}", str(tmp_path), config)
    engine = B.make_engine(case, "float32", DEVICE)
    B.case_whole(engine, case)
    B.case_portions_down_to_two_tokens(engine, case)
    B.case_prefill_then_token_by_token(engine, case)
    B.case_mixed_with_pages_and_slots_used_again(engine, case)
    double = B.make_engine(case, "bfloat16", "cpu", kernels=TorchKernels())
    allowed = B.spread(schedules.run(double, case["requests"], schedules.whole(case["requests"]))[0], case)
    engine = B.make_engine(case, "bfloat16", DEVICE)
    for schedule in (schedules.whole(case["requests"]), schedules.portions(case["requests"]), schedules.last_one_by_one(case["requests"], 32),
                     schedules.mixed(case["requests"], B.PROMPTS, case["page_size"], engine.config.num_pages, seed=5, max_live=3)):
        got = B.spread(schedules.run(engine, case["requests"], schedule)[0], case)
        assert all(g <= 1.5 * a + 0.004 for g, a in zip(got, allowed)), f"bfloat16 (median, 90 %) {got}, the double {allowed}"


LONG = {
    "attention beside time mixing": dict(type="parallel", mlp=None, mixer=B.PARALLEL(B.LEFT(4, 2, 32, 64, 0.4, 0.5, 70), B.RIGHT(3, 24, 8))),
    "delta rule": dict(type="delta", mlp=None, mixer=B.DELTA(4, 2, 24, 16, 4)),
    "matrix memory": dict(type="mlstm", mlp=None, mixer=B.MLSTM(3, 16, 24, 10.0)),
}


@pytest.mark.filterwarnings("ignore:a bfloat16 matrix")
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mechanism", list(LONG))
def test_long_requests_whose_far_tokens_count(mechanism, dtype, tmp_path):
    """One mixer alone, made sharp, over requests of several hundred tokens in pages of 16: a query's few heavy keys lie
    anywhere in its history and states carry hundreds of tokens, so a page, a tile of keys or a tile of the recurrence that
    went missing far back moves the logits.  Whole, in portions of 2 to 128 tokens, and with the last 40 tokens one by one."""
    from ampere_kv_engine_amd.config import EngineConfig
    from ampere_kv_engine_amd.engine import Engine
    from conftest import random_ids
    raw = dict(architecture="Bolatar", vocab=150, width=64, max_positions=600, norm=dict(eps=1e-6), embedding=dict(scale=2.0),
               layers=[LONG[mechanism]])
    folder = B.make_folder(str(tmp_path), raw, 71 + list(LONG).index(mechanism))
    requests = {"a": random_ids(150, 530, seed=1), "b": random_ids(150, 263, seed=2)}
    expected = {name: B.plain_logits(folder, ids) for name, ids in requests.items()}
    engine = Engine.from_folder(folder, EngineConfig(dtype=dtype, page_size=16, num_pages=56, max_seqs=4, max_batched_tokens=640,
                                                     max_seq_len=640, device=DEVICE))
    for what, schedule in (("whole", schedules.whole(requests)),
                           ("portions", schedules.portions(requests, sizes=(2, 3, 37, 64, 5, 128, 2, 16, 90, 2))),
                           ("last tokens one by one", schedules.last_one_by_one(requests, 40))):
        got, _ = schedules.run(engine, requests, schedule)
        for name, want in expected.items():
            B.assert_close(got[name], want, dtype, f"{mechanism}, {what}, request {name}")
    assert engine.cache.num_free_pages == [56] * len(engine.cache.groups)


# ---- the kernels one by one, against the plain functions ----------------------------------------------------------------

def _eye(lo, hi, width):
    return torch.eye(width)[lo:hi]


def _run_steps(lengths, steps, run):
    """Feeds requests of `lengths` tokens in `steps` (tokens held before, tokens brought, per request), in slots that are not
    their rows; `run(ctx, cut)` computes one step's outputs, `cut(rows)` picking the step's tokens out of per-request rows.
    Returns every request's outputs in order."""
    got = [[] for _ in lengths]
    for befores, counts in steps:
        ctx = _ctx(befores, counts)
        ctx.seq_slots = torch.tensor([3, 1], dtype=torch.int32, device=DEVICE)
        ctx.host_seq_slots = [3, 1]
        cut = lambda rows: torch.cat([r[b:b + c] for r, b, c in zip(rows, befores, counts)]).to(DEVICE)
        out, at = run(ctx, cut).float().cpu(), 0
        for r, count in enumerate(counts):
            got[r].append(out[at:at + count])
            at += count
    return [torch.cat(pieces) for pieces in got]


THREE_STEPS = lambda a, b: [((0, 0), (33, 2)), ((33, 2), (1, 1)), ((34, 3), (a - 34, b - 3))]      # a tile and more, single tokens, the rest


def _close(got, want, dtype, f32=3e-5, bf16=0.03):
    error = (got - want).abs().max() / want.abs().max()
    assert not torch.isnan(got).any() and error < (f32 if dtype == torch.float32 else bf16), f"{error:.2e}"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,page,coef,every", [
    (4, 2, 16, 24, 4, 0.4, 19), (3, 1, 40, 8, 16, 0.7, 64), (8, 2, 64, 64, 16, -0.1, 1), (2, 1, 128, 256, 16, 0.3, 100), (8, 8, 64, 32, 8, None, None),
    (2, 2, 32, 128, 32, 1.0, 7), (1, 1, 256, 32, 16, 0.2, 256), (6, 3, 5, 9, 16, 0.5, 30)])
def test_attention_with_a_distance_bias_alone(hip, dtype, heads, kv_heads, dim, vdim, page, coef, every):
    """Two requests in two portions each and a last token alone, through the temperature, the value norm, the cache write and
    the attention, against the plain attention of the whole sequences.  Keys at position 0, at a page's edges and in the
    middle of the long request are made to stand out: how far back they count is the bias's doing - one head has none, one
    forgets within a few tokens -, and the temperature sharpens the far queries, in prompts and for the token that comes
    alone."""
    torch.manual_seed(heads * 100 + dim)
    lengths, eps = (75, 700 if dim <= 64 else 330), 1e-5
    scale = 2.0 / math.sqrt(dim)
    q_size, k_size = heads * dim, kv_heads * dim
    width = q_size + k_size + kv_heads * vdim
    along = torch.randint(0, 2, (dim,)).float() * 2 - 1
    rows = [torch.randn(n, width) for n in lengths]
    for projected, n in zip(rows, lengths):
        projected[:, :q_size].view(n, heads, dim).add_(0.7 * along)
        for needle in {0, page - 1, page, n // 2}:
            projected[needle, q_size:q_size + k_size].view(kv_heads, dim)[:] = along * 5
    rows = [r.to(dtype).float() for r in rows]
    r1 = torch.linspace(0.0, 3.0, heads) if heads > 1 else torch.tensor([1.5])
    r2 = torch.linspace(1.5, 0.02, heads) if heads > 1 else torch.tensor([0.3])
    bias = torch.stack((r1, r2)).to(DEVICE)
    temperature = (coef, every) if every else None
    k_pages, v_pages, block_table = _pages_for(lengths, page, kv_heads, dim, vdim, dtype)
    got = [torch.zeros(n, heads * vdim) for n in lengths]
    steps = [((0, 0), (41, 5)), ((41, 5), (lengths[0] - 42, lengths[1] - 6)), ((lengths[0] - 1, lengths[1] - 1), (1, 1))]
    for befores, counts in steps:
        ctx = _ctx(befores, counts)
        projected = torch.cat([rows[r][b:b + c] for r, (b, c) in enumerate(zip(befores, counts))]).to(dtype).to(DEVICE)
        slot_map = torch.tensor([int(block_table[r, p // page]) * page + p % page for r, (b, c) in enumerate(zip(befores, counts))
                                 for p in range(b, b + c)], dtype=torch.int32, device=DEVICE)
        meta = SimpleNamespace(block_table=block_table.to(DEVICE), rows=None, width=block_table.shape[1], slot_map=slot_map)
        q = torch.empty(ctx.num_tokens, q_size, dtype=dtype, device=DEVICE)
        out = torch.empty(ctx.num_tokens, heads * vdim, dtype=dtype, device=DEVICE)
        hip.unit_norm_write(projected, heads, kv_heads, dim, vdim, None, slot_map, k_pages, v_pages, q, positions=ctx.positions,
                            value_eps=eps, temperature=temperature)
        hip.gated_attention(q, k_pages, v_pages, None, 0, ctx, meta, heads, kv_heads, dim, vdim, scale, None, None, None, False,
                            out, distance_bias=bias)
        at = 0
        for r, (b, c) in enumerate(zip(befores, counts)):
            got[r][b:b + c] = out[at:at + c].float().cpu()
            at += c
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, **({"q_temp": dict(coef=coef, every=every)} if every else {}))
    w = {"q": _eye(0, q_size, width), "k": _eye(q_size, q_size + k_size, width), "v": _eye(q_size + k_size, width, width),
         "o": torch.eye(heads * vdim), "r1": r1, "r2": r2}
    for r, n in enumerate(lengths):
        _close(got[r], plain.biased_attention(rows[r], w, m, eps), dtype, bf16=0.05)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,groups,dim,vdim", [(4, 2, 16, 28), (2, 2, 64, 64), (6, 1, 24, 20), (3, 3, 128, 128), (2, 1, 5, 3), (1, 1, 256, 40),
                                                   (2, 2, 300, 12), (2, 1, 2, 70), (5, 5, 1, 1)])
def test_delta_rule_with_a_decay_per_head_alone(hip, dtype, heads, groups, dim, vdim):
    """Two requests through three steps: unit vectors, decays from keeping everything to forgetting within a token, the walk and
    the normed, gated read-out."""
    torch.manual_seed(dim + vdim)
    lengths, eps = (110, 40), 1e-6
    channels = 2 * groups * dim + heads * vdim
    width = channels + 2 * heads + heads * vdim
    rows = [(torch.randn(n, width) * 1.5).to(dtype).float() for n in lengths]
    a_log, dt_bias = torch.linspace(-6.0, 1.0, heads), torch.linspace(-1.0, 1.0, heads)
    weight = 1 + 0.3 * torch.randn(vdim)
    state = torch.zeros(4, heads * dim * vdim, device=DEVICE)

    def run(ctx, cut):
        x = cut([r.to(dtype) for r in rows])
        out = torch.empty(ctx.num_tokens, heads * vdim, dtype=dtype, device=DEVICE)
        hip.delta_rule(x[:, :channels].contiguous(), x, channels, x, dt_bias.to(DEVICE), torch.exp(a_log).to(DEVICE), x, weight.to(DEVICE),
                       1e-6, eps, dim ** -0.5, heads, groups, dim, vdim, state, ctx, out, decay_at=channels + heads,
                       gate_at=channels + 2 * heads, gate="silu")
        return out

    got = _run_steps(lengths, THREE_STEPS(*lengths), run)
    assert not state[0].any() and not state[2].any() and state[3].any() and state[1].any()
    at = [0, groups * dim, 2 * groups * dim, channels, channels + heads, channels + 2 * heads, width]
    for r, n in enumerate(lengths):
        q, k, v, b, a, g = (rows[r][:, lo:hi] for lo, hi in zip(at, at[1:]))
        q, k = q.reshape(n, groups, dim), k.reshape(n, groups, dim)
        q = (q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * dim ** -0.5).repeat_interleave(heads // groups, 1)
        k = (k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)).repeat_interleave(heads // groups, 1)
        v = v.reshape(n, heads, vdim)
        keep, beta = torch.exp(-torch.exp(a_log) * plain.softplus(a + dt_bias)), torch.sigmoid(b)
        S, out = torch.zeros(heads, dim, vdim), torch.empty(n, heads, vdim)
        for t in range(n):
            S = keep[t][:, None, None] * S
            u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
            S = S + k[t][:, :, None] * u[:, None, :]
            out[t] = (S * q[t][:, :, None]).sum(1)
        want = plain.rms_norm(out, weight, eps) * plain.silu(g).view(n, heads, vdim)
        _close(got[r], want.reshape(n, -1), dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,dim,width,rank", [(2, 16, 40, 8), (1, 64, 64, 16), (3, 20, 36, 5), (4, 32, 70, 24), (2, 128, 96, 8), (1, 3, 10, 4), (2, 260, 24, 8)])
def test_time_mixing_alone(hip, dtype, heads, dim, width, rank):
    """Mixes with the row before (kept in the slot between steps), decays from none to all within a token, the bonus that only
    the current token's write gets, the norm per head and the gate."""
    torch.manual_seed(dim + width)
    lengths, eps, wide = (110, 40), 1e-6, heads * dim
    rows = [torch.randn(n, width).to(dtype).float() for n in lengths]
    w = {s: (torch.randn(wide, width) / math.sqrt(width)).to(dtype).float() for s in "rkvg"}
    w.update({f"mu.{s}": torch.rand(width) for s in "rkvgw"}, w1=torch.randn(rank, width) / math.sqrt(width), w2=torch.randn(wide, rank),
             w0=torch.linspace(-7.0, 1.5, wide), u=torch.randn(heads, dim), norm=1 + 0.3 * torch.randn(wide), o=torch.eye(wide))
    kept_at = heads * dim * dim
    state = torch.zeros(4, kept_at + width, device=DEVICE)
    mu = torch.stack([w[f"mu.{s}"] for s in "rkvgw"]).to(DEVICE)
    inputs = []               # what the recurrence was given, step by step: in bfloat16 it is held to its rounded inputs

    def run(ctx, cut):
        x = cut([r.to(dtype) for r in rows])
        n = ctx.num_tokens
        mixes = torch.empty(5, n, width, dtype=dtype, device=DEVICE)
        hip.token_shift(x, mu, state, kept_at, ctx, mixes)
        rkvg = torch.stack([(mixes[i].float() @ w[s].T.to(DEVICE)).to(dtype) for i, s in enumerate("rkvg")])
        down = mixes[4].float() @ w["w1"].T.to(DEVICE)
        low = torch.empty(n, rank, dtype=torch.float32, device=DEVICE)
        hip.tanh_rows(down, low)
        out = torch.empty(n, wide, dtype=dtype, device=DEVICE)
        logits = low @ w["w2"].T.to(DEVICE)
        inputs.append((ctx.host_q_start, rkvg.float().cpu(), logits.cpu()))
        hip.time_mixing(rkvg, logits, w["w0"].to(DEVICE), w["u"].reshape(-1).to(DEVICE), w["norm"].to(DEVICE), eps, x, heads,
                        dim, state, kept_at, ctx, out)
        return out

    got = _run_steps(lengths, THREE_STEPS(*lengths), run)
    assert not state[0].any() and not state[2].any()
    for r, slot in enumerate((3, 1)):
        torch.testing.assert_close(state[slot, kept_at:].cpu(), rows[r][-1], rtol=0, atol=0)
        if dtype == torch.float32:
            _close(got[r], plain.time_mixing(rows[r], w, dict(heads=heads, dim=dim), eps), dtype, f32=1e-4)
        given = torch.cat([x[:, q[r]:q[r + 1]] for q, x, _ in inputs], dim=1)
        logits = torch.cat([x[q[r]:q[r + 1]] for q, _, x in inputs])
        keep = torch.exp(-torch.exp(logits + w["w0"]))
        raw = plain.mixed_states(*(x.reshape(-1, heads, dim) for x in (*given[:3], keep)), w["u"])
        _close(got[r], plain.unit_rms(raw, eps).reshape(-1, wide) * w["norm"] * plain.silu(given[3]), dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,dim,vdim,cap,length", [(2, 16, 12, 8.0, 110), (1, 64, 64, 15.0, 1500), (3, 24, 40, 2.0, 300), (4, 128, 32, 12.0, 110),
                                                       (2, 3, 1, 5.0, 110), (1, 256, 256, 10.0, 70), (2, 260, 7, 6.0, 70)])
def test_matrix_memory_alone(hip, dtype, heads, dim, vdim, cap, length):
    """Gates from shut to wide open under the running maximum (which starts at zero and must outlast steps, tiles and the scan's
    blocks of 1,024 tokens), the read-out's denominator with its floor, the norm per head and the gate.  Stretches of small
    input gates follow tokens with a large one: the maximum then falls by the forget gates alone, and the floor decides."""
    torch.manual_seed(dim + vdim)
    lengths, eps, qk, vs = (length, 40), 1e-6, heads * dim, heads * vdim
    width = 2 * (qk + vs + heads)
    rows = [torch.randn(n, width) for n in lengths]
    for x, n in zip(rows, lengths):
        gates = x[:, 2 * (qk + vs):]
        gates[:, :heads] = gates[:, :heads] * 2 - 6.0
        gates[torch.arange(0, n, 29), :heads] = torch.linspace(3.0, 20.0, len(range(0, n, 29)))[:, None]
        gates[:, heads:] += 1.0
    rows = [r.to(dtype).float() for r in rows]
    i_bias, f_bias = torch.linspace(-1.0, 1.0, heads), torch.linspace(0.0, 4.0, heads)
    weight = 1 + 0.3 * torch.randn(vs)
    top_at = heads * dim * (vdim + 1)
    state = torch.zeros(4, (top_at + heads + 3) // 4 * 4, device=DEVICE)

    def run(ctx, cut):
        x = cut([r.to(dtype) for r in rows])
        out = torch.empty(ctx.num_tokens, vs, dtype=dtype, device=DEVICE)
        hip.matrix_memory(x, i_bias.to(DEVICE), f_bias.to(DEVICE), cap, 1e-6, weight.to(DEVICE), eps, heads, dim, vdim, state, top_at, ctx, out)
        return out

    at = [0, qk, 2 * qk, 2 * qk + vs, 2 * (qk + vs), 2 * (qk + vs) + heads, width]
    w = {name: _eye(lo, hi, width) for name, lo, hi in zip(("q", "k", "v", "g", "i", "f"), at, at[1:])}
    w.update({"i.b": i_bias, "f.b": f_bias, "norm": weight, "o": torch.eye(vs)})
    want = [plain.matrix_memory(r, w, dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap), eps) for r in rows]
    whole = _run_steps(lengths, [((0, 0), lengths)], run)
    assert not state[0].any() and not state[2].any() and state[3].any() and state[1].any()
    state.zero_()
    pieces = _run_steps(lengths, THREE_STEPS(*lengths), run)
    for r in range(2):
        for got in (whole[r], pieces[r]):
            _close(got, want[r], dtype, f32=2e-4)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_token_wise_kernels(hip, dtype):
    """Two branches normed and added in the next norm's kernel; scaled embeddings with position vectors (also of a token that the
    sampler left in the request's slot, and beyond the known positions); the softcap; the clamped feed-forward activation."""
    torch.manual_seed(3)
    relative = 1e-5 if dtype == torch.float32 else 8e-3
    for tokens, hidden in ((5, 96), (3, 40), (2, 4100), (1, 10), (4, 2048)):
        stream = torch.randn(tokens, hidden, device=DEVICE)
        a, b = ((torch.randn(tokens, hidden, device=DEVICE) * s).to(dtype) for s in (0.3, 5.0))
        wa, wb, weight = (1 + 0.2 * torch.randn(hidden, device=DEVICE) for _ in range(3))
        out = torch.empty(tokens, hidden, dtype=dtype, device=DEVICE)
        want_stream = stream + 0.5 * (plain.rms_norm(a.float(), wa, 1e-4) + plain.rms_norm(b.float(), wb, 1e-4))
        alone = stream.clone()
        hip.norm_add_norm(stream, a, wa, 1e-4, weight, 1e-5, out, delta_scale=0.5, delta2=b, post_weight2=wb)
        torch.testing.assert_close(stream, want_stream, rtol=1e-5, atol=1e-5)
        torch.testing.assert_close(out.float(), plain.rms_norm(want_stream, weight, 1e-5).to(dtype).float(), rtol=relative, atol=1e-5)
        hip.norm_add_norm(alone, a, wa, 1e-4, None, 0.0, None, delta_scale=0.5, delta2=b, post_weight2=wb)
        torch.testing.assert_close(alone, stream, rtol=0, atol=0)
    for hidden in (72, 7):
        table, places = (torch.randn(rows, hidden, device=DEVICE).to(dtype) for rows in (50, 10))
        ctx = _ctx((0, 9, 3), (2, 1, 1))
        ctx.slot_words = torch.zeros(3, 8, dtype=torch.int32, device=DEVICE)
        ctx.slot_words[1, 1] = 17
        ids = torch.tensor([3, 49, -1, 0], dtype=torch.int32, device=DEVICE)
        got = torch.zeros(4, hidden, device=DEVICE)
        hip.embed_scaled(ids, table, 2.5, places, got, ctx)
        want = table[[3, 49, 17, 0]].float() * 2.5 + places[[0, 1, 9, 3]].float()
        torch.testing.assert_close(got, want, rtol=1e-6, atol=1e-6)
        hip.embed_scaled(ids, table, 2.5, places[:9].contiguous(), got, ctx)
        assert torch.isnan(got[2]).all() and not torch.isnan(got[[0, 1, 3]]).any()
        hip.embed_scaled(ids, table, 0.5, None, got, ctx)
        torch.testing.assert_close(got, table[[3, 49, 17, 0]].float() * 0.5, rtol=0, atol=0)
    for shape in ((3, 50), (1, 7), (2, 4096)):
        logits = torch.randn(*shape, device=DEVICE) * 20
        want = plain.soft_cap(logits, 6.0)
        hip.softcap(logits, 6.0)
        torch.testing.assert_close(logits, want, rtol=1e-5, atol=1e-6)
    for tokens, inter in ((5, 24), (3, 33), (1, 1028)):
        gate_up = (torch.randn(tokens, 2 * inter, device=DEVICE) * 2).to(dtype)
        out = torch.empty(tokens, inter, dtype=dtype, device=DEVICE)
        hip.gated_activation(gate_up, out, "clamped", limit=1.3, slope=1.702, shift=1.0)
        want = plain.limited_activation(gate_up[:, :inter].float(), gate_up[:, inter:].float(), 1.3)
        torch.testing.assert_close(out.float(), want.to(dtype).float(), rtol=relative, atol=1e-5)


def test_what_the_kernels_do_not_take_is_refused_on_the_host(hip):
    from ampere_kv_engine_amd.kernels.hip import KernelError
    rows = torch.zeros(2, 8, device=DEVICE)
    with pytest.raises(KernelError, match="both are normed or neither"):
        hip.norm_add_norm(rows, rows, torch.ones(8, device=DEVICE), 1e-5, None, 0.0, None, delta2=rows)
    with pytest.raises(KernelError, match="second branch"):
        hip.norm_add_norm(rows, rows, torch.ones(8, device=DEVICE), 1e-5, None, 0.0, None, post_weight2=torch.ones(8, device=DEVICE))
    with pytest.raises(KernelError, match="2048"):
        hip.check_state_sizes(2, 4096, 8)
    with pytest.raises(KernelError, match="at least"):
        hip.token_shift(rows, torch.zeros(5, 8, device=DEVICE), torch.zeros(1, 4, device=DEVICE), 0, _ctx((0,), (2,)), torch.zeros(5, 2, 8, device=DEVICE))
    with pytest.raises(KernelError, match="positive"):
        hip.softcap(rows, 0.0)
