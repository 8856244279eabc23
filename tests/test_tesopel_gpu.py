"""Tesopel on the GPU: each mechanism's kernels alone against the plain implementation's function of that mechanism,
then the engine (a cache that several layers read, state slots, batches, portions, captured graphs, the entry point)
against the plain forward pass, in float32 and bfloat16."""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

from helpers import max_live_tokens, replay_and_collect, trace_mixed, trace_portions, trace_tail, trace_whole
from plain import tesopel_plain as plain
from tesopel_helpers import (CONFIGS, compare_rows, compare_with_rounding, middling_config, plain_logits, random_config,
                             reach_config, read_folder, requests_for, rounding_noise, write_folder)
from wllm_amd.engine import LLM, ModelRunner
from wllm_amd.engine.replay import TraceReplayer, pages_for_max_tokens
from wllm_amd.kernels import ops
from wllm_amd.parts import load_model

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LENGTHS = {"mixed": [70, 45, 150, 33, 58], "odd": [40, 66, 25, 151], "sharp": [120, 137, 64, 50]}
FAMILIES = {"whole": trace_whole, "tail": trace_tail, "portions": trace_portions, "mixed": trace_mixed}
# a row's distance from the exact row, as a share of the row's own size or as a multiple of what rounding alone does to
# that row in the plain implementation (`rounding_noise`), whichever is larger: float32 sums in another order; bfloat16
# activations through some ten roundings a layer, and now and then a key or a denominator that the engine's rounding
# moves where the plain implementation's does not
BOUND = {torch.float32: dict(relative=1e-4, times=6.0), torch.bfloat16: dict(relative=0.04, outliers=0.1)}
SHARP_BOUND = {torch.float32: dict(relative=6e-4, times=6.0), torch.bfloat16: dict(relative=0.2, outliers=0.15)}


def check_rows(got, folder, requests, exact, dtype, sharp=False):
    return compare_with_rounding(got, exact, rounding_noise(folder, requests, dtype, exact), **(SHARP_BOUND if sharp else BOUND)[dtype])


def close(got, ref, dtype, what="", scale=1.0):
    atol, rtol = (3e-5 * scale, 3e-5) if dtype == torch.float32 else (1.5e-2 * scale, 1e-2)
    got, ref = got.double().cpu(), ref.double().cpu()
    assert torch.isfinite(got).all(), f"{what}: not finite"
    err = ((got - ref).abs() / (atol + rtol * ref.abs())).max().item()
    assert err <= 1.0, f"{what}: worst error {err:.2f} x tolerance, max abs diff {(got - ref).abs().max().item():.3e}"


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("tesopel_gpu")
    return {name: write_folder(name, str(root / name)) for name in CONFIGS}


def replay(folder, trace, dtype, page_size, max_requests=4, pages=None):
    model = load_model(folder, dtype, DEV)
    pages = pages or pages_for_max_tokens(max_live_tokens(trace), page_size)
    runner = ModelRunner.create(model, num_pages=pages, page_size=page_size, max_requests=max_requests, poison_freed_pages=True)
    with torch.inference_mode():
        got = replay_and_collect(TraceReplayer(runner), trace)
    runner.cache.check()
    assert not runner.cache.requests
    return got


def _pieces(total, sizes):
    out, at, i = [], 0, 0
    while at < total:
        n = min(sizes[i % len(sizes)], total - at)
        out.append((at, at + n))
        at, i = at + n, i + 1
    return out


# ---- mechanisms alone ---------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,ff,limit,slope,shift", [
    (1, 64, 48, 1.5, 1.702, 1.0), (7, 128, 50, 0.8, 1.702, 1.0), (20, 64, 80, 2.0, 1.0, 0.0), (40, 512, 96, 1.0, 2.5, -0.5),
    (64, 256, 16, 7.0, 1.702, 1.0), (100, 128, 130, 0.6, 1.702, 1.0), (256, 64, 64, 1.5, 0.7, 1.0), (300, 96, 72, 1.1, 1.702, 1.0),
    (5, 40, 30, 1.3, 1.702, 1.0), (513, 512, 512, 1.5, 1.702, 2.0)])
def test_a_gated_product_held_under_a_limit(dtype, rows, width, ff, limit, slope, shift):
    """Every kernel that makes the gate's step: few rows (tile-major weights or not), tiles, the two products and then
    the step alone; values on either side of both limits."""
    g = torch.Generator().manual_seed(rows + ff)
    x = torch.randn(rows, width, generator=g).to(dtype)
    w = (torch.randn(2 * ff, width, generator=g) * 1.5 * width ** -0.5).to(dtype)
    gate = ops.ClampedSwish(limit, slope, shift)
    z, u = x.double() @ w[:ff].double().T, x.double() @ w[ff:].double().T
    assert (z > limit).any() and (u > limit).any() or limit > 5
    assert (u < -limit).any() or limit > 5
    zc = torch.clamp(z, max=limit)
    want = zc * torch.sigmoid(slope * zc) * (torch.clamp(u, -limit, limit) + shift)
    if slope == 1.702 and shift == 1.0:
        assert torch.equal(want, plain.clamped_swish_gate(z, u, limit))
    xd, wd = x.to(DEV), w.to(DEV)
    tiles = ops.tile_weight(wd, 2) if width % 64 == 0 else None
    for t in {None, tiles}:
        out = torch.full((rows, ff), float("nan"), dtype=dtype, device=DEV)
        scratch = torch.zeros(rows, 2 * ff, dtype=dtype, device=DEV)
        ops.gated_linear(xd, wd, out, gate, scratch, t)
        close(out, want, dtype, "the gated product", scale=2.0)
    alone = torch.full((rows, ff), float("nan"), dtype=dtype, device=DEV)
    both = torch.cat([z, u], 1).to(dtype)
    ops.gated_activation(both.to(DEV), alone, gate)
    zb, ub = both[:, :ff].double(), both[:, ff:].double()
    zc = torch.clamp(zb, max=limit)
    close(alone, zc * torch.sigmoid(slope * zc) * (torch.clamp(ub, -limit, limit) + shift), dtype, "the step alone")


def test_the_limit_with_the_norm_on_load():
    g = torch.Generator().manual_seed(9)
    rows, width, ff = 9, 512, 96
    x = torch.randn(rows, width, generator=g) * 3
    norm_w = 1.0 + 0.3 * torch.randn(width, generator=g)
    w = (torch.randn(2 * ff, width, generator=g) * width ** -0.5).to(torch.bfloat16)
    sumsq = (x * x).view(rows, -1, 16).sum(-1)
    h = plain.rms_norm(x.double(), norm_w.double(), 1e-6).to(torch.bfloat16).double()
    want = plain.clamped_swish_gate(h @ w[:ff].double().T, h @ w[ff:].double().T, 0.9)
    norm = ops.NormOnLoad(x.to(DEV), sumsq.to(DEV), norm_w.to(DEV), 1e-6, 0.0, torch.bfloat16)
    out = torch.zeros(rows, ff, dtype=torch.bfloat16, device=DEV)
    ops.gated_linear(norm, w.to(DEV), out, ops.ClampedSwish(0.9, 1.702, 1.0), None, ops.tile_weight(w.to(DEV), 2))
    close(out, want, torch.bfloat16, scale=2.0)


@pytest.mark.parametrize("n,heads,outs,keys", [(1, 3, 96, 32), (16, 5, 40, 24), (17, 2, 256, 128), (33, 3, 30, 8), (64, 16, 256, 128),
                                               (300, 4, 128, 256), (1100, 16, 250, 40), (1030, 16, 256, 64), (129, 7, 18, 56)])
def test_products_head_by_head_on_the_matrix_cores(n, heads, outs, keys):
    """bfloat16 bands whose rows begin at multiples of 16 bytes; every row has the bits it has alone or among any others,
    and nothing beside the band is written."""
    g = torch.Generator().manual_seed(n + keys)
    wide = torch.randn(n, heads * keys + 16, generator=g).to(torch.bfloat16)
    wide[:, :8], wide[:, heads * keys + 8:] = float("nan"), float("nan")
    w = (torch.randn(heads, outs, keys, generator=g) * keys ** -0.5).to(torch.bfloat16)
    x, wd = wide.to(DEV)[:, 8:heads * keys + 8], w.to(DEV)

    def made(lo, hi):
        y = torch.full((hi - lo, heads * outs + 8), 3.0, dtype=torch.bfloat16, device=DEV)
        ops.head_linear(x[lo:hi], wd, y[:, :heads * outs])
        assert (y[:, heads * outs:] == 3.0).all()
        return y[:, :heads * outs]

    got = made(0, n)
    want = torch.stack([wide[:, 8 + h * keys:8 + (h + 1) * keys].double() @ w[h].double().T for h in range(heads)], 1)
    close(got, want.reshape(n, -1), torch.bfloat16)
    for lo, hi in ((0, 1), (n // 2, min(n, n // 2 + 5)), (max(0, n - 20), n), (0, min(n, 50))):
        assert torch.equal(made(lo, hi), got[lo:hi])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden,stack", [(64, 0), (300, 3), (2048, 0), (48, 2), (3072, 4)])
def test_a_norm_behind_a_sublayer_and_the_stream_as_the_next_one_reads_it(dtype, hidden, stack):
    g = torch.Generator().manual_seed(hidden)
    n, eps = 9, 1e-5
    x = torch.randn(n, hidden, generator=g) * 5
    delta = torch.randn(stack, n, hidden, generator=g) if stack else (torch.randn(n, hidden, generator=g) * 0.01).to(dtype)
    w = 1.0 + 0.3 * torch.randn(hidden, generator=g)
    want = x.double() + plain.rms_norm((delta.sum(0) if stack else delta).double(), w.double(), eps)
    xd = x.to(DEV)
    out = torch.zeros(n, hidden, dtype=dtype, device=DEV)
    ops.norm_add(xd, delta=delta.to(DEV), delta_norm=ops.NormRecipe("rms", w.to(DEV), eps, 0.0), out=out)
    close(xd, want, torch.float32, "the stream", scale=4.0)
    assert torch.equal(out, xd.to(dtype))


def _attention_problem(dtype, nh, d, ps, segs, seed):
    g = torch.Generator().manual_seed(seed)
    n = sum(q for q, _ in segs)
    pages = sum(-(-c // ps) for _, c in segs) + 3
    order = torch.randperm(pages, generator=g).tolist()
    bt = torch.zeros(len(segs), max(-(-c // ps) for _, c in segs), dtype=torch.int32)
    for s, (_, c) in enumerate(segs):
        for p in range(-(-c // ps)):
            bt[s, p] = order.pop()
    cache = torch.randn(pages, 2, 1, ps * d, generator=g).to(dtype)
    rows = torch.randn(n, nh * d, generator=g).to(dtype)
    q_len = torch.tensor([q for q, _ in segs], dtype=torch.int32)
    ctx = torch.tensor([c for _, c in segs], dtype=torch.int32)
    q_start = (torch.cumsum(q_len, 0) - q_len).to(torch.int32)
    tok_seg = torch.repeat_interleave(torch.arange(len(segs), dtype=torch.int32), q_len.long())
    return rows, cache, bt, tok_seg, q_start, q_len, ctx


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nh,d,ps,window,segs", [
    (4, 96, 16, 64, [(1, 700), (70, 70), (1, 64), (1, 65), (5, 200), (1, 66)]),
    (16, 256, 16, 200, [(1, 641), (130, 300), (1, 1), (201, 201)]),
    (3, 20, 8, 24, [(1, 350), (33, 40), (1, 24), (1, 25), (2, 26)]),
    (6, 64, 16, 300, [(1, 900), (320, 320), (64, 1000), (16, 301)]),
    (5, 36, 4, 7, [(1, 129), (1, 7), (1, 8), (200, 520)]),
    (20, 128, 16, 33, [(1, 48), (1, 33), (40, 80), (17, 33)]),
    (2, 32, 16, 1, [(1, 17), (30, 30), (3, 19)]),
])
def test_keys_just_inside_and_just_outside_a_window_in_every_attention_kernel(dtype, nh, d, ps, window, segs):
    """One shared key/value head (the cached vectors).  In every segment whose last query's window does not reach the
    start, the oldest key it sees would take most of its first head's weight, and the next older one all of it, if it
    were seen; pages out of every query's reach hold NaN, and the block table names page 0 for them, as the engine does
    for pages that were given back."""
    rows, cache, bt, tok_seg, q_start, q_len, ctx = _attention_problem(dtype, nh, d, ps, segs, seed=d + ps)
    scale = 1.0 / math.sqrt(d)
    kview, vview = cache[:, 0, 0].view(-1, ps, d), cache[:, 1, 0].view(-1, d, ps)
    edges = []
    for s, (ql, cl) in enumerate(segs):
        last, oldest = int(q_start[s]) + ql - 1, cl - window
        if oldest < 1:
            continue
        q0 = rows[last, :d].float()
        for j, score in ((oldest, 30.0), (oldest - 1, 60.0)):
            kview[int(bt[s, j // ps]), j % ps] = (q0 * score / scale / q0.norm() ** 2).to(dtype)
        edges.append((s, last, oldest))
    assert edges
    plain_k, plain_v, plain_bt = kview.clone(), vview.clone(), bt.clone()
    for s, (ql, cl) in enumerate(segs):
        for page in range(max(0, cl - ql - window + 1) // ps):
            kview[int(bt[s, page])] = float("nan")
            vview[int(bt[s, page])] = float("nan")
            bt[s, page] = 0
    out = torch.zeros(rows.shape[0], nh * d, dtype=dtype, device=DEV)
    args = [t.to(DEV) for t in (rows, cache, bt, tok_seg, q_start, q_len, ctx)] + [out]
    plan = ops.plan_paged_attention(q_len.numpy(), ctx.numpy(), num_heads=nh, num_kv_heads=1, head_dim=d, page_size=ps,
                                    window=window, dtype=dtype, device=torch.device(DEV))
    ops.paged_attention(*args, num_heads=nh, num_kv_heads=1, head_dim=d, page_size=ps, scale=scale, window=window,
                        max_q_len=int(q_len.max()), max_ctx_len=int(ctx.max()), exact_weights=True, plan=plan)
    torch.cuda.synchronize()
    weight_of = {}
    for s, (ql, cl) in enumerate(segs):
        ids = plain_bt[s, :-(-cl // ps)].long()
        keys, values = plain_k.double()[ids].reshape(-1, d)[:cl], plain_v.double()[ids].transpose(1, 2).reshape(-1, d)[:cl]
        q = torch.zeros(cl, nh, d, dtype=torch.float64)
        q[cl - ql:] = rows[int(q_start[s]):int(q_start[s]) + ql].double().view(ql, nh, d)
        weights = plain.masked_softmax(torch.einsum("ihd,jd->hij", q, keys) * scale, plain.window_mask(cl, window))
        want = torch.einsum("hij,jd->ihd", weights, values)[cl - ql:].reshape(ql, nh * d)
        close(out[int(q_start[s]):int(q_start[s]) + ql], want, dtype, f"segment {s} ({ql} of {cl})")
        weight_of[s] = weights[0, cl - 1]
    for s, last, oldest in edges:
        assert weight_of[s][oldest] > 0.9 and weight_of[s][oldest - 1] == 0.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,d,dv,cap", [(2, 16, 32, 8.0), (3, 10, 12, 3.0), (1, 130, 5, 15.0), (4, 64, 72, 1.0), (1, 256, 40, 15.0),
                                            (5, 4, 130, 20.0)])
def test_the_mlstm_whole_and_token_by_token(dtype, heads, d, dv, cap):
    """The gates, the recurrence with its normaliser and running maximum, and what follows, over a prompt and over the
    same prompt in pieces down to single tokens, through a state row that lies beside rows that must not change."""
    g = torch.Generator().manual_seed(heads * d + dv)
    T, eps, qw, vw = 90, 1e-5, heads * d, heads * dv
    width = 2 * qw + 2 * vw + 2 * heads
    eye = torch.eye(width, dtype=torch.float64)
    at = [0, qw, 2 * qw, 2 * qw + vw, 2 * qw + 2 * vw, 2 * qw + 2 * vw + heads, width]
    w = {"m." + n: eye[at[i]:at[i + 1]] for i, n in enumerate(("q", "k", "v", "g", "i", "f"))}
    w |= {"m.o": torch.eye(vw, dtype=torch.float64), "m.norm": 1.0 + 0.3 * torch.randn(vw, generator=g).double(),
          "m.i.b": torch.randn(heads, generator=g).double(), "m.f.b": 2.0 + torch.randn(heads, generator=g).double()}
    row = torch.randn(T, width, generator=g)
    row[:, at[4]:] *= 4.0                       # gates of some units either way, beyond the smaller caps
    row = row.to(dtype)
    c = {"heads": heads, "dim": d, "vdim": dv, "gate_cap": cap}
    want = plain.mlstm(row.double(), w, "m.", c, eps)
    # rows whose n . q nearly cancels amplify the float32 rounding of the sums; how much, the plain mixer in float32 says
    noise = (plain.mlstm(row.float(), {k: v.float() for k, v in w.items()}, "m.", c, eps).double() - want).abs().amax(-1)
    memory, slots_total = heads * d * dv, 5
    f32 = lambda name: w[name].float().to(DEV)
    for sizes in ([1000], [16, 5, 2, 1, 33], [1]):
        state = torch.full((slots_total, memory + qw + heads + 3), 9.0, device=DEV)
        state[2] = 0.0
        outs = []
        for lo, hi in _pieces(T, sizes):
            n = hi - lo
            r = row[lo:hi].to(DEV)
            one = lambda v: torch.tensor([v], dtype=torch.int32, device=DEV)
            seg = (one(0), one(n), one(2))
            qk = torch.zeros(2, n, qw, device=DEV)
            ops.memory_inputs(r, torch.arange(lo, hi, dtype=torch.int32, device=DEV), None, qk, heads=heads, head_dim=d, q_scale=d ** -0.5)
            steps, nq = torch.zeros(3, n, heads, device=DEV), torch.zeros(n, heads, device=DEV)
            ops.memory_gates(r[:, at[4]:], f32("m.i.b"), f32("m.f.b"), state, memory + qw, *seg, steps, heads=heads, cap=cap)
            y = torch.zeros(n, vw, device=DEV)
            ops.memory_scan(qk, r[:, at[2]:at[3]], steps, None, state, *seg, y, heads=heads, head_dim=d, value_dim=dv, nq=nq, n_offset=memory)
            out = torch.zeros(n, vw, dtype=dtype, device=DEV)
            ops.head_norm_gate(y, r[:, at[3]:at[4]], f32("m.norm"), out, heads=heads, eps=eps, activation="sigmoid", nq=nq, floor=steps[2],
                               den_eps=1e-6)
            outs.append(out.cpu())
        got = torch.cat(outs)
        for t in range(T):
            close(got[t], want[t], dtype, f"token {t}, pieces {sizes}", scale=4.0 + 8.0 * float(noise[t]) / 3e-5)
        assert (state[[0, 1, 3, 4]] == 9.0).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,d,dv,dims,base,start", [(2, 16, 32, 16, 1e4, 0), (3, 10, 12, 6, 50.0, 0), (1, 130, 5, 2, 1e6, 0),
                                                        (4, 64, 72, 32, 1e4, 0), (1, 256, 40, 256, 1e5, 0)])
def test_retention_whole_and_token_by_token(dtype, heads, d, dv, dims, base, start):
    g = torch.Generator().manual_seed(heads * d + dv)
    T, eps, qw, vw = 90, 1e-5, heads * d, heads * dv
    decay = [1.0, 0.0, 0.97, 0.5][:heads] if heads > 1 else [0.99]
    width = 2 * qw + 2 * vw
    eye = torch.eye(width, dtype=torch.float64)
    at = [0, qw, 2 * qw, 2 * qw + vw, width]
    w = {"m." + n: eye[at[i]:at[i + 1]] for i, n in enumerate(("q", "k", "v", "g"))} | {"m.o": torch.eye(vw, dtype=torch.float64)}
    row = torch.randn(T, width, generator=g).to(dtype)
    want = plain.retention(row.double(), w, "m.", {"heads": heads, "dim": d, "vdim": dv, "decay": decay, "rot": {"dims": dims, "base": base}}, eps)
    inv_freq = (base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)).float().to(DEV)
    memory = heads * d * dv
    for sizes in ([1000], [16, 5, 2, 1, 33], [1]):
        state = torch.full((5, memory + 3), 9.0, device=DEV)
        state[2] = 0.0
        outs = []
        for lo, hi in _pieces(T, sizes):
            n = hi - lo
            r = row[lo:hi].to(DEV)
            one = lambda v: torch.tensor([v], dtype=torch.int32, device=DEV)
            qk, y = torch.zeros(2, n, qw, device=DEV), torch.zeros(n, vw, device=DEV)
            ops.memory_inputs(r, torch.arange(lo, hi, dtype=torch.int32, device=DEV), inv_freq, qk, heads=heads, head_dim=d, k_scale=d ** -0.5)
            ops.memory_scan(qk, r[:, at[2]:at[3]], None, torch.tensor(decay, device=DEV), state, one(0), one(n), one(2), y, heads=heads,
                            head_dim=d, value_dim=dv)
            out = torch.zeros(n, vw, dtype=dtype, device=DEV)
            ops.head_norm_gate(y, r[:, at[3]:], None, out, heads=heads, eps=eps, activation="silu")
            outs.append(out.cpu())
        close(torch.cat(outs), want, dtype, f"pieces {sizes}", scale=20.0 if dtype == torch.float32 else 2.0)
        assert (state[[0, 1, 3, 4]] == 9.0).all()


# ---- the engine -----------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("family", list(FAMILIES))
@pytest.mark.parametrize("name", list(CONFIGS))
def test_replay_matches_plain(folders, name, family, dtype):
    requests = requests_for(name, LENGTHS[name])
    exact = plain_logits(folders[name], requests, torch.float64)
    got = replay(folders[name], FAMILIES[family](requests), dtype, CONFIGS[name]["page_size"])
    check_rows(got, folders[name], requests, exact, dtype, sharp=name == "sharp")


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(tmp_path, seed):
    c = random_config(200 + seed)
    folder = write_folder(c, str(tmp_path / "m"))
    requests = requests_for(c, [37, 18, 150, 64])
    exact = plain_logits(folder, requests, torch.float64)
    for dtype in DTYPES:
        for family in ("portions", "mixed"):
            check_rows(replay(folder, FAMILIES[family](requests), dtype, c["page_size"]), folder, requests, exact, dtype)


@pytest.mark.parametrize("seed", range(3))
def test_long_requests_at_middling_sizes(tmp_path, seed):
    """Widths of some hundred and requests of up to 700 tokens, whole (the library's products, the tiled kernels,
    blocks of 64 rows in the attention, recurrences carried over hundreds of tokens) and four at a time."""
    c = middling_config(300 + seed)
    folder = write_folder(c, str(tmp_path / "m"))
    requests = requests_for(c, [700, 129, 300, 65])
    exact = plain_logits(folder, requests, torch.float64)
    for dtype in DTYPES:
        for family in ("whole", "mixed"):
            trace = trace_whole(requests) if family == "whole" else trace_mixed(requests, seed=seed, portion_sizes=(2, 64, 100, 128, 29))
            for step in trace:      # every tenth row is enough of a long request
                for e in step["entries"]:
                    e["want"] = [w for w in e["want"] if w % 10 == 0 or len(e["tokens"]) == 1]
            check_rows(replay(folder, trace, dtype, 16), folder, requests, exact, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_with_sharp_attention(folders, dtype):
    """400 tokens of which 300 are decoded one by one, in a pool that holds the request whole: single keys decide, both
    windows and many pages pass, and the states go through every step."""
    requests = requests_for("sharp", [400])
    exact = plain_logits(folders["sharp"], requests, torch.float64)
    got = replay(folders["sharp"], trace_tail(requests, tail=300), dtype, 16, max_requests=2, pages=26)
    check_rows(got, folders["sharp"], requests, exact, dtype, sharp=True)


def test_a_long_request_in_pages_for_its_window_alone(folders):
    """350 tokens decoded in a pool of 6 pages of 16: the wider of the two windows over the vectors is 64, so a page
    that went back too late would end the run and one that went back too early reads as NaN."""
    requests = requests_for("sharp", [370])
    exact = plain_logits(folders["sharp"], requests, torch.float64)
    got = replay(folders["sharp"], trace_tail(requests, tail=350), "float32", 16, max_requests=1, pages=6)
    check_rows(got, folders["sharp"], requests, exact, torch.float32, sharp=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("windows,page_size,prompt", [((33, 50), 16, 60), ((48, 16), 16, 20), ((7,), 4, 150), ((100, 64), 8, 110)])
def test_a_logit_depends_on_the_tokens_in_the_window_and_on_no_other(tmp_path, dtype, windows, page_size, prompt):
    """Two requests that differ in one token, prompt and then decoding: the rows differ from that token to the widest
    window's edge, to the token, whether the edge falls into the prompt or among decoded tokens, and agree elsewhere."""
    c = reach_config(windows, page_size)
    folder = write_folder(c, str(tmp_path / "m"))
    total, p, reach = 160, 13, max(windows)
    toks = requests_for(c, [total])["q0"]
    other = list(toks)
    other[p] = (toks[p] + 31) % c["config"]["vocab"]
    rows = []
    for t in (toks, other):
        got = replay(folder, trace_tail({"q": t}, tail=total - prompt), dtype, page_size)
        rows.append(torch.stack([got[("q", i)] for i in range(total)]))
    assert [i for i in range(total) if not torch.equal(rows[0][i], rows[1][i])] == list(range(p, p + reach))
    exact = plain_logits(folder, {"q": toks}, torch.float64)
    check_rows({("q", i): rows[0][i] for i in range(total)}, folder, {"q": toks}, exact, dtype)


def test_a_row_does_not_depend_on_the_batch_or_the_cut(folders):
    requests = requests_for("sharp", [90, 200])
    model = load_model(folders["sharp"], "float32", DEV)

    def run(trace):
        runner = ModelRunner.create(model, num_pages=40, page_size=16, max_requests=4)
        with torch.inference_mode():
            return replay_and_collect(TraceReplayer(runner), trace)

    one = {"q0": requests["q0"]}
    whole, cut, tail = run(trace_whole(one)), run(trace_portions(one)), run(trace_tail(one, tail=40))
    toks = requests["q0"]
    beside = [{"step": 0, "entries": [{"id": "q0", "tokens": toks[:50], "want": list(range(50))}], "end": []},
              {"step": 1, "entries": [{"id": "q1", "tokens": requests["q1"][:137], "want": []},
                                      {"id": "q0", "tokens": [toks[50]], "want": [0]}], "end": []},
              {"step": 2, "entries": [{"id": "q0", "tokens": toks[51:], "want": list(range(39))},
                                      {"id": "q1", "tokens": requests["q1"][137:], "want": []}], "end": ["q0", "q1"]}]
    mixed = run(beside)
    for key, ref in whole.items():
        for got in (cut, tail, mixed):
            assert (got[key] - ref).abs().max().item() <= 3e-4 * max(1.0, ref.abs().max().item()), key


@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_entry_point(folders, graphs):
    """`LLM.generate` (scheduler, chunked prefill, sampling kernels, captured graphs or not) against greedy decoding
    with the plain implementation, in float32 so that the tokens are comparable one by one."""
    name = "mixed"
    prompts = list(requests_for(name, [37, 5, 64, 18, 1]).values())
    new = 24
    llm = LLM(folders[name], dtype="float32", num_blocks=64, block_size=16, max_prefill_tokens_per_step=32, max_requests=4,
              hip_graphs=graphs)
    outs = llm.generate(prompts, max_new_tokens=new)
    raw, w = read_folder(folders[name])
    compared = 0
    for prompt, out in zip(prompts, outs):
        tokens = list(prompt)
        for step in range(new):
            logits = plain.forward(tokens, w, raw)[-1]
            top2 = logits.topk(2).values
            if (top2[0] - top2[1]).item() < 1e-3:       # a tie within rounding: the rest is not comparable
                break
            assert out.token_ids[step] == int(logits.argmax()), f"prompt of {len(prompt)}: token {step} differs"
            tokens.append(out.token_ids[step])
            compared += 1
        assert len(out.token_ids) == new
    assert compared > 2 * new
    if graphs:
        assert llm.runner.graph_steps > 0


def test_the_trace_runner_and_the_command_line(folders, tmp_path):
    name = "odd"
    toks = requests_for(name, [45])["q0"]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:30], "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[30:32], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[32:], "want": [12]}], "end": ["a"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders[name], "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [line for line in r.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
    exact = plain_logits(folders[name], {"a": toks}, torch.float64)
    first = torch.frombuffer(bytearray((out / "0.f32").read_bytes()), dtype=torch.float32).view(2, -1)
    last = torch.frombuffer(bytearray((out / "2.f32").read_bytes()), dtype=torch.float32).view(1, -1)
    assert not (out / "1.f32").exists()
    compare_rows({("a", 0): first[0], ("a", 29): first[1], ("a", 44): last[0]}, exact, relative=1e-3)
    # the command line: a model folder of a named shape, then greedy generation from it
    made = tmp_path / "made"
    r = subprocess.run([sys.executable, "-m", "wllm_amd.cli", "random-model", "--out", str(made), "--config", "tesopel-tiny",
                        "--seed", "3", "--std", "0.3", "--norm-std", "0.6"], cwd=ROOT, capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    r = subprocess.run([sys.executable, "-m", "wllm_amd.cli", "generate", "--model", str(made), "--dtype", "float32",
                        "--prompt-ids", "5,17,3,200,41", "--max-new-tokens", "6"], cwd=ROOT, capture_output=True, text=True,
                       timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    line = json.loads([x for x in r.stdout.splitlines() if x.startswith("{")][-1])
    raw, w = read_folder(str(made))
    tokens = [5, 17, 3, 200, 41]
    for t in line["token_ids"]:
        logits = plain.forward(tokens, w, raw)[-1]
        if (logits.topk(2).values[0] - logits.topk(2).values[1]).item() < 1e-3:
            break
        assert t == int(logits.argmax())
        tokens.append(t)
    assert len(line["token_ids"]) == 6
