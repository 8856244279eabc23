"""Modasun on the GPU: each mechanism's kernels alone against the plain implementation's function of that mechanism,
then the engine (caches, state slots, batches, portions, runs that share weights, captured graphs, the entry point)
against the plain forward pass, in float32 and bfloat16."""
import json
import os
import subprocess
import sys

import pytest
import torch

from helpers import max_live_tokens, replay_and_collect, trace_mixed, trace_portions, trace_tail, trace_whole
from modasun_helpers import (CONFIGS, compare_rows, compare_with_rounding, middling_config, plain_logits, random_config, read_folder,
                             requests_for, rounding_noise, seek_config, seeking, seeks, to_bfloat16, write_folder)
from plain import modasun_plain as plain
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
# activations through some ten roundings a layer, and now and then an expert or a key that the engine's rounding moves
# where the plain implementation's does not
BOUND = {torch.float32: dict(relative=1e-4, times=6.0), torch.bfloat16: dict(relative=0.05, outliers=0.1)}
SHARP_BOUND = {torch.float32: dict(relative=6e-4, times=6.0), torch.bfloat16: dict(relative=0.2, outliers=0.15)}


def check_rows(got, folder, requests, exact, dtype, sharp=False):
    noise, bound = rounding_noise(folder, requests, dtype, exact), dict((SHARP_BOUND if sharp else BOUND)[dtype])
    if dtype == torch.bfloat16:
        # where the plain implementation's own rounding chooses other experts for many rows, the engine's may for as many others
        far = [float(noise[rid][pos]) > bound["relative"] * (exact[rid][pos] - exact[rid][pos].mean()).pow(2).mean().sqrt().item()
               for rid, pos in got]
        bound["outliers"] = max(bound["outliers"], 1.5 * sum(far) / len(far))
    return compare_with_rounding(got, exact, noise, **bound)


def close(got, ref, dtype, what="", scale=1.0):
    atol, rtol = (3e-5 * scale, 3e-5) if dtype == torch.float32 else (1.5e-2 * scale, 1e-2)
    got, ref = got.double().cpu(), ref.double().cpu()
    assert torch.isfinite(got).all(), f"{what}: not finite"
    err = ((got - ref).abs() / (atol + rtol * ref.abs())).max().item()
    assert err <= 1.0, f"{what}: worst error {err:.2f} x tolerance, max abs diff {(got - ref).abs().max().item():.3e}"


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("modasun_gpu")
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


def _i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


# ---- mechanisms alone ---------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden,stack,extra,alpha", [(64, 0, None, 2.0), (300, 3, 0, 0.5), (2048, 0, 2, 1.3), (48, 2, None, 1.0), (3072, 4, 0, 2.0),
                                                      (50, 1, 3, 0.0), (2048, 3, 0, 2.0), (6144, 0, 4, 1.1)])
@pytest.mark.parametrize("rows", [9, 300])
def test_the_norm_takes_the_sum_of_the_weighed_stream_and_the_result(dtype, hidden, stack, extra, alpha, rows):
    """A result in one term or two (the second a tensor or a stack, its rows weighed), what the next sublayer reads, and
    gathered rows under one more norm, which leave the stream alone."""
    g = torch.Generator().manual_seed(hidden + rows)
    eps = 1e-5
    x = torch.randn(rows, hidden, generator=g) * 3
    delta = torch.randn(stack, rows, hidden, generator=g) if stack else (torch.randn(rows, hidden, generator=g) * 0.5).to(dtype)
    w, wf = 0.3 * torch.randn(hidden, generator=g), 0.3 * torch.randn(hidden, generator=g)
    y = (delta.sum(0) if stack else delta).double()
    options = {}
    if extra is not None:
        e = torch.randn(extra, rows, hidden, generator=g) if extra else torch.randn(rows, hidden, generator=g).to(dtype)
        scale = torch.rand(rows, generator=g)
        y = y + scale.double()[:, None] * (e.sum(0) if extra else e).double()
        options = dict(extra=e.to(DEV), extra_scale=scale.to(DEV))
    want = plain.norm_of_the_sum(x.double(), y, alpha, w.double(), eps)
    options |= dict(delta=delta.to(DEV), x_scale=alpha, sum_norm=ops.NormRecipe("rms", w.to(DEV), eps, 1.0))
    gather = torch.tensor([rows - 1, 0, 5], dtype=torch.int32)
    xd = x.to(DEV)
    few = torch.zeros(3, hidden, dtype=dtype, device=DEV)
    ops.norm_add(xd, out=few, out_norm=ops.NormRecipe("rms", wf.to(DEV), eps, 1.0), rows=gather.to(DEV), **options)
    assert torch.equal(xd.cpu(), x)
    close(few, plain.offset_norm(want[gather.long()], wf.double(), eps), dtype, "gathered rows", scale=2.0)
    out = torch.zeros(rows, hidden, dtype=dtype, device=DEV)
    ops.norm_add(xd, out=out, **options)
    close(xd, want, torch.float32, "the stream", scale=2.0)
    assert torch.equal(out, xd.to(dtype))
    alone = x.to(DEV)
    ops.norm_add(alone, **options)
    assert torch.equal(alone, xd)
    if rows > 16:           # a row has the bits it has among few rows, up to the kernel's own division of the work
        some = x[:9].to(DEV)
        cut = {k: (v if not isinstance(v, torch.Tensor) else v[:, :9].contiguous() if v.dim() == 3 else v[:9].contiguous())
               for k, v in options.items()}
        ops.norm_add(some, **cut)
        close(some, xd[:9], torch.float32, "fewer rows")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nh,nkv,d,pad,coef,every", [(4, 2, 32, 0, 0.5, 9), (3, 3, 20, 2, 1.0, 1), (8, 1, 256, 0, -0.3, 128), (2, 2, 6, 2, 0.2, 1000),
                                                     (5, 1, 33, 3, 0.7, 16)])
def test_unit_heads_and_the_temperature(dtype, nh, nkv, d, pad, coef, every):
    """Query and key heads over their root mean square, the queries times the temperature at the places around its steps,
    keys and values in their pages, with the projection given whole or as partial sums."""
    g = torch.Generator().manual_seed(nh * d)
    ps, eps, dim = 16, 1e-5, d + pad
    pos = sorted({0, 1, every - 1, every, max(0, every - 2), 2 * every - 1, 2 * every - 2, 5 * every - 1, 5 * every, 70000})
    n, width = len(pos), (nh + 2 * nkv) * dim
    heads = torch.randn(n, nh + 2 * nkv, dim, generator=g)
    heads[..., d:] = 0.0
    for stack in (0, 3):
        if stack:
            parts = torch.randn(stack, n, nh + 2 * nkv, dim, generator=g)
            parts[..., d:] = 0.0
            src = parts.sum(0).double()
            rows, parts = torch.zeros(n, width, dtype=dtype, device=DEV), parts.view(stack, n, width).to(DEV)
        else:
            src, parts = heads.to(dtype).double(), None
            rows = heads.to(dtype).view(n, width).to(DEV)
        cache = torch.zeros(2 * n, 2, nkv, ps * dim, dtype=dtype, device=DEV)
        slots = torch.randperm(2 * n * ps, generator=g)[:n].to(torch.int32)
        ops.head_prepare(rows, None, _i32(pos), None, slots.to(DEV), cache, num_heads=nh, num_kv_heads=nkv, head_dim=dim,
                         page_size=ps, norm_eps=eps, norm_dim=d, parts=parts, q_temperature=(coef, every))
        temp = plain.query_temperature(torch.tensor(pos).double(), coef, every)
        q = plain.unit_rms(src[:, :nh, :d], eps) * temp[:, None, None]
        k = plain.unit_rms(src[:, nh:nh + nkv, :d], eps)
        got = rows.view(n, -1, dim)
        close(got[:, :nh, :d], q, dtype, "queries", scale=4.0)
        close(got[:, nh:nh + nkv, :d], k, dtype, "keys", scale=2.0)
        page, off = (slots // ps).long(), (slots % ps).long()
        assert torch.equal(cache[:, 0].view(-1, nkv, ps, dim)[page, :, off], got[:, nh:nh + nkv])
        assert torch.equal(cache[:, 1].view(-1, nkv, dim, ps)[page, :, :, off], got[:, nh + nkv:])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,ff", [(1, 64, 48), (7, 128, 50), (20, 64, 82), (40, 512, 96), (64, 256, 16), (100, 128, 130), (256, 64, 64),
                                           (300, 96, 72), (5, 40, 30), (513, 512, 512), (3, 64, 37), (130, 64, 33), (17, 96, 64), (9, 2048, 160)])
def test_a_product_and_its_squared_relu(dtype, rows, width, ff):
    """Every kernel that makes the step: few rows (tile-major weights or not), tiles, the product and then the step alone."""
    g = torch.Generator().manual_seed(rows + ff)
    x = torch.randn(rows, width, generator=g).to(dtype)
    w = (torch.randn(ff, width, generator=g) * width ** -0.5).to(dtype)
    z = x.double() @ w.double().T
    want = plain.squared_relu(z)
    xd, wd = x.to(DEV), w.to(DEV)
    paired = ops.tile_weight(wd, 2) if ff % 2 == 0 else None
    for tiles, pairs in {(None, None), (ops.tile_weight(wd), None), (None, paired)}:
        out = torch.full((rows, ff), float("nan"), dtype=dtype, device=DEV)
        ops.activated_linear(xd, wd, out, "squared_relu", tiles, pairs)
        close(out, want, dtype, "the product", scale=4.0)
    for name, ref in (("squared_relu", want), ("silu", plain.silu(z))):
        zd = z.to(dtype).to(DEV)
        ops.activation(zd, zd, name)
        close(zd, plain.squared_relu(z.to(dtype).double()) if name == "squared_relu" else plain.silu(z.to(dtype).double()), dtype, name)
    out = torch.zeros(rows, ff, dtype=dtype, device=DEV)
    xd[0, 0] = float("nan")
    ops.activated_linear(xd, wd, out, "squared_relu", None, paired)
    assert torch.isnan(out[0]).all() and torch.isfinite(out[1:]).all(), "what is not a number stays visible"


def _route(h, router, correction, top, groups, keep, gate=None):
    n = h.shape[0]
    ids = torch.zeros(n, top, dtype=torch.int32, device=DEV)
    wts, gates = torch.zeros(n, top, device=DEV), torch.zeros(n, device=DEV) if gate is not None else None
    rows = router if gate is None else torch.cat([router, gate])
    ops.moe_route(h.to(DEV), rows.float().to(DEV), ids, wts, groups=groups, keep=keep, scoring="sigmoid",
                  correction=correction.float().to(DEV), group_best=2, gates=gates)
    return ids.cpu(), wts.cpu(), gates.cpu() if gates is not None else None


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,count,top,groups,keep,spread", [(64, 8, 3, 4, 2, 0.5), (48, 5, 5, 1, 1, 2.0), (100, 12, 4, 3, 2, 1.0), (64, 6, 2, 6, 4, 1.0),
                                                                (128, 256, 8, 8, 4, 0.3), (64, 1, 1, 1, 1, 1.0), (96, 130, 6, 65, 10, 0.5), (64, 16, 4, 2, 1, 3.0)])
def test_the_router_with_its_correction(dtype, width, count, top, groups, keep, spread):
    """Choices by score + correction (of either sign) among the groups with the largest sums of two, weights by the scores
    alone, and the gate of the shared expert beside them."""
    g = torch.Generator().manual_seed(width + count)
    n = 70
    h = torch.randn(n, width, generator=g).to(dtype)
    router = (torch.randn(count, width, generator=g) * width ** -0.5).double()
    correction = (torch.randn(count, generator=g) * spread - 0.5).to(torch.float32).double()
    gate = (torch.randn(1, width, generator=g) * width ** -0.5).double()
    router, gate = router.float().double(), gate.float().double()
    ids, wts, gates = _route(h, router, correction, top, groups, keep, gate)
    z = h.double() @ router.T
    clear = 0
    for r in range(n):
        c = torch.sigmoid(z[r]) + correction
        chosen, weights = plain.choose_experts(z[r], correction, top, groups, keep)
        # rows where another choice lies within rounding are left out
        per = count // groups
        sums = torch.stack([c[i * per:(i + 1) * per].topk(min(2, per)).values.sum() for i in range(groups)]).sort(descending=True).values
        allowed = sorted(c[[e for e in range(count) if e // per in {x // per for x in chosen} or keep == groups]].tolist(), reverse=True)
        if (keep < groups and sums[keep - 1] - sums[keep] < 1e-4) or any(a - b < 1e-4 for a, b in zip(allowed[:top], allowed[1:top + 1])):
            continue
        clear += 1
        assert ids[r].tolist() == chosen, f"row {r}"
        close(wts[r], weights, torch.float32, f"row {r}")
    assert clear > 20 or (clear > 0 and count > 100)
    close(gates, torch.sigmoid(h.double() @ gate.T)[:, 0], torch.float32, "the gate")
    again, _, none = _route(h[:9], router, correction, top, groups, keep)
    assert torch.equal(again, ids[:9]) and none is None


def test_a_router_whose_scores_are_no_numbers_names_experts():
    h = torch.full((3, 64), float("nan"))
    ids, _, _ = _route(h, torch.randn(6, 64).double(), torch.zeros(6).double(), 2, 3, 2)
    assert ((ids >= 0) & (ids < 6)).all()


def _delta_weights(g, H, G, d, dv, taps, width, r1, r2):
    eye = lambda rows, at: torch.eye(width, dtype=torch.float64)[at:at + rows]
    at, w = 0, {}
    for name, rows in (("q", G * d), ("k", G * d), ("v", H * dv), ("b", H), ("a1", r1), ("g1", r2)):
        w["m." + name] = eye(rows, at)
        at += rows
    assert at == width
    for name, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
        w[f"m.{name}.conv"] = torch.randn(rows, taps, generator=g).double() * 0.6
    w |= {"m.a2": torch.randn(H * d, r1, generator=g).double() * r1 ** -0.5, "m.g2": torch.randn(H * dv, r2, generator=g).double(),
          "m.A_log": torch.randn(H, generator=g).double() * 0.7, "m.dt_bias": -3.0 + 2.5 * torch.randn(H * d, generator=g).double(),
          "m.norm": 1.0 + 0.3 * torch.randn(dv, generator=g).double(), "m.o": torch.eye(H * dv, dtype=torch.float64)}
    return w


DELTA_SIZES = [(4, 2, 16, 32, 4), (3, 1, 10, 6, 1), (1, 1, 130, 5, 7), (4, 2, 7, 9, 2), (2, 2, 64, 72, 3), (2, 1, 128, 128, 4), (1, 1, 256, 40, 2),
               (3, 3, 192, 12, 5), (5, 5, 4, 130, 2), (2, 2, 100, 33, 4)]


def _walk(chunked, qk, kq, f, beta, v, state, of, seg, y, sizes):
    """The recurrence over a step: token by token, or (the segments of `chunked` tokens and more) in chunks."""
    if chunked:
        n = v.shape[0]
        chunks = torch.full((ops.delta_chunk_size(n, seg[0].shape[0], sizes["heads"], sizes["head_dim"]),), float("nan"), device=DEV)
        ops.delta_chunk_scan(qk, f, beta, v, state, of, *seg, y, chunks, from_tokens=chunked, **sizes)
    ops.delta_scan(qk, kq, f, beta, v, state, *seg, y, shorter_than=chunked, **sizes)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunked", [None, 16, 40])
@pytest.mark.parametrize("H,G,d,dv,taps", DELTA_SIZES)
def test_the_delta_rule_whole_and_token_by_token(dtype, H, G, d, dv, taps, chunked):
    """The convolutions, unit vectors, decays, step sizes, the recurrence and the gated norm, over a prompt and over the
    same prompt in pieces down to single tokens, through a state row that lies beside rows that must not change."""
    g = torch.Generator().manual_seed(H * d + dv)
    T, eps, r1, r2 = 150, 1e-5, 6, 5
    width = 2 * G * d + H * dv + H + r1 + r2
    w = _delta_weights(g, H, G, d, dv, taps, width, r1, r2)
    row = torch.randn(T, width, generator=g).to(dtype)
    c = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "conv": taps}
    rounding = to_bfloat16 if dtype == torch.bfloat16 else plain.same
    want = plain.channel_delta(row.double(), w, "m.", c, eps, rounding)
    noise = (plain.channel_delta(row.float(), {k: v.float() for k, v in w.items()}, "m.", c, eps).double()
             - plain.channel_delta(row.double(), w, "m.", c, eps)).abs().amax(-1)
    qk_w, v_w, f_w, dp = G * d, H * dv, H * d, ops.delta_padded(d)
    channels, b_at = 2 * qk_w + v_w, 2 * qk_w + v_w
    z = rounding(row[:, b_at + H:b_at + H + r1].double() @ w["m.a2"].T).to(dtype).to(DEV)
    gate = rounding(row[:, b_at + H + r1:].double() @ w["m.g2"].T).to(dtype).to(DEV)
    conv = torch.cat([w[f"m.{n}.conv"] for n in "qkv"]).t().contiguous().float().to(DEV)
    rate, bias = torch.exp(w["m.A_log"]).float().to(DEV), w["m.dt_bias"].float().to(DEV)
    norm = w["m.norm"].repeat(H).float().to(DEV)
    memory = ops.delta_state_size(H, d, dv)
    total = -(-(memory + (taps - 1) * channels) // 4) * 4 + 4
    sizes = dict(heads=H, groups=G, head_dim=d, value_dim=dv)
    wide = torch.full((T, -(-width // 8) * 8 + 8), float("nan"), dtype=dtype)
    wide[:, 8:8 + width] = row
    wide = wide.to(DEV)
    for pieces in ([1000], [64, 33], [16, 5, 2, 1, 33, 17]) + (() if chunked else ([1],)):
        state = torch.full((5, total), 9.0, device=DEV)
        state[2] = 0.0
        outs = []
        for lo, hi in _pieces(T, pieces):
            n = hi - lo
            seg = (_i32([0]), _i32([n]), _i32([2]))
            r = wide[lo:hi, 8:8 + width]
            nan = lambda *s: torch.full(s, float("nan"), device=DEV)
            qk, kq, f, beta, y = nan(2, n, G * dp), nan(n, G), nan(n, H * dp), nan(n, H), nan(n, v_w)
            v = nan(n, v_w).to(dtype)
            ops.delta_inputs(r[:, :channels], z[lo:hi], r[:, b_at:b_at + H], conv, rate, bias, state, memory, _i32([0] * n), *seg, qk, kq,
                             v, f, beta, q_scale=d ** -0.5, unit_eps=1e-6, single_tokens=n == 1, **sizes)
            _walk(chunked, qk, kq, f, beta, v, state, _i32([0] * n), seg, y, sizes)
            out = torch.zeros(n, v_w, dtype=dtype, device=DEV)
            ops.head_norm_gate(y, gate[lo:hi], norm, out, heads=H, eps=eps, activation="sigmoid")
            outs.append(out.cpu())
        got = torch.cat(outs)
        for t in range(T):
            close(got[t], want[t], dtype, f"token {t}, pieces {pieces}", scale=3.0 + 8.0 * float(noise[t]) / 3e-5)
        assert (state[[0, 1, 3, 4]] == 9.0).all()


@pytest.mark.parametrize("chunked", [None, 16, 33])
@pytest.mark.parametrize("H,G,d,dv,taps", [(4, 2, 16, 32, 4), (2, 1, 128, 128, 4), (3, 1, 10, 6, 3), (1, 1, 256, 40, 2), (2, 2, 192, 17, 4)])
def test_a_batch_of_unequal_requests_against_each_alone(H, G, d, dv, taps, chunked):
    """Segments of a few tokens to some hundred side by side, in slots of any order, each with a memory and carried rows
    of its own: the results and what is left behind are those of each request alone."""
    g = torch.Generator().manual_seed(d)
    lengths, slots = [1, 2, 70, 1, 17, 200, 16, 33, 15, 16], [3, 0, 7, 1, 5, 2, 8, 6, 10, 9]
    n, channels = sum(lengths), 2 * G * d + H * dv
    dp, memory = ops.delta_padded(d), ops.delta_state_size(H, d, dv)
    total = -(-(memory + (taps - 1) * channels) // 4) * 4
    x, z, b = torch.randn(n, channels, generator=g).to(DEV), torch.randn(n, H * d, generator=g).to(DEV), torch.randn(n, H, generator=g).to(DEV)
    conv, rate = torch.randn(taps, channels, generator=g).to(DEV), (torch.rand(H, generator=g) + 0.1).to(DEV)
    bias = (-3.0 + torch.randn(H * d, generator=g)).to(DEV)
    state0 = torch.randn(11, total, generator=g).to(DEV) * 0.3
    sizes = dict(heads=H, groups=G, head_dim=d, value_dim=dv)

    def run(x, z, b, lengths, slots, state):
        n = x.shape[0]
        start = torch.cumsum(torch.tensor([0] + lengths), 0)[:-1].tolist()
        seg = (_i32(start), _i32(lengths), _i32(slots))
        of = torch.repeat_interleave(torch.arange(len(lengths), dtype=torch.int32), torch.tensor(lengths)).to(DEV)
        e = lambda *s: torch.zeros(s, device=DEV)
        qk, kq, f, beta, y, v = e(2, n, G * dp), e(n, G), e(n, H * dp), e(n, H), e(n, H * dv), e(n, H * dv)
        ops.delta_inputs(x, z, b, conv, rate, bias, state, memory, of, *seg, qk, kq, v, f, beta, q_scale=d ** -0.5, unit_eps=1e-6, **sizes)
        _walk(chunked, qk, kq, f, beta, v, state, of, seg, y, sizes)
        return y

    pad = state0[:, :memory].view(11, H, dv, dp)
    pad[..., d:] = 0.0                          # what lies behind a head's channels is zero
    together = state0.clone()
    y = run(x, z, b, lengths, slots, together)
    at = 0
    for length, slot in zip(lengths, slots):
        alone = state0.clone()
        part = slice(at, at + length)
        mine = run(x[part].contiguous(), z[part].contiguous(), b[part].contiguous(), [length], [slot], alone)
        assert torch.equal(mine, y[part]), f"request of {length}"
        assert torch.equal(alone[slot], together[slot])
        at += length
    assert torch.equal(together[4], state0[4])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,taps", [(16, 2, 128, 128, 4), (16, 4, 96, 160, 3), (8, 4, 192, 256, 4), (16, 2, 128, 128, 1), (16, 2, 128, 132, 6)])
def test_the_inputs_of_many_tokens_are_those_of_few(H, G, d, dv, taps, dtype):
    """A step of some thousand tokens (several a wavefront, their inputs asked for together where they are of one portion)
    against the same requests 50 tokens at a time: the same bits, whatever borders fall among a wavefront's tokens."""
    g = torch.Generator().manual_seed(d + taps)
    lengths = [2, 1, 1001, 5, 3, 1, 1, 4, 766, 7, 6, 2, 503]
    n, channels, count = sum(lengths), 2 * G * d + H * dv, len(lengths)
    dp, memory = ops.delta_padded(d), ops.delta_state_size(H, d, dv)
    total = -(-(memory + (taps - 1) * channels) // 4) * 4
    x = torch.randn(n, channels, generator=g).to(DEV, dtype)
    z, b = torch.randn(n, H * d, generator=g).to(DEV, dtype), torch.randn(n, H, generator=g).to(DEV, dtype)
    conv, rate = torch.randn(taps, channels, generator=g).to(DEV), (torch.rand(H, generator=g) + 0.1).to(DEV)
    bias = (-3.0 + torch.randn(H * d, generator=g)).to(DEV)
    state0 = torch.randn(count, total, generator=g).to(DEV)

    def run(x, z, b, lengths, slots, state):
        m = x.shape[0]
        start = torch.cumsum(torch.tensor([0] + lengths), 0)[:-1].tolist()
        of = torch.repeat_interleave(torch.arange(len(lengths), dtype=torch.int32), torch.tensor(lengths)).to(DEV)
        nan = lambda *s: torch.full(s, float("nan"), device=DEV)
        out = nan(2, m, G * dp), nan(m, G), nan(m, H * dv).to(dtype), nan(m, H * dp), nan(m, H)
        ops.delta_inputs(x, z, b, conv, rate, bias, state, memory, of, _i32(start), _i32(lengths), _i32(slots), *out, q_scale=d ** -0.5,
                         unit_eps=1e-6, single_tokens=False, heads=H, groups=G, head_dim=d, value_dim=dv)
        return out

    together, apart = state0.clone(), state0.clone()
    all_at_once = run(x, z, b, lengths, list(range(count)), together)
    at = 0
    for slot, length in enumerate(lengths):
        for lo in range(at, at + length, 50):
            part = slice(lo, min(lo + 50, at + length))
            few = run(x[part], z[part], b[part], [part.stop - lo], [slot], apart)
            for name, one, other in zip(("qk", "kq", "v", "f", "beta"), all_at_once, few):
                assert torch.equal(one[:, part] if name == "qk" else one[part], other), f"{name}, request {slot}, tokens from {lo - at}"
        at += length
    assert torch.equal(together, apart)


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
    """400 tokens of which 300 are decoded one by one: single keys decide, the temperature passes many steps, and the
    states go through every step."""
    requests = requests_for("sharp", [400])
    exact = plain_logits(folders["sharp"], requests, torch.float64)
    got = replay(folders["sharp"], trace_tail(requests, tail=300), dtype, 16, max_requests=2, pages=26)
    check_rows(got, folders["sharp"], requests, exact, dtype, sharp=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page_size", [4, 16])
def test_far_keys_that_are_sought(tmp_path, dtype, page_size):
    """The last token seeks the one at a place far back, at a page's first and last slot, at the very start: as the end of a
    prompt's portion and decoded alone."""
    c = seek_config(page_size)
    folder = write_folder(c, str(tmp_path / "m"), seeks)
    raw, w = read_folder(folder)
    for place in (0, 1, page_size - 1, page_size, 255, 256, 499):
        toks = seeking(600, place)
        requests = {"q": toks}
        exact = {"q": plain.forward(toks, w, raw)}
        lost = list(toks)
        lost[place] = 1
        moved = (plain.forward(lost, w, raw)[-1] - exact["q"][-1]).pow(2).mean().sqrt()
        assert moved > 0.2 * exact["q"][-1].pow(2).mean().sqrt()
        for cut in ([600], [599, 1], [300, 298, 2]):
            steps, at = [], 0
            for k in cut:
                steps.append({"step": len(steps), "entries": [{"id": "q", "tokens": toks[at:at + k], "want": [k - 1] if at + k == 600 else []}],
                              "end": ["q"] if at + k == 600 else []})
                at += k
            got = replay(folder, steps, dtype, page_size)
            assert list(got) == [("q", 599)]
            compare_rows(got, exact, relative=2e-4 if dtype == torch.float32 else 0.05)


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


def test_a_slot_that_is_used_again_starts_from_nothing(folders):
    requests = requests_for("sharp", [40, 33, 64, 20])
    exact = plain_logits(folders["sharp"], requests, torch.float64)
    for dtype in DTYPES:
        got = replay(folders["sharp"], trace_portions(requests, sizes=(7, 2, 12)), dtype, 16, max_requests=1, pages=6)
        check_rows(got, folders["sharp"], requests, exact, dtype, sharp=True)


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


def test_captured_steps_in_bfloat16_are_the_eager_ones(folders):
    prompts = list(requests_for("sharp", [37, 5, 64]).values())
    outs = []
    for graphs in (False, True):
        llm = LLM(folders["sharp"], dtype="bfloat16", num_blocks=64, block_size=16, max_prefill_tokens_per_step=32, max_requests=4,
                  hip_graphs=graphs)
        outs.append([o.token_ids for o in llm.generate(prompts, max_new_tokens=40)])
        assert not graphs or llm.runner.graph_steps > 0
    assert outs[0] == outs[1]


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
    r = subprocess.run([sys.executable, "-m", "wllm_amd.cli", "random-model", "--out", str(made), "--config", "modasun-tiny",
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
