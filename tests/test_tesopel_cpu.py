"""Tesopel without a GPU: its configuration, its plan, the plain implementation's own mechanisms against a second way
of computing each, and the engine's bookkeeping around it (a cache that several layers read and whose pages go back by
the widest of their windows, state slots that are zeroed and used again) against the plain implementation, the kernels
replaced by the emulation of their contracts."""
import copy

import pytest
import torch

from helpers import max_live_tokens, replay_and_collect, trace_mixed, trace_portions, trace_tail, trace_whole
from kernel_emulation import EmulatedKernels
from plain import tesopel_plain as plain
from tesopel_helpers import (CONFIGS, compare_rows, config, latent, layer, memory, plain_logits, random_config, reach_config,
                             requests_for, retention, write_folder)
from wllm_amd.architectures import TesopelConfig
from wllm_amd.config import ConfigError
from wllm_amd.engine import ModelRunner
from wllm_amd.engine.replay import TraceReplayer, pages_for_max_tokens
from wllm_amd.kernels import ops
from wllm_amd.parts import build_model, load_model
from wllm_amd.parts.feed_forward import GatedMLP
from wllm_amd.parts.latent_attention import LatentAttention
from wllm_amd.parts.specs import GatedMLPSpec, LatentAttentionSpec

LENGTHS = {"mixed": [70, 45, 90, 33, 58], "odd": [40, 66, 25, 51], "sharp": [100, 37, 64, 80]}
FAMILIES = {"whole": trace_whole, "tail": trace_tail, "portions": trace_portions, "mixed": trace_mixed}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("tesopel")
    return {name: write_folder(name, str(root / name)) for name in CONFIGS}


@pytest.fixture(scope="module")
def exact(folders):
    return {name: plain_logits(folders[name], requests_for(name, LENGTHS[name]), torch.float64) for name in CONFIGS}


# ---- configuration and plan ------------------------------------------------------------------------
def test_the_plan_follows_the_file():
    model = build_model(copy.deepcopy(CONFIGS["mixed"]["config"]))
    plan = model.plan
    assert [type(b.mixer).__name__ for b in plan.layers] == [
        "MatrixMemorySpec", "LatentAttentionSpec", "MatrixMemorySpec", "LatentAttentionSpec", "LatentAttentionSpec",
        "LatentAttentionSpec", "MatrixMemorySpec"]
    assert all(b.arrangement == "post_norm" and b.mixer_norm is None and b.mixer_post_norm.kind == "rms"
               and b.mixer_post_norm.weight_offset == 0.0 and b.mixer_post_norm.eps == 1e-5 and b.mixer_input_conv is None
               for b in plan.layers)
    first, own, ret, wide, other, narrow, _ = (b.mixer for b in plan.layers)
    assert first.gating == "exponential" and first.gate_cap == 8.0 and first.q_scale == 16 ** -0.5 and first.k_scale == 1.0
    assert first.den_eps == 1e-6 and first.gate_activation == "sigmoid" and first.norm_weight == "l0.mix.norm"
    assert (first.i_bias, first.f_bias) == ("l0.mix.i.b", "l0.mix.f.b")
    assert ret.gating == "decay" and ret.decays == (0.8, 0.995) and ret.k_scale == 32 ** -0.5 and ret.q_scale == 1.0
    assert ret.position.rotary_dim == 16 and ret.position.pairing == "half" and ret.position.theta == 10000.0
    assert ret.gate_activation == "silu" and ret.norm_weight is None
    assert (own.num_heads, own.head_dim, own.value_dim, own.kv_rank, own.scale, own.window) == (4, 32, 16, 80, 0.3, 21)
    assert own.q_weight == "l1.mix.q" and own.owns_cache and own.dkv_norm_weight == "l1.mix.dkv.norm" and own.rope_dim == 0
    assert own.gate_weight is None and own.sink_weight is None and own.weights_in_float32 and own.norm_eps == 1e-5
    # the pages of the vectors go back by the widest window of the three layers that read them
    assert own.release_window == wide.release_window == narrow.release_window == 50
    assert not wide.owns_cache and not wide.dkv_weight and wide.window == 50 and narrow.window == 7 and narrow.scale == 0.5
    assert other.owns_cache and other.window == other.release_window == 33
    assert [e.reads_cache_of for e in plan.schedule] == [None, None, None, 1, None, 1, None]
    ff = plan.layers[0].feed_forward
    assert (ff.activation, ff.gate_limit, ff.gate_slope, ff.up_shift, ff.intermediate_size) == ("clamped_swish", 1.2, 1.702, 1.0, 96)
    assert plan.layers[3].feed_forward is None and plan.layers[3].feed_forward_post_norm is None
    assert plan.head.weight is None and plan.head.logit_scale == 0.7 and plan.embedding.scale == 1.0
    shapes = {k: tuple(v.shape) for k, v in model.expected_tensors().items()}
    assert shapes["l1.mix.dkv"] == (80, 64) and shapes["l1.mix.dkv.norm"] == (80,) and shapes["l3.mix.uk"] == (32, 80)
    assert shapes["l3.mix.uv"] == (64, 80) and shapes["l0.mix.i"] == (2, 64) and shapes["l0.mix.norm"] == (64,)
    assert shapes["l2.mix.g"] == (32, 64) and shapes["l6.mlp.up"] == (32, 64)
    assert not {"l3.mix.dkv", "l3.mix.dkv.norm", "l3.norm2", "l2.mix.norm", "head"} & set(shapes)


def test_what_a_request_carries():
    model = build_model(copy.deepcopy(CONFIGS["mixed"]["config"]))
    assert model.state_shapes() == {0: (2 * 16 * 32 + 2 * 16 + 2,), 2: (2 * 32 * 16,), 6: (3 * 8 * 24,)}
    needs = model.cache_needs()
    assert set(needs) == {1, 4} and needs[1].num_kv_heads == 1 and needs[1].head_dim == 96 and needs[1].window == 50
    assert needs[4].head_dim == 64 and needs[4].window == 33


def test_config_errors_name_the_key():
    good = CONFIGS["mixed"]["config"]
    for path, value, word in [(("layers", 1, "mixer", "kv_rank"), None, "kv_rank"), (("layers", 3, "mixer", "kv_rank"), 40, "kv_rank"),
                              (("layers", 3, "mixer", "kv_from"), 0, "kv_from"), (("layers", 3, "mixer", "kv_from"), 4, "kv_from"),
                              (("layers", 5, "mixer", "kv_from"), 3, "kv_from"), (("layers", 0, "type"), "mamba", "type"),
                              (("layers", 0, "mlp", "limit"), None, "limit"), (("layers", 0, "mlp", "kind"), "moe", "kind"),
                              (("layers", 0, "mlp", "limit"), 0.0, "limit"), (("layers", 1, "mixer", "mask"), {"size": 0}, "size"),
                              (("layers", 2, "mixer", "decay"), [0.5], "decay"), (("layers", 2, "mixer", "rot", "dims"), 34, "dims"),
                              (("layers", 0, "mixer", "gate_cap"), None, "gate_cap"), (("norm",), None, "norm")]:
        raw = copy.deepcopy(good)
        at = raw
        for k in path[:-1]:
            at = at[k]
        if value is None:
            del at[path[-1]]
        else:
            at[path[-1]] = value
        with pytest.raises(ConfigError, match=word):
            TesopelConfig.from_dict(raw)
    read = TesopelConfig.from_dict(copy.deepcopy(good))
    assert read.to_dict() == good
    from dataclasses import replace
    assert replace(read, raw=None).to_dict() == good


def test_parts_refuse_what_they_cannot_do():
    base = dict(hidden_size=32, num_heads=2, head_dim=8, value_dim=8, kv_rank=16, q_weight="q", uk_weight="uk", uv_weight="uv",
                o_weight="o")
    for bad in (dict(window=0, dkv_weight="d"), dict(window=9, release_window=8, dkv_weight="d"), dict(release_window=8, dkv_weight="d"),
                dict(owns_cache=False, dkv_weight="d"), dict(kv_rank=300, dkv_weight="d")):
        with pytest.raises(ValueError):
            LatentAttention(LatentAttentionSpec(**{**base, **bad}))
    for bad in (dict(activation="clamped_swish"), dict(activation="silu", gate_limit=2.0), dict(activation="clamped_swish", gate_limit=-1.0)):
        with pytest.raises(ValueError):
            GatedMLP(GatedMLPSpec(hidden_size=32, intermediate_size=16, gate_weight="g", up_weight="u", down_weight="d", **bad))
    with pytest.raises(ops.KernelShapeError):
        ops.gated_activation(torch.zeros(2, 8), torch.zeros(2, 4), "swish")


# ---- the plain implementation's mechanisms, each against another way of computing it ----------------
def test_a_window_holds_the_token_and_those_before_it():
    for size in (1, 3, 7, 50):
        m = plain.window_mask(12, size)
        for i in range(12):
            assert [j for j in range(12) if m[i, j]] == list(range(max(0, i - size + 1), i + 1))


def test_latent_attention_is_attention_in_the_latent_space():
    c = {"heads": 2, "dim": 4, "vdim": 3, "kv_rank": 5, "scale": 0.6, "mask": {"size": 4}}
    g = torch.Generator().manual_seed(6)
    width, T = 7, 11
    w = {"m.q": torch.randn(8, width, generator=g), "m.dkv": torch.randn(5, width, generator=g), "m.dkv.norm": torch.rand(5, generator=g) + 0.5,
         "m.uk": torch.randn(8, 5, generator=g), "m.uv": torch.randn(6, 5, generator=g), "m.o": torch.eye(6)}
    w = {k: v.double() for k, v in w.items()}
    h, elsewhere = torch.randn(T, width, generator=g).double(), torch.randn(T, width, generator=g).double()
    for source in (h, elsewhere):         # its own vectors, and those made of another stream
        lat = plain.compressed(source, w, "m.", 1e-6)
        got = plain.latent_attention(h, lat, w, "m.", c)
        for t in range(T):
            seen = range(max(0, t - 3), t + 1)
            out = []
            for head in range(2):
                q = w["m.uk"][4 * head:4 * head + 4].T @ (h[t] @ w["m.q"][4 * head:4 * head + 4].T)
                s = torch.softmax(torch.stack([q @ lat[j] for j in seen]) * 0.6, 0)
                out.append(w["m.uv"][3 * head:3 * head + 3] @ sum(s[n] * lat[j] for n, j in enumerate(seen)))
            assert torch.allclose(got[t], torch.cat(out), atol=1e-10)


def _memory_weights(g, heads, dim, vdim, width):
    w = {"m." + n: torch.randn(heads * d, width, generator=g).double() for n, d in (("q", dim), ("k", dim), ("v", vdim), ("g", vdim))}
    w["m.o"] = torch.eye(heads * vdim).double()
    return w


def test_the_mlstm_is_a_weighted_sum_of_what_was_written():
    """Without the running maximum: S_t = sum_s exp(i_s + f_(s+1) + .. + f_t) k_s v_s^T, n alike, and the denominator
    max(|n . q|, 1): the maximum, which starts at 0, scales both by exp(-m)."""
    g = torch.Generator().manual_seed(2)
    T, H, d, dv, width, cap = 14, 2, 3, 4, 6, 2.5
    w = _memory_weights(g, H, d, dv, width)
    for n in ("i", "f"):
        w["m." + n], w[f"m.{n}.b"] = torch.randn(H, width, generator=g).double() * 2, torch.randn(H, generator=g).double()
    w["m.norm"] = torch.rand(H * dv, generator=g).double() + 0.5
    h = torch.randn(T, width, generator=g).double()
    got = plain.mlstm(h, w, "m.", {"heads": H, "dim": d, "vdim": dv, "gate_cap": cap}, 1e-9)
    q, k = (h @ w["m.q"].T).view(T, H, d) / d ** 0.5, (h @ w["m.k"].T).view(T, H, d)
    v, gate = (h @ w["m.v"].T).view(T, H, dv), torch.sigmoid(h @ w["m.g"].T)
    li = cap * torch.tanh((h @ w["m.i"].T + w["m.i.b"]) / cap)
    lf = torch.log(torch.sigmoid(cap * torch.tanh((h @ w["m.f"].T + w["m.f.b"]) / cap)))
    for t in range(T):
        for head in range(H):
            num, nq, m = torch.zeros(dv).double(), 0.0, torch.zeros(()).double() + lf[:t + 1, head].sum()
            for s in range(t + 1):
                log_left = li[s, head] + lf[s + 1:t + 1, head].sum()
                m = torch.maximum(m, log_left)
                qk = (q[t, head] * k[s, head]).sum() * torch.exp(log_left)
                num, nq = num + qk * v[s, head], nq + qk
            # |n . q| and 1 stand over exp(m); the 1e-6 is added after that scaling
            o = num / (torch.maximum(nq.abs(), torch.ones(()).double()) + 1e-6 * torch.exp(m))
            o = o / torch.sqrt((o * o).mean() + 1e-9) * w["m.norm"][head * dv:(head + 1) * dv] * gate[t, head * dv:(head + 1) * dv]
            assert torch.allclose(got[t, head * dv:(head + 1) * dv], o, atol=1e-8)


def test_retention_is_attention_with_decaying_scores():
    g = torch.Generator().manual_seed(3)
    T, H, d, dv, width, decay = 13, 2, 6, 4, 5, [0.7, 0.99]
    w = _memory_weights(g, H, d, dv, width)
    h = torch.randn(T, width, generator=g).double()
    got = plain.retention(h, w, "m.", {"heads": H, "dim": d, "vdim": dv, "decay": decay, "rot": {"dims": 4, "base": 30.0}}, 1e-9)
    q, k, v = ((h @ w["m." + n].T).view(T, H, -1) for n in "qkv")
    z = h @ w["m.g"].T
    f = [30.0 ** (-2 * i / 4) for i in range(2)]
    for t in range(T):
        for head in range(H):
            o = torch.zeros(dv).double()
            for s in range(t + 1):
                # a rotated pair's product depends on the distance alone: as complex numbers, q conj(k) e^(i (t - s) f)
                score = (q[t, head, 4:] * k[s, head, 4:]).sum()
                for i in range(2):
                    a = torch.complex(q[t, head, i], q[t, head, i + 2]) * torch.complex(k[s, head, i], k[s, head, i + 2]).conj()
                    angle = torch.tensor((t - s) * f[i]).double()
                    score = score + (a * torch.complex(torch.cos(angle), torch.sin(angle))).real
                o = o + decay[head] ** (t - s) * score * d ** -0.5 * v[s, head]
            o = o / torch.sqrt((o * o).mean() + 1e-9)
            at = slice(head * dv, (head + 1) * dv)
            assert torch.allclose(got[t, at], o * z[t, at] * torch.sigmoid(z[t, at]), atol=1e-8)


def test_the_feed_forward_holds_its_inputs_under_the_limit():
    g = torch.tensor([-9.0, -1.0, 0.3, 2.0, 50.0]).double()
    u = torch.tensor([-9.0, -1.9, 0.4, 1.0, 50.0]).double()
    got = plain.clamped_swish_gate(g, u, 2.0)
    sig = lambda z: 1 / (1 + torch.exp(torch.tensor(-1.702 * z).double()))
    want = torch.stack([-9.0 * sig(-9.0) * (-2.0 + 1), -1.0 * sig(-1.0) * (-1.9 + 1), 0.3 * sig(0.3) * 1.4,      # the gate has no lower limit
                        2.0 * sig(2.0) * 2.0, 2.0 * sig(2.0) * 3.0])
    assert torch.allclose(got, want)


# ---- the engine's bookkeeping, with emulated kernels ---------------------------------------------------
def _replay(folder, trace, page_size, max_requests=4, pages=None):
    with ops.use_backend(EmulatedKernels(precise=True)):
        model = load_model(folder, "float32", "cpu")
        pages = pages or pages_for_max_tokens(max_live_tokens(trace), page_size)
        runner = ModelRunner.create(model, num_pages=pages, page_size=page_size, max_requests=max_requests, poison_freed_pages=True)
        got = replay_and_collect(TraceReplayer(runner), trace)
    runner.cache.check()
    assert not runner.cache.requests
    return got


@pytest.mark.parametrize("family", list(FAMILIES))
@pytest.mark.parametrize("name", list(CONFIGS))
def test_replay_matches_plain(folders, exact, name, family):
    trace = FAMILIES[family](requests_for(name, LENGTHS[name]))
    got = _replay(folders[name], trace, CONFIGS[name]["page_size"])
    compare_rows(got, exact[name], relative=2e-4 if name != "sharp" else 2e-3)


@pytest.mark.parametrize("seed", range(6))
def test_configurations_drawn_at_random(tmp_path, seed):
    c = random_config(100 + seed)
    folder = write_folder(c, str(tmp_path / "m"))
    requests = requests_for(c, [37, 18, 50, 26])
    exact = plain_logits(folder, requests, torch.float64)
    for family in ("portions", "mixed"):
        compare_rows(_replay(folder, FAMILIES[family](requests), c["page_size"]), exact, relative=5e-4)


def test_a_slot_that_is_used_again_starts_from_nothing(folders):
    requests = requests_for("sharp", [40, 33])
    exact = plain_logits(folders["sharp"], requests, torch.float64)
    got = _replay(folders["sharp"], trace_portions(requests, sizes=(7, 2, 12)), 16, max_requests=1, pages=6)
    compare_rows(got, exact, relative=2e-3)


def test_pages_go_back_by_the_widest_window_of_the_layers_that_read_them():
    """A request of any length in pages for the window alone: the owner's window of 21 would give back pages that the
    reader with a window of 50 still sees, and keeping everything would run out of pages."""
    from wllm_amd.cache.manager import CacheManager
    model = build_model(config(50, 32, [layer(latent(2, 8, 8, 16, 21)), layer(latent(1, 8, 8, 16, 50, kv_from=0)),
                                        layer(memory(1, 8, 8, 5.0)), layer(retention(1, 8, 8, 4, 10.0, [0.9]))]))
    cache = CacheManager(model.cache_needs(), 8, 9, 1, torch.float32, "cpu", allocate_storage=False)
    cache.open("a")
    for _ in range(300):
        cache.reserve("a", 1)
        cache.commit("a", 1)
        first = max(0, cache.context_len("a") - 49) // 8
        table = cache.block_table("a", 0)
        assert all(p < 0 for p in table[:first]) and all(p >= 0 for p in table[first:])
    # and a window of none (a reader that sees everything) keeps everything
    raw = config(50, 32, [layer(latent(2, 8, 8, 16, 21)), layer(latent(1, 8, 8, 16, 50, kv_from=0))])
    del raw["layers"][1]["mixer"]["mask"]
    assert build_model(raw).cache_needs()[0].window is None


@pytest.mark.parametrize("windows", [(5, 9), (16, 8), (7,)])
def test_a_logit_depends_on_the_tokens_in_the_window_and_on_no_other(tmp_path, windows):
    """Every layer reads the vectors of the first, which depend on one token each: the reach is the widest window, not a
    sum over the layers, as it would be if a later layer made its vectors of its own stream."""
    c = reach_config(windows, page_size=4)
    folder = write_folder(c, str(tmp_path / "m"))
    toks = requests_for(c, [45])["q0"]
    p, reach = 13, max(windows)
    other = list(toks)
    other[p] = (toks[p] + 31) % c["config"]["vocab"]
    rows = []
    for t in (toks, other):
        got = _replay(folder, trace_portions({"q": t}), 4)
        rows.append(torch.stack([got[("q", i)] for i in range(45)]))
    differ = [i for i in range(45) if not torch.equal(rows[0][i], rows[1][i])]
    assert differ == list(range(p, p + reach))
