"""Modasun without a GPU: its configuration, its plan, the plain implementation's own mechanisms against a second way
of computing each, and the engine's bookkeeping around it (state slots that are zeroed and used again, runs that share
weights and keep caches and states of their own) against the plain implementation, the kernels replaced by the emulation
of their contracts."""
import copy
import math

import pytest
import torch

from helpers import max_live_tokens, replay_and_collect, trace_mixed, trace_portions, trace_tail, trace_whole
from kernel_emulation import EmulatedKernels
from modasun_helpers import (CONFIGS, attention, compare_rows, config, delta, dense, experts, layer, plain_logits, random_config,
                             read_folder, requests_for, seek_config, seeking, seeks, write_folder)
from plain import modasun_plain as plain
from wllm_amd.architectures import ModasunConfig
from wllm_amd.config import ConfigError
from wllm_amd.engine import ModelRunner
from wllm_amd.engine.replay import TraceReplayer, pages_for_max_tokens
from wllm_amd.kernels import ops
from wllm_amd.parts import build_model, load_model
from wllm_amd.parts.attention import PagedAttention
from wllm_amd.parts.delta_rule import DeltaRuleMixer
from wllm_amd.parts.feed_forward import MLP
from wllm_amd.parts.mixture_of_experts import MixtureOfExperts
from wllm_amd.parts.specs import AttentionSpec, DeltaRuleSpec, MixtureOfExpertsSpec, MLPSpec
from wllm_amd.weights.checkpoint import ExpectedTensor, WeightError

LENGTHS = {"mixed": [70, 45, 90, 33, 58], "odd": [40, 66, 25, 51], "sharp": [100, 37, 64, 80]}
FAMILIES = {"whole": trace_whole, "tail": trace_tail, "portions": trace_portions, "mixed": trace_mixed}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("modasun")
    return {name: write_folder(name, str(root / name)) for name in CONFIGS}


@pytest.fixture(scope="module")
def exact(folders):
    return {name: plain_logits(folders[name], requests_for(name, LENGTHS[name]), torch.float64) for name in CONFIGS}


# ---- configuration and plan ------------------------------------------------------------------------
def test_the_plan_follows_the_file():
    model = build_model(copy.deepcopy(CONFIGS["mixed"]["config"]))
    plan = model.plan
    assert [type(b.mixer).__name__ for b in plan.layers] == ["DeltaRuleSpec", "AttentionSpec", "AttentionSpec", "DeltaRuleSpec",
                                                             "AttentionSpec"]
    assert all(b.arrangement == "norm_of_sum" and b.stream_weight == 1.5 and b.mixer_norm is None and b.mixer_input_conv is None
               and b.mixer_post_norm.kind == "rms" and b.mixer_post_norm.weight_offset == 1.0 and b.mixer_post_norm.eps == 1e-5
               for b in plan.layers)
    # eight runs: two of them run layer 0 again (one by way of a run that does), one layer 1
    assert [e.layer for e in plan.schedule] == [0, 1, 2, 3, 0, 1, 4, 0] and all(e.reads_cache_of is None for e in plan.schedule)
    d, a, bare, _, last = plan.layers
    m = d.mixer
    assert (m.num_heads, m.num_kv_heads, m.head_dim, m.value_dim, m.conv_taps) == (4, 2, 16, 32, 4)
    assert m.q_scale == 0.25 and m.unit_eps == 1e-6 and m.norm_eps == 1e-5 and m.q_conv_weight == "l0.mix.q.conv"
    m = a.mixer
    assert (m.num_heads, m.num_kv_heads, m.head_dim, m.value_dim, m.scale, m.q_temperature) == (4, 2, 32, 16, 0.4, (0.5, 9))
    assert m.qk_norm_eps == 1e-5 and m.position.kind == "none" and m.window is None and m.weights_in_float32
    assert bare.feed_forward is None and bare.feed_forward_post_norm is None and bare.mixer.q_temperature is None
    assert last.mixer.q_weight == "l6.mix.q" and last.mixer.q_temperature == (-0.2, 40)
    ff = d.feed_forward
    assert (ff.num_experts, ff.top, ff.num_groups, ff.keep_groups, ff.group_best, ff.scoring, ff.normalize) == (8, 3, 4, 2, 2, "sigmoid", True)
    assert ff.correction_weight == "l0.mlp.correction" and ff.shared.intermediate_size == 48 and ff.weight_eps == 1e-20
    assert ff.shared_gate_weight == "l0.mlp.shared.sg" and last.feed_forward.shared_gate_weight is None
    assert (a.feed_forward.kind, a.feed_forward.activation, a.feed_forward.intermediate_size) == ("mlp", "squared_relu", 96)
    assert plan.head.weight is None and plan.embedding.scale == 2.0 and plan.final_norm.weight_offset == 1.0
    shapes = {k: tuple(v.shape) for k, v in model.expected_tensors().items()}
    assert shapes["l0.mix.q"] == (32, 64) and shapes["l0.mix.v"] == (128, 64) and shapes["l0.mix.k.conv"] == (32, 4)
    assert shapes["l0.mix.dt_bias"] == (64,) and shapes["l0.mix.A_log"] == (4,) and shapes["l0.mix.norm"] == (32,)
    assert shapes["l0.mix.a2"][0] == 64 and shapes["l0.mix.g2"][0] == 128 and shapes["l0.mlp.shared.sg"] == (1, 64)
    assert not {"l2.norm2", "l4.mix.q", "l5.mix.q", "l7.norm1", "head"} & set(shapes)


def test_what_a_request_carries():
    model = build_model(copy.deepcopy(CONFIGS["mixed"]["config"]))
    first = 4 * 32 * 16 + 3 * (2 * 32 + 128)
    # every run of a delta rule has a state of its own, every run of an attention a cache
    assert model.state_shapes() == {0: (first,), 3: (2 * 16 * 32 + 2 * (2 * 64 + 32),), 4: (first,), 7: (first,)}
    assert set(model.cache_needs()) == {1, 2, 5, 6}
    # heads of 7 channels are held as 8, and a row is a whole number of fours
    odd = build_model(copy.deepcopy(CONFIGS["odd"]["config"])).state_shapes()
    assert odd[4] == (4 * 9 * 8 + (2 * 2 * 7 + 4 * 9),) and all(s[0] % 4 == 0 for s in odd.values())


def test_config_errors_name_the_key():
    good = CONFIGS["mixed"]["config"]
    for path, value, word in [(("layers", 0, "mixer", "conv"), None, "conv"), (("layers", 0, "mixer", "kv_heads"), 3, "kv_heads"),
                              (("layers", 1, "mixer", "scale"), None, "scale"), (("layers", 1, "mixer", "q_temp", "every"), 0, "every"),
                              (("layers", 1, "mixer", "q_temp", "coef"), None, "coef"), (("layers", 0, "type"), "mamba", "type"),
                              (("layers", 1, "mlp", "ff"), None, "ff"), (("layers", 1, "mlp", "kind"), "gated", "kind"),
                              (("layers", 0, "mlp", "router", "groups", "count"), 3, "groups"),
                              (("layers", 0, "mlp", "router", "top"), 5, "top"), (("layers", 0, "mlp", "shared"), {}, "shared"),
                              (("layers", 4, "weights_of"), 4, "weights_of"), (("layers", 4, "weights_of"), -1, "weights_of"),
                              (("layers", 4, "weights_of"), 3, "weights_of"), (("layers", 5, "mixer", "scale"), 0.5, "weights_of"),
                              (("postln_alpha",), None, "postln_alpha"), (("embedding",), None, "embedding"), (("norm",), None, "norm")]:
        raw = copy.deepcopy(good)
        at = raw
        for k in path[:-1]:
            at = at[k]
        if value is None:
            del at[path[-1]]
        else:
            at[path[-1]] = value
        with pytest.raises(ConfigError, match=word):
            ModasunConfig.from_dict(raw)
    from dataclasses import replace
    for name in CONFIGS:
        read = ModasunConfig.from_dict(copy.deepcopy(CONFIGS[name]["config"]))
        assert read.to_dict() == CONFIGS[name]["config"]
        made = ModasunConfig.from_dict(replace(read, raw=None).to_dict())
        assert replace(made, raw=None) == replace(read, raw=None)


def test_an_axis_that_is_the_checkpoints_to_say(folders, tmp_path):
    e = ExpectedTensor((8, 64), free_axes=(0,))
    assert e.takes((3, 64)) and e.takes((8, 64)) and not e.takes((8, 63)) and not e.takes((0, 64)) and not e.takes((8,))
    model = load_model(folders["mixed"], "float32", "cpu", tiled_copies=False)
    assert [model.blocks[i].mixer.inner for i in (0, 3)] == [24, 8]         # the larger of 12 and 20, of 8 and 5, in eights

    def shorten(tensors):
        tensors["l0.mix.a2"] = tensors["l0.mix.a2"][:, :-1].contiguous()

    with pytest.raises(WeightError, match="l0.mix.a2"):
        load_model(write_folder("mixed", str(tmp_path / "m"), shorten), "float32", "cpu", tiled_copies=False)


def test_parts_refuse_what_they_cannot_do():
    base = dict(hidden_size=32, num_heads=2, num_kv_heads=2, head_dim=8, value_dim=8)
    for bad in (dict(num_kv_heads=3), dict(head_dim=260), dict(conv_taps=0), dict(conv_taps=65), dict(value_dim=0)):
        with pytest.raises(ValueError):
            DeltaRuleMixer(DeltaRuleSpec(**{**base, **bad}))
    with pytest.raises(ValueError):
        MLP(MLPSpec(hidden_size=32, intermediate_size=16, activation="relu"))
    for bad in (dict(group_best=3), dict(shared_gate_weight="g")):
        with pytest.raises(ValueError):
            MixtureOfExperts(MixtureOfExpertsSpec(hidden_size=32, intermediate_size=16, num_experts=4, top=1, **bad))
    for bad in ((0.1, 0), (0.1, 2.5)):
        with pytest.raises(ValueError):
            PagedAttention(AttentionSpec(hidden_size=32, num_heads=2, num_kv_heads=2, head_dim=8, q_temperature=bad))


# ---- the plain implementation's mechanisms, each against another way of computing it ----------------
def test_the_norm_takes_the_sum():
    g = torch.Generator().manual_seed(1)
    x, y, w = torch.randn(5, 9, generator=g).double(), torch.randn(5, 9, generator=g).double(), torch.randn(9, generator=g).double()
    got = plain.norm_of_the_sum(x, y, 1.7, w, 1e-5)
    for t in range(5):
        v = [1.7 * float(x[t, i]) + float(y[t, i]) for i in range(9)]
        rms = math.sqrt(sum(a * a for a in v) / 9 + 1e-5)
        assert torch.allclose(got[t], torch.tensor([a / rms * (1 + float(w[i])) for i, a in enumerate(v)]).double())


def test_the_temperature_rises_at_whole_multiples():
    p = torch.arange(40).double()
    got = plain.query_temperature(p, 0.5, 9)
    for i in range(40):
        assert abs(float(got[i]) - (1 + 0.5 * math.log((i + 1) // 9 + 1))) < 1e-12
    assert got[7] == 1.0 and got[8] > 1.0 and got[16] == got[8] and got[17] > got[16]


def test_attention_looks_at_every_earlier_key():
    g = torch.Generator().manual_seed(4)
    T, width, c = 9, 5, {"heads": 4, "kv_heads": 2, "dim": 3, "vdim": 2, "scale": 0.8, "q_temp": {"coef": 0.4, "every": 3}}
    w = {"m." + n: torch.randn(r, width, generator=g).double() for n, r in (("q", 12), ("k", 6), ("v", 4))}
    w["m.o"] = torch.eye(8).double()
    h = torch.randn(T, width, generator=g).double()
    got = plain.attention(h, w, "m.", c, 1e-5)
    for t in range(T):
        for head in range(4):
            kv = head // 2
            q = w["m.q"][3 * head:3 * head + 3] @ h[t]
            q = q / math.sqrt(float((q * q).mean()) + 1e-5) * (1 + 0.4 * math.log((t + 1) // 3 + 1))
            scores, values = [], []
            for j in range(t + 1):
                k = w["m.k"][3 * kv:3 * kv + 3] @ h[j]
                scores.append(float(q @ (k / math.sqrt(float((k * k).mean()) + 1e-5))) * 0.8)
                values.append(w["m.v"][2 * kv:2 * kv + 2] @ h[j])
            e = [math.exp(s) for s in scores]
            want = sum(a / sum(e) * v for a, v in zip(e, values))
            assert torch.allclose(got[t, 2 * head:2 * head + 2], want, atol=1e-10)


def test_the_short_convolution_ends_with_the_current_token():
    z = torch.tensor([[1.0], [10.0], [100.0]]).double()
    taps = torch.tensor([[0.5, 0.25, 2.0]]).double()
    want = torch.tensor([2.0, 20.25, 200.0 + 2.5 + 0.5]).double()
    assert torch.allclose(plain.short_convolution(z, taps)[:, 0], want * torch.sigmoid(want))


def test_the_delta_rule_is_a_product_of_matrices():
    """S_t = (I - beta k k^T) diag(g) S_(t-1) + beta k v^T, with the product written out."""
    g = torch.Generator().manual_seed(5)
    T, H, d, dv = 12, 2, 4, 3
    q, k = torch.randn(T, H, d, generator=g).double(), plain.unit_vector(torch.randn(T, H, d, generator=g).double())
    v, decay = torch.randn(T, H, dv, generator=g).double(), torch.rand(T, H, d, generator=g).double()
    beta = torch.rand(T, H, generator=g).double()
    got = plain.delta_rule(q, k, v, decay, beta)
    for h in range(H):
        for t in range(T):
            S = torch.zeros(d, dv).double()
            for s in range(t + 1):
                write = beta[s, h] * torch.outer(k[s, h], v[s, h])
                for r in range(s + 1, t + 1):
                    write = (torch.eye(d).double() - beta[r, h] * torch.outer(k[r, h], k[r, h])) @ torch.diag(decay[r, h]) @ write
                S = S + write
            assert torch.allclose(got[t, h], S.T @ q[t, h], atol=1e-10)


def test_what_was_written_last_is_read_back():
    """With beta 1 and a unit key the memory answers the key with the value just written, whatever it held."""
    g = torch.Generator().manual_seed(6)
    k = plain.unit_vector(torch.randn(7, 1, 6, generator=g).double() * 100)
    v, decay = torch.randn(7, 1, 4, generator=g).double(), torch.rand(7, 1, 6, generator=g).double()
    got = plain.delta_rule(k, k, v, decay, torch.ones(7, 1).double())
    assert torch.allclose(got, v, atol=1e-6)


def test_decays_lie_between_nothing_and_one():
    z, a_log, bias = torch.randn(50, 2, 3).double() * 5, torch.tensor([0.3, -1.0]).double(), torch.randn(2, 3).double()
    got = plain.channel_decay(z, a_log, bias)
    want = torch.empty_like(got)
    for h in range(2):
        want[:, h] = (1 + torch.exp(z[:, h] + bias[h])) ** -math.exp(float(a_log[h]))
    assert torch.allclose(got, want, atol=1e-12) and (got > 0).all() and (got < 1).all()


def test_the_choice_of_experts():
    # the correction decides the choice and not the weights
    z = torch.tensor([2.0, 1.0, 0.0, -1.0]).double()
    s = torch.sigmoid(z)
    chosen, weights = plain.choose_experts(z, torch.tensor([-5.0, 0.0, 0.0, 1.0]).double(), 2)
    assert chosen == [3, 1] and torch.allclose(weights, s[[3, 1]] / (s[3] + s[1]))
    # a group's score is the sum of its two best: 0.9 + 0.1 loses against 0.6 + 0.6, though 0.9 is the best of all
    s = torch.tensor([0.9, 0.1, 0.05, 0.6, 0.6, 0.05]).double()
    z, none = torch.log(s / (1 - s)), torch.zeros(6).double()
    assert plain.choose_experts(z, none, 1, 2, 1)[0] == [3]
    # what may not be chosen is below every choice score, negative ones too
    z, c = torch.zeros(4).double(), torch.tensor([-3.0, -4.0, -4.5, -2.0]).double()
    assert plain.choose_experts(z, c, 2, 2, 1)[0] == [3, 2]
    # groups of one expert: its score alone
    assert plain.choose_experts(z, c, 2, 4, 2)[0] == [3, 0]


def test_the_feed_forwards():
    g = torch.Generator().manual_seed(7)
    w = {"f.up": torch.randn(5, 4, generator=g).double(), "f.down": torch.randn(4, 5, generator=g).double()}
    h = torch.randn(3, 4, generator=g).double()
    for t in range(3):
        z = w["f.up"] @ h[t]
        want = w["f.down"] @ torch.tensor([max(float(a), 0.0) ** 2 for a in z]).double()
        assert torch.allclose(plain.dense_feed_forward(h, w, "f.")[t], want)
    c = experts(5, 3, 2, shared=6)
    for e in ("e0", "e1", "e2", "shared"):
        ff = 6 if e == "shared" else 5
        w |= {f"f.{e}.{n}": torch.randn(ff, 4, generator=g).double() for n in ("gate", "up")} | {f"f.{e}.down": torch.randn(4, ff, generator=g).double()}
    w |= {"f.router": torch.randn(3, 4, generator=g).double(), "f.correction": torch.randn(3, generator=g).double(),
          "f.shared.sg": torch.randn(1, 4, generator=g).double()}
    got = plain.expert_feed_forward(h, w, "f.", c)

    def one(x, e):
        z = w[f"f.{e}.gate"] @ x
        return w[f"f.{e}.down"] @ (z / (1 + torch.exp(-z)) * (w[f"f.{e}.up"] @ x))

    for t in range(3):
        chosen, weights = plain.choose_experts(w["f.router"] @ h[t], w["f.correction"], 2)
        want = sum(a * one(h[t], f"e{e}") for e, a in zip(chosen, weights)) + torch.sigmoid(w["f.shared.sg"] @ h[t]) * one(h[t], "shared")
        assert torch.allclose(got[t], want)


# ---- the engine's bookkeeping, with emulated kernels ---------------------------------------------------
def _replay(folder, trace, page_size, max_requests=4, pages=None, splits=1):
    with ops.use_backend(EmulatedKernels(precise=True, splits=splits)):
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
    got = _replay(folders[name], trace, CONFIGS[name]["page_size"], splits=2 if family == "portions" else 1)
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


def test_runs_that_share_weights_keep_what_is_theirs(tmp_path):
    """The same layer three times: a run that read another's cache or state would see another depth's keys."""
    layers = [layer(attention(2, 1, 16, 16, scale=0.7), dense(24)), layer(delta(2, 1, 8, 8, 3), None)]
    layers += [{**copy.deepcopy(layers[i % 2]), "weights_of": i % 2} for i in range(4)]
    c = dict(page_size=8, seed=55, config=config(50, 32, layers, alpha=1.3))
    folder = write_folder(c, str(tmp_path / "m"))
    requests = requests_for(c, [40, 21])
    exact = plain_logits(folder, requests, torch.float64)
    compare_rows(_replay(folder, trace_mixed(requests), 8), exact, relative=2e-4)
    raw, w = read_folder(folder)
    other = copy.deepcopy(raw)
    other["layers"] = other["layers"][:4]
    assert (plain.forward(requests["q0"], w, other) - exact["q0"]).abs().max() > 0.1


def test_a_far_token_that_is_sought_decides(tmp_path):
    c = seek_config(page_size=8)
    folder = write_folder(c, str(tmp_path / "m"), seeks)
    raw, w = read_folder(folder)
    for place in (0, 7, 8, 50):
        toks = seeking(70, place)
        exact = {"q": plain.forward(toks, w, raw)}
        lost = list(toks)
        lost[place] = 1
        moved = (plain.forward(lost, w, raw)[-1] - exact["q"][-1]).pow(2).mean().sqrt()
        assert moved > 0.2 * exact["q"][-1].pow(2).mean().sqrt()
        compare_rows(_replay(folder, trace_tail({"q": toks}, tail=5), 8), exact, relative=2e-4)
