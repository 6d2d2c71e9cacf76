"""Vufasun without a GPU: configuration, registry, cache layout per layer run, the rotation's frequencies; and the plain
statement's own mechanisms against closed forms, and against wrong ones."""
import json
import math
import os

import pytest
import torch

import vufasun_util as vu
from oracle import vufasun as oracle

F64 = torch.float64


def test_configuration_registry_and_cache_layout(tmp_path):
    from splitwise_amd.config import ModelConfig
    from splitwise_amd.model_executor.models.layer_list import layer_runs
    from splitwise_amd.model_executor.models.vufasun import VufasunForCausalLM
    cfg = vu.model_a()
    path = vu.write_model(str(tmp_path / "m"), cfg, vu.random_weights(cfg, 1))
    mc = ModelConfig(path, "float32")
    assert mc.architecture == "vufasun" and mc.uses_ragged_steps and mc.model_class() is VufasunForCausalLM
    assert mc.get_vocab_size() == cfg["vocab"] and mc.get_hidden_size() == cfg["width"]
    assert [i for i, _ in layer_runs(cfg)] == [0, 1, 2, 1, 2, 3] == oracle.layer_order(cfg)
    # one entry per layer RUN: every pass of the loop has pages, and a state, of its own
    par0 = {"paged": [(16, 32), (16, 24)], "state": [(3, 8, 12)]}
    attn1, par2 = {"paged": [(16, 32), (16, 24)]}, {"paged": [(16, 24), (16, 60)], "state": [(2, 12, 8)]}
    assert mc.get_cache_layout(16) == [par0, attn1, par2, attn1, par2, {"paged": [(16, 20), (16, 40)]}]
    with open(os.path.join(path, "config.json")) as f:
        assert json.load(f)["architecture"] == "Vufasun"


def test_layers_and_loops_that_cannot_run_are_refused():
    from splitwise_amd.model_executor.models.vufasun import VufasunForCausalLM, normalize_config
    for loop in [(1, 1, 2), (0, 5, 2), (-1, 2, 2), (0, 2, 0)]:
        with pytest.raises(ValueError):
            normalize_config(dict(vu.model_a(), loop=dict(zip(("start", "stop", "times"), loop))))
    cfg = vu.model_c()
    cfg["layers"][1]["type"] = "windowed"
    with pytest.raises(ValueError):
        VufasunForCausalLM.cache_layout(cfg, 16)


def test_bench_presets_are_whole_models():
    from splitwise_amd.config import ModelConfig
    for name in ("vufasun-2k", "vufasun-4k"):
        layout = ModelConfig(name, "bfloat16").get_cache_layout(16)
        assert len(layout) == 10 and [("state" in spec) for spec in layout].count(True) == 4


def test_weights_find_their_places(tmp_path):
    """Loading on the CPU (no kernel runs): fused projections, padding, stream connections, constants."""
    from splitwise_amd.config import ModelConfig
    from splitwise_amd.model_executor.model_loader import get_model
    for name in vu.MODELS:
        cfg, sd, _ = vu.load(name)
        model = get_model(ModelConfig(vu.write_model(str(tmp_path / name), cfg, sd), "float32"), torch.device("cpu"))
        f = {k: v.float() for k, v in sd.items()}
        for i, (layer, entry) in enumerate(zip(model.layers, cfg["layers"])):
            p = f"l{i}."
            assert torch.equal(layer.hc1.mix, f[p + "hc1.mix"]) and torch.equal(layer.hc1.reads, f[p + "hc1.in"])
            assert torch.equal(layer.hc1.writes, f[p + "hc1.out"]) and torch.equal(layer.norm1.weight, f[p + "norm1"])
            assert (layer.mlp is None) == (entry["mlp"] is None) == (layer.hc2 is None)
            w = layer.mix.in_proj.weight
            names = ["left.q", "left.k", "left.v", "right.q", "right.k", "right.v", "right.g"] if entry["type"] == "parallel" else ["q", "k", "v"]
            want = torch.cat([f[p + "mix." + n] for n in names])
            assert torch.equal(w[:len(want)], want) and (w[len(want):] == 0).all() and w.shape[0] % 16 == 0
            if entry["type"] == "parallel":
                assert layer.mix.retention.decay.tolist() == pytest.approx(entry["mixer"]["right"]["decay"])
                assert torch.equal(layer.mix.attn.k_norm, f[p + "mix.left.k.norm"]) and layer.mix.attn.sink is None
                assert torch.equal(layer.mix.right_norm, f[p + "mix.right.out"])
            else:
                assert torch.equal(layer.mix.attn.sink, f[p + "mix.sink"]) and layer.mix.attn.q_norm is None


@pytest.mark.parametrize("dims,base,sc", [
    (16, 10000.0, None), (64, 500000.0, vu.scaling(8.0, 1.0, 4.0, 8192)), (8, 30.0, vu.scaling(2.0, 1.0, 3.0, 20)),
    (2, 100.0, vu.scaling(4.0, 0.5, 2.0, 5)), (24, 1e6, vu.scaling(4.0, 1.0, 4.0, 300))])
def test_scaled_frequencies(dims, base, sc):
    from splitwise_amd.model_executor.layers.basic import scaled_rotary_frequencies
    f = torch.tensor(oracle.rotary_frequencies({"dims": dims, "base": base, "scaling": sc}), dtype=F64)
    assert torch.allclose(scaled_rotary_frequencies(dims, base, sc).double(), f, rtol=1e-7, atol=0)
    plain = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    if sc is None:
        assert torch.allclose(f, plain, rtol=1e-12)
        return
    wave = 2 * math.pi / plain
    for i in range(dims // 2):
        if wave[i] < sc["original"] / sc["high"]:
            assert f[i] == pytest.approx(float(plain[i]))
        elif wave[i] > sc["original"] / sc["low"]:
            assert f[i] == pytest.approx(float(plain[i]) / sc["factor"])
        else:
            assert plain[i] / sc["factor"] <= f[i] <= plain[i]


def test_streams_are_mixed_from_the_old_ones():
    X = torch.tensor([[[1.0, 2.0]], [[10.0, 20.0]]], dtype=F64)
    mix = torch.tensor([[1.0, 3.0], [2.0, 0.0]], dtype=F64)                # [from, to]
    new = oracle.write_streams(X, mix, torch.tensor([1.0, -1.0], dtype=F64), torch.tensor([[5.0, 7.0]], dtype=F64))
    assert new.tolist() == [[[1 + 20 + 5.0, 2 + 40 + 7.0]], [[3 - 5.0, 6 - 7.0]]]
    assert oracle.read_streams(X, torch.tensor([2.0, 0.5], dtype=F64)).tolist() == [[7.0, 14.0]]


def test_a_sink_takes_its_share():
    g = torch.Generator().manual_seed(0)
    n, H, G, d = 17, 4, 2, 6
    q, k = (torch.randn(n, h, d, generator=g, dtype=F64) for h in (H, G))
    ones, sink = torch.ones(n, G, 1, dtype=F64), torch.tensor([0.0, 2.0, -3.0, 700.0], dtype=F64)
    total = oracle.causal_attention(q, k, ones, 0.7, sink)[..., 0]
    for t, a in ((0, 0), (9, 1), (16, 2)):
        s = torch.exp(0.7 * (k[:t + 1, a // 2] @ q[t, a])).sum()
        assert torch.allclose(total[t, a], s / (torch.exp(sink[a]) + s))
    assert total[:, 3].abs().max() < 1e-200                                # a huge sink: nothing overflows, nothing is left
    assert torch.allclose(oracle.causal_attention(q, k, ones, 0.7), torch.ones(n, H, 1, dtype=F64))
    k2 = k.clone()
    k2[9:] = 30.0                                                          # later keys change nothing
    assert torch.equal(oracle.causal_attention(q, k, ones, 0.7, sink)[:9], oracle.causal_attention(q, k2, ones, 0.7, sink)[:9])


def test_retention_is_a_decayed_sum():
    g = torch.Generator().manual_seed(1)
    n, H, d, dv = 13, 2, 5, 3
    q, k, v = (torch.randn(n, H, s, generator=g, dtype=F64) for s in (d, d, dv))
    decay = [0.8, 1.0]
    o, S = oracle.retention(q, k, v, decay)
    for t in (0, 5, 12):
        for a in range(H):
            want = sum(decay[a] ** (t - j) * (q[t, a] @ k[j, a]) * v[j, a] for j in range(t + 1))
            assert torch.allclose(o[t, a], want)
    o1, S1 = oracle.retention(q[:6], k[:6], v[:6], decay)
    o2, S2 = oracle.retention(q[6:], k[6:], v[6:], decay, S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)


def test_rotation_keeps_lengths_and_depends_on_differences():
    g = torch.Generator().manual_seed(2)
    f = oracle.rotary_frequencies({"dims": 6, "base": 50.0})
    y, z = (torch.randn(1, 8, generator=g, dtype=F64) for _ in range(2))
    r = oracle.rotate_halves(y, 12, f)
    assert torch.allclose(r.norm(), y.norm()) and torch.equal(r[:, 6:], y[:, 6:]) and not torch.allclose(r, y)
    assert torch.allclose((oracle.rotate_halves(y, 12, f) * oracle.rotate_halves(z, 5, f)).sum(),
                          (oracle.rotate_halves(y, 47, f) * oracle.rotate_halves(z, 40, f)).sum(), rtol=1e-5)


def test_activations():
    z = torch.linspace(-6, 6, 49, dtype=F64)
    assert torch.allclose(oracle.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert torch.allclose(oracle.silu(z), torch.nn.functional.silu(z))


def test_every_mechanism_moves_the_logits(monkeypatch):
    """A wrong statement of any one mechanism must be far outside the tolerances of the GPU tests (which compare the
    engine with the right one): planted here in the plain statement."""
    cfg, sd, requests = vu.load("a")
    tokens = requests["r5"][:24]
    right = oracle.logits(cfg, sd, tokens)

    def moved(cfg2=cfg, sd2=sd):
        return vu.row_error(oracle.logits(cfg2, sd2, tokens), right)

    def patched(name, fn):
        with monkeypatch.context() as m:
            m.setattr(oracle, name, fn)
            return moved()
    attention, route, freqs, write, rotate = (getattr(oracle, n) for n in
                                              ("causal_attention", "route", "rotary_frequencies", "write_streams", "rotate_all"))
    assert patched("causal_attention", lambda q, k, v, s, sink=None, first_position=0: attention(q, k, v, s)) > 0.02       # no sink
    assert patched("causal_attention", lambda q, k, v, s, sink=None, first_position=0:
                   attention(q, k, v, s, None if sink is None else 0 * sink)) > 0.02                                       # a sink of 0
    assert patched("rotary_frequencies", lambda rot: freqs({k: v for k, v in rot.items() if k != "scaling"})) > 0.02
    assert patched("rotate_all", lambda y, f: y) > 0.02
    assert patched("write_streams", lambda X, M, b, y: write(X, M.T, b, y)) > 0.02                                         # [to, from]
    assert patched("write_streams", lambda X, M, b, y: X + b.view(-1, 1, 1) * y) > 0.02                                    # no mix
    assert patched("gelu_tanh", oracle.silu) > 0.02
    assert patched("gelu_tanh", lambda z: torch.nn.functional.gelu(z)) > 1e-3                                              # the exact form
    assert patched("route", lambda h, r, top: (route(h, r, top)[0], torch.softmax(torch.topk(h @ r.T, top).values, -1))) > 0.02

    def one_by_one(X, mix, writes, y):                         # streams written one after the other
        X = X.clone()
        for j in range(X.shape[0]):
            X[j] = sum(mix[i, j] * X[i] for i in range(X.shape[0])) + writes[j] * y
        return X
    assert patched("write_streams", one_by_one) > 0.02

    def weights_behind(h, w, mlp):                             # the weight on what the expert returns
        chosen, weights = route(h, w["router"], mlp["router"]["top"])
        out = oracle.gated_ff(h, w["shared.gate"], w["shared.up"], w["shared.down"], oracle.silu)
        for t in range(h.shape[0]):
            for e, p in zip(chosen[t].tolist(), weights[t]):
                out[t] += p * oracle.gated_ff(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], oracle.silu)
        return out
    assert patched("moe_ff", weights_behind) > 0.02
    for times in (1, 3):
        assert moved(dict(cfg, loop=dict(cfg["loop"], times=times))) > 0.02
    for name in ("l0.mix.left.q.norm", "l0.mix.left.out", "l0.mix.right.out", "l1.hc1.in", "l1.hc2.out"):
        assert moved(sd2=dict(sd, **{name: torch.ones_like(sd[name])})) > 0.02, name
    no_shared = json.loads(json.dumps(cfg))
    no_shared["layers"][1]["mlp"].pop("shared")
    assert moved(no_shared) > 0.02
    for decay in ([1.0, 1.0, 1.0], [0.98, 0.9, 0.75]):         # none, and that of another head
        other = json.loads(json.dumps(cfg))
        other["layers"][0]["mixer"]["right"]["decay"] = decay
        assert moved(other) > 0.02
    per_head = oracle.rms_norm

    def heads_apart(u, w, eps):                                # queries and keys normed head by head
        if u.shape[-1] == 64 and w.shape[-1] == 64:
            return (oracle.rms_unit(u.unflatten(-1, (4, 16)), eps).flatten(-2)) * w
        return per_head(u, w, eps)
    assert patched("rms_norm", heads_apart) > 0.01
    assert patched("rms_unit", lambda u, eps: u if u.dim() == 3 else u / torch.sqrt(u.pow(2).mean(-1, keepdim=True) + eps)) > 0.02


def test_no_router_choice_of_the_test_models_is_close(monkeypatch):
    """Where the GPU tests compare whole models, the last chosen score stands clear of the first one left out."""
    right, gaps = oracle.route, []

    def watched(h, router, top):
        scores = torch.sigmoid(h @ router.T).sort(-1, descending=True).values
        if top < scores.shape[1]:
            gaps.append(float((scores[:, top - 1] - scores[:, top]).min()))
        return right(h, router, top)
    monkeypatch.setattr(oracle, "route", watched)
    for name in vu.MODELS:
        cfg, sd, requests = vu.load(name)
        for tokens in requests.values():
            oracle.logits(cfg, sd, tokens)
    assert gaps and min(gaps) > 1e-4
