"""Dovisun without a GPU: configuration, registry, cache layout per layer run, the rotation's frequencies, the sampler's
soft cap; and the plain statement's own mechanisms against closed forms, and against wrong ones."""
import json
import math
import os

import pytest
import torch

import dovisun_util as du
from oracle import dovisun as oracle

F64 = torch.float64


def test_configuration_registry_and_cache_layout(tmp_path):
    from splitwise_amd.config import ModelConfig
    from splitwise_amd.model_executor.model_loader import _safetensors_shapes
    from splitwise_amd.model_executor.models.dovisun import DovisunForCausalLM, layer_runs
    cfg = du.model_a()
    sd = du.random_weights(cfg, 1)
    path = du.write_model(str(tmp_path / "m"), cfg, sd)
    mc = ModelConfig(path, "float32")
    assert mc.architecture == "dovisun" and mc.uses_ragged_steps and mc.model_class() is DovisunForCausalLM
    assert mc.get_vocab_size() == cfg["vocab"] and mc.get_hidden_size() == cfg["width"]
    # one entry per layer RUN: every pass of the loop has pages of its own
    assert layer_runs(cfg) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)] == oracle.layer_runs(cfg)
    attn1, lat2 = {"paged": [(16, 32), (16, 24)]}, {"paged": [(16, 32)]}
    assert mc.get_cache_layout(16) == [{"paged": [(16, 24)]}, attn1, lat2, attn1, lat2, {"paged": [(16, 20), (16, 40)]}]
    del mc.hf_config["layers"][0]["mixer"]["q_rank"]           # not named: a tensor's shape
    DovisunForCausalLM.note_tensor_shapes(mc.hf_config, _safetensors_shapes(os.path.join(path, "model.safetensors")))
    assert mc.hf_config["layers"][0]["mixer"]["q_rank"] == 14
    with open(os.path.join(path, "config.json")) as f:
        assert json.load(f)["architecture"] == "Dovisun"


@pytest.mark.parametrize("loop", [(1, 1, 2), (2, 1, 2), (0, 5, 2), (-1, 2, 2), (0, 2, 0)])
def test_loops_that_cannot_run_are_refused(loop):
    from splitwise_amd.model_executor.models.dovisun import layer_runs
    cfg = du.model_a()
    cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    with pytest.raises(ValueError):
        layer_runs(cfg)


def test_layer_runs_of_every_shape_of_loop():
    from splitwise_amd.model_executor.models.dovisun import layer_runs
    for make, _ in du.MODELS.values():
        cfg = make()
        assert layer_runs(cfg) == oracle.layer_runs(cfg)
        n, loop = len(cfg["layers"]), cfg.get("loop")
        extra = (loop["stop"] - loop["start"]) * (loop["times"] - 1) if loop else 0
        assert len(layer_runs(cfg)) == n + extra
        assert sum(first for _, first in layer_runs(cfg)) == (loop["times"] if loop else 0)


def test_bench_presets_are_whole_models():
    from splitwise_amd.config import ModelConfig
    for name in ("dovisun-2k", "dovisun-4k"):
        mc = ModelConfig(name, "bfloat16")
        layout = mc.get_cache_layout(16)
        assert len(layout) == 10 and {len(spec["paged"]) for spec in layout} == {1, 2}


@pytest.mark.parametrize("dims,base,scaling", [
    (16, 10000.0, None), (32, 500000.0, dict(factor=8.0, original=4096, fast=32.0, slow=1.0)),
    (8, 30.0, dict(factor=2.0, original=64, fast=6.0, slow=1.0)), (2, 100.0, dict(factor=4.0, original=128, fast=2.0, slow=1.0)),
    (64, 10000.0, dict(factor=1.0, original=2048, fast=32.0, slow=1.0)), (6, 10.0, dict(factor=16.0, original=7, fast=40.0, slow=0.01))])
def test_yarn_frequencies_and_amplitude(dims, base, scaling):
    from splitwise_amd.model_executor.layers.basic import yarn_rotary
    freqs, amplitude = yarn_rotary(dims, base, scaling)
    rot = {"dims": dims, "base": base, "scaling": scaling}
    assert torch.allclose(freqs.double(), torch.tensor(oracle.yarn_frequencies(rot), dtype=F64), rtol=1e-7, atol=0)
    assert amplitude == pytest.approx(oracle.yarn_amplitude(rot), rel=1e-12)
    plain = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    if scaling is None:
        assert amplitude == 1.0 and torch.allclose(freqs.double(), plain, rtol=1e-7)
        return
    assert amplitude == pytest.approx(1.0 + 0.1 * math.log(scaling["factor"]))
    ratio = plain / freqs.double()                              # from 1 (kept) to factor (slowed), never outside
    assert (ratio > 1 - 1e-6).all() and (ratio < scaling["factor"] * (1 + 1e-6)).all()
    turns = scaling["original"] * plain / (2 * math.pi)         # waves that turn often keep their frequency
    for i in range(dims // 2):
        if turns[i] > scaling["fast"] * (1 + 1e-9):
            assert ratio[i] == pytest.approx(1.0, rel=1e-6)
    assert (ratio[1:] >= ratio[:-1] - 1e-6).all()


def test_unit_heads_attention_and_sink_closed_forms():
    g = torch.Generator().manual_seed(0)
    n, H, G, d, dv = 17, 4, 2, 6, 5
    q, k, v = (torch.randn(n, h, s, generator=g, dtype=F64) for h, s in ((H, d), (G, d), (G, dv)))
    assert torch.allclose(oracle.rms_unit(q, 0.0).pow(2).mean(-1), torch.ones(n, H, dtype=F64))
    ones = torch.ones(n, G, 1, dtype=F64)
    assert torch.allclose(oracle.causal_attention(q, k, ones, 0.7), torch.ones(n, H, 1, dtype=F64))
    total = oracle.causal_attention(q, k, ones, 0.7, sink=True)[..., 0]          # s / (1 + s), s the sum of exp(score)
    for t, a in ((0, 0), (9, 1), (16, 3)):
        s = torch.exp(0.7 * (k[:t + 1, a // 2] @ q[t, a])).sum()
        assert torch.allclose(total[t, a], s / (1 + s))
    # large scores of either sign: nothing overflows, and the sink takes all where every score is far below 0
    far = oracle.causal_attention(100 * q, 100 * k, ones, 1.0, sink=True)
    assert torch.isfinite(far).all()
    neg = oracle.causal_attention(torch.ones(1, 1, d, dtype=F64), -200 * torch.ones(1, 1, d, dtype=F64), torch.ones(1, 1, 1, dtype=F64),
                                  1.0, sink=True)
    assert neg.abs().max() < 1e-300
    # later keys change nothing
    k2 = k.clone()
    k2[9:] = 30.0
    assert torch.equal(oracle.causal_attention(q, k, v, 0.7)[:9], oracle.causal_attention(q, k2, v, 0.7)[:9])


def test_rotation_keeps_lengths_times_the_amplitude_and_depends_on_differences():
    g = torch.Generator().manual_seed(1)
    rot = {"dims": 8, "base": 50.0, "scaling": dict(factor=4.0, original=100, fast=8.0, slow=1.0)}
    f, amp = oracle.yarn_frequencies(rot), oracle.yarn_amplitude(rot)
    y, z = torch.randn(1, 8, generator=g, dtype=F64), torch.randn(1, 8, generator=g, dtype=F64)
    r = oracle.rotate_halves(y, 12, f, amp)
    assert torch.allclose(r.norm(), y.norm() * amp) and not torch.allclose(r, y)
    assert torch.allclose((oracle.rotate_halves(y, 12, f, amp) * oracle.rotate_halves(z, 5, f, amp)).sum(),
                          (oracle.rotate_halves(y, 47, f, amp) * oracle.rotate_halves(z, 40, f, amp)).sum(), rtol=1e-5)


def test_router_weights_are_a_softmax_over_the_chosen():
    h = torch.eye(4, dtype=F64)
    router = torch.tensor([[2.0, 0, 0, -300.0], [1.0, 0, 0, -200.0], [0.5, 0, 0, -100.0]], dtype=F64)
    bias = torch.tensor([0.0, 1.5, 0.0], dtype=F64)
    chosen, w = oracle.route(h, router, bias, 2)
    assert chosen[0].tolist() == [1, 0] and torch.allclose(w[0, 0], 1 / (1 + torch.exp(torch.tensor(-0.5, dtype=F64))))
    assert chosen[3].tolist() == [2, 1] and torch.allclose(w.sum(-1), torch.ones(4, dtype=F64))


def test_sampler_bounds_its_logits():
    from splitwise_amd.model_executor.layers.sampler import Sampler
    g = torch.Generator().manual_seed(2)
    hidden, head = torch.randn(3, 16, generator=g), torch.randn(29, 16, generator=g) * 3
    got = Sampler(29, logit_softcap=4.0)._get_logits(hidden, head, None)
    assert torch.allclose(got, 4.0 * torch.tanh(hidden @ head.T / 4.0), atol=1e-5) and got.abs().max() <= 4.0
    assert torch.equal(Sampler(29)._get_logits(hidden, head, None), torch.matmul(hidden, head.t()))


def test_every_mechanism_moves_the_logits(monkeypatch):
    """A wrong statement of any one mechanism must be far outside the tolerances of the GPU tests (which compare the
    engine with the right one): planted here in the plain statement."""
    cfg = du.model_a()
    sd = du.random_weights(cfg, 21)
    tokens = torch.randint(0, cfg["vocab"], (24,), generator=torch.Generator().manual_seed(3)).tolist()
    right = oracle.logits(cfg, sd, tokens)

    def moved(cfg2=cfg, sd2=sd):
        return du.row_error(oracle.logits(cfg2, sd2, tokens), right)

    def patched(name, fn):
        with monkeypatch.context() as m:
            m.setattr(oracle, name, fn)
            return moved()
    attention, route, rms = oracle.causal_attention, oracle.route, oracle.rms_unit
    assert patched("causal_attention", lambda q, k, v, s, sink=False, first_position=0: attention(q, k, v, s)) > 0.02    # no sink
    assert patched("yarn_amplitude", lambda rot: 1.0) > 0.005
    assert patched("yarn_frequencies", lambda rot: [rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)]) > 0.005
    assert patched("soft_cap", lambda z, cap: z) > 0.02

    def softmax_over_all(h, router, bias, top):
        chosen, _ = route(h, router, bias, top)
        return chosen, torch.softmax(h @ router.T + bias, -1).gather(1, chosen)
    assert patched("route", softmax_over_all) > 0.02
    assert patched("route", lambda h, r, b, top: route(h, r, 0 * b, top)) > 0.02
    for times in (1, 3):
        assert moved(dict(cfg, loop=dict(cfg["loop"], times=times))) > 0.02
    blind = dict(sd)
    blind["loop.in"] = sd["loop.in"].clone()
    blind["loop.in"][:, cfg["width"]:] = 0                     # the embedding left out of a pass's input
    assert moved(sd2=blind) > 0.02
    assert moved(dict(cfg, embedding={"scale": 1.0})) > 0.02
    plain = dict(sd)
    plain["l0.mix.dq.norm"] = torch.ones_like(sd["l0.mix.dq.norm"])
    assert moved(sd2=plain) > 0.005

    # queries and keys as they are in layers that norm their heads
    def no_unit(u, eps):
        return u if u.dim() == 3 else rms(u, eps)
    assert patched("rms_unit", no_unit) > 0.02
