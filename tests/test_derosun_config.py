"""The Derosun configuration without a GPU: parser, round trip, errors that name the key, the spec and its run order, the
tensors the parts ask for, the frequencies of both scaled rotations; and the plain implementation's own invariants."""
import copy
import math

import pytest
import torch

import plain_derosun as P
from agave_amd.config import ConfigError, DerosunConfig, find_architecture
from agave_amd.config.spec import BiasedAttentionSpec, GatedFfnSpec, LatentAttentionSpec, MlstmSpec
from agave_amd.engine.model import tensor_needs


def sample():
    return P.config([
        P.attention_layer(6, 3, 16, 20, 8, base=900.0, factor=3.0, low=1.5, high=5.0, original=70, softcap=12.0, mlp=P.dense(24)),
        P.mlstm_layer(3, 12, 20, gate_cap=7.5, mlp=None),
        P.latent_layer(3, 12, 6, 20, 28, 40, base=500.0, factor=5.0, fast=20.0, slow=2.0, original=90, mlp=P.dense(56)),
        P.mlstm_layer(2, 16, 8, gate_cap=11.0, mlp=P.dense(40))], vocab=131, width=40, eps=2e-6, alpha=1.75, embed_scale=0.8)


def test_found_by_its_name_and_round_trip():
    raw = sample()
    arch = find_architecture(raw)
    assert arch.name == "Derosun"
    cfg = arch.parse(raw)
    assert isinstance(cfg, DerosunConfig) and DerosunConfig.from_dict(cfg.to_dict()) == cfg and cfg.to_dict() == raw
    assert (cfg.alpha, cfg.embed_scale, cfg.eps) == (1.75, 0.8, 2e-6)
    assert cfg.layers[0].mixer.rot.scaling.high == 5.0 and cfg.layers[1].mixer.gate_cap == 7.5 and cfg.layers[1].ff is None
    assert cfg.layers[2].mixer.rot.scaling.slow == 2.0 and cfg.layers[2].mixer.q_rank == 28 and cfg.layers[3].ff == 40


def test_what_is_not_there_does_not_exist():
    raw = sample()
    del raw["layers"][0]["mixer"]["softcap"], raw["layers"][0]["mixer"]["rot"], raw["layers"][2]["mixer"]["rot"]["scaling"]
    cfg = DerosunConfig.from_dict(raw)
    assert cfg.to_dict() == raw
    spec = cfg.model_spec()
    assert spec.layers[0].mixer.softcap == 0.0 and spec.layers[0].mixer.position.kind == "none"
    assert spec.layers[2].mixer.position.kind == "rope"


@pytest.mark.parametrize("change, word", [
    (lambda c: c.pop("vocab"), "vocab"), (lambda c: c["norm"].pop("eps"), "eps"), (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c.pop("postln_alpha"), "postln_alpha"), (lambda c: c["embedding"].pop("scale"), "scale"), (lambda c: c.pop("embedding"), "embedding"),
    (lambda c: c["layers"][0].update(type="mamba"), "mamba"), (lambda c: c["layers"][0].update(type=["mlstm"]), "type"),
    (lambda c: c["layers"][1]["mixer"].pop("gate_cap"), "gate_cap"), (lambda c: c["layers"][1]["mixer"].update(gate_cap=0.0), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].pop("vdim"), "vdim"), (lambda c: c["layers"][2]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=4), "rot_dim"), (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=5), "even"),
    (lambda c: c["layers"][2]["mixer"].pop("rot"), "rot"), (lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].pop("fast"), "fast"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "kv_heads"), (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "at most 16"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("high"), "high"), (lambda c: c["layers"][0]["mixer"].update(scale="x"), "scale"),
    (lambda c: c["layers"][0]["mixer"].update(softcap=-1.0), "softcap"), (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "moe"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"), (lambda c: c["layers"][0].update(mlp=3), "mlp")])
def test_errors_name_the_key(change, word):
    raw = copy.deepcopy(sample())
    change(raw)
    with pytest.raises(ConfigError, match=word):
        DerosunConfig.from_dict(raw)


def test_spec_and_run_order():
    spec = DerosunConfig.from_dict(sample()).model_spec()
    assert [(e.layer, e.memory, e.writes) for e in spec.order] == [(i, i, True) for i in range(4)]
    assert all(x.kind == "postnorm_sum" and x.residual_scale == 1.75 and x.pre_mixer_norm is None for x in spec.layers)
    a, m, c = (spec.layers[i].mixer for i in range(3))
    assert isinstance(a, BiasedAttentionSpec) and (a.softcap, a.window, a.chunk, a.sink, a.q_bias) == (12.0, None, None, "", "")
    assert (a.q_row_norm.size, a.q_row_norm.weight, a.k_row_norm.size, a.k_row_norm.add_one) == (96, "l0.mix.q.norm", 48, False)
    assert (a.position.kind, a.position.interleaved, a.position.band_low, a.position.band_original) == ("rope_banded", False, 1.5, 70)
    assert isinstance(m, MlstmSpec) and (m.gate_cap, m.floor_eps, m.norm_eps, m.i_bias, m.gate_proj) == (7.5, 1e-6, 2e-6, "l1.mix.i.b", "l1.mix.g")
    assert isinstance(c, LatentAttentionSpec) and (c.q_down, c.q_rank, c.sink, c.gate_proj, c.window) == ("l2.mix.dq", 28, "", "", None)
    assert (c.position.kind, c.position.interleaved, c.position.yarn_fast, c.position.yarn_magnitude_slope) == ("rope_yarn", True, 20.0, 0.1)
    f = spec.layers[0].ffn
    assert isinstance(f, GatedFfnSpec) and (f.activation, f.gate_bias, f.up_bias, f.down_bias) == ("silu", "l0.mlp.gate.b", "l0.mlp.up.b", "l0.mlp.down.b")
    assert spec.layers[1].ffn is None and spec.layers[1].post_ffn_norm is None
    assert spec.final_norm.weight == "final.norm" and spec.head_weight == "head" and spec.embed_scale == 0.8


def test_tensors_the_parts_ask_for():
    raw = sample()
    assert {n.name: tuple(n.shape) for n in tensor_needs(DerosunConfig.from_dict(raw).model_spec())} == P.tensor_shapes(raw)


@pytest.mark.parametrize("layer", [
    P.attention_layer(1, 1, 64, 8, 64, base=1e4, factor=8.0, low=1.0, high=4.0, original=512),       # all three bands
    P.attention_layer(1, 1, 8, 8, 2, base=50.0, factor=2.0, low=1.0, high=4.0, original=3),          # one pair, its wavelength above original
    P.attention_layer(1, 1, 40, 8, 24, base=1e6, factor=4.0, low=2.0, high=2.0, original=300),       # no band between
    P.latent_layer(1, 8, 32, 8, 8, 8, base=1e4, factor=16.0, fast=32.0, slow=1.0, original=256),
    P.latent_layer(1, 8, 2, 8, 8, 8, base=30.0, factor=2.5, fast=8.0, slow=0.5, original=40),
    P.latent_layer(1, 8, 16, 8, 8, 8, base=1e5, factor=1.0, fast=32.0, slow=1.0, original=4096)])     # a factor of 1: the plain rotation
def test_frequencies_of_the_scaled_rotations(layer):
    """The position parts' tables against the plain functions."""
    from agave_amd.parts import BuildEnv, lookup
    spec = DerosunConfig.from_dict(P.config([layer])).model_spec().layers[0].mixer.position
    part = lookup("position", spec.kind)(spec, BuildEnv(torch.float32, torch.device("cpu"), None))
    table, neighbours = part.rotation_table()
    rot = layer["mixer"]["rot"]
    yarn = layer["type"] == "latent_attention"
    want = P.yarn_frequencies(rot) if yarn else P.banded_frequencies(rot)
    assert table.tolist() == pytest.approx(want, rel=1e-12) and neighbours is yarn
    assert part.magnitude == pytest.approx(P.yarn_magnitude(rot) if yarn else 1.0)


def test_state_and_pages_that_the_mixers_ask_for():
    """The bookkeeping without a GPU: three named state tensors for the recurrent mixer, one latent row, grouped heads."""
    from agave_amd.cache import KVCache
    from agave_amd.parts import lookup
    spec = DerosunConfig.from_dict(sample()).model_spec()
    needs = {}
    for i in (0, 2):
        cls = lookup("mixer", spec.layers[i].mixer.kind)
        part = cls.__new__(cls)
        part.spec = spec.layers[i].mixer
        part.kd = part.spec.kv_rank + part.spec.rot_dim if i == 2 else 0
        needs[i] = part.kv_need()
    assert (needs[0].n_kv_heads, needs[0].head_dim, needs[0].v_head_dim, needs[0].window) == (3, 16, 20, None)
    assert (needs[2].n_kv_heads, needs[2].head_dim, needs[2].v_head_dim) == (1, 46, 40)
    cls = lookup("mixer", "mlstm")
    part = cls.__new__(cls)
    part.spec = spec.layers[1].mixer
    state = part.state_need()
    assert {k: v.shape for k, v in state.items()} == {"S": (3, 20, 12), "n": (3, 12), "m": (3,)} and all(v.dtype == torch.float32 for v in state.values())
    cache = KVCache(needs, {1: state}, 2, {k: 4 for k in needs.values()}, torch.float32, None, 200)
    slot = cache.alloc_slot()
    cache.plan_step([slot], [130])
    cache.commit_step([slot], [130])
    assert all(len(g.held(slot)) == 3 for g in cache.groups)
    cache.free_slot(slot)
    assert all(g.pool.n_free == 4 for g in cache.groups)


# ---------------------------------------------------------------- the plain implementation itself
def test_plain_rotations_by_hand():
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 9.0]]], dtype=P.F)
    pos = torch.tensor([3])
    h = P.turn_halves(x, pos, [1.0, 0.1])[0, 0].tolist()
    assert h == pytest.approx([math.cos(3) - 3 * math.sin(3), 2 * math.cos(0.3) - 4 * math.sin(0.3),
                               3 * math.cos(3) + math.sin(3), 4 * math.cos(0.3) + 2 * math.sin(0.3), 9.0])
    n = P.turn_neighbours(x, pos, [1.0, 0.1], 2.0)[0, 0].tolist()
    assert n == pytest.approx([2 * (math.cos(3) - 2 * math.sin(3)), 2 * (2 * math.cos(3) + math.sin(3)),
                               2 * (3 * math.cos(0.3) - 4 * math.sin(0.3)), 2 * (4 * math.cos(0.3) + 3 * math.sin(0.3)), 9.0])


def test_plain_frequencies_by_hand():
    rot = {"base": 100.0, "dims": 6, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 40}}
    f = [1.0, 100.0 ** (-1 / 3), 100.0 ** (-2 / 3)]                       # wavelengths 6.3, 29, 135; kept below 10, slowed above 40
    s = (40 / (2 * math.pi / f[1]) - 1.0) / 3.0
    assert P.banded_frequencies(rot) == pytest.approx([f[0], (1 - s) * f[1] / 4 + s * f[1], f[2] / 4])
    rot = {"base": 10000.0, "dims": 8, "scaling": {"factor": 4.0, "original": 1024, "fast": 32.0, "slow": 1.0}}
    def d(t):
        return 8 * math.log(1024 / (2 * math.pi * t)) / (2 * math.log(10000.0))
    lo, hi = math.floor(d(32.0)), math.ceil(d(1.0))
    assert (lo, hi) == (0, 3)
    ramp = [0.0, 1 / 3, 2 / 3, 1.0]
    base = [10000.0 ** (-2 * e / 8) for e in range(4)]
    assert P.yarn_frequencies(rot) == pytest.approx([b / 4 * r + b * (1 - r) for b, r in zip(base, ramp)])
    assert P.yarn_magnitude(rot) == pytest.approx(1.0 + 0.1 * math.log(4.0))


def test_plain_matrix_memory_by_hand():
    """Two tokens written out; and the stabiliser changes nothing where the divisor's floor does not hold."""
    q, k, v = (torch.tensor(x, dtype=P.F) for x in ([[2.0], [3.0]], [[5.0], [7.0]], [[11.0], [13.0]]))
    i, f = torch.tensor([1.0, 0.5], dtype=P.F), torch.tensor([-0.3, -0.2], dtype=P.F)
    o, (S, n, m) = P.matrix_memory(q, k, v, i, f)
    e = math.exp
    assert m == pytest.approx(0.8)                                          # max(-0.3, 1) = 1, then max(0.8, 0.5)
    S1, n1 = 55.0, 5.0
    assert float(o[0]) == pytest.approx(S1 * 2 / (max(10.0, e(-1.0)) + 1e-6))
    S2, n2 = S1 + e(0.5 - 0.8) * 91.0, n1 + e(0.5 - 0.8) * 7.0
    assert float(S) == pytest.approx(S2) and float(n) == pytest.approx(n2) and float(o[1]) == pytest.approx(S2 * 3 / (n2 * 3 + 1e-6))
    # m starts at 0: a first input gate of -2 leaves m at the forget gate's value, and a small n . q meets the floor
    o, (_, n, m) = P.matrix_memory(q[:1] * 1e-3, k[:1], v[:1], torch.tensor([-2.0], dtype=P.F), torch.tensor([-0.5], dtype=P.F))
    assert m == pytest.approx(-0.5) and float(o) == pytest.approx(e(-1.5) * 55.0 * 2e-3 / (e(0.5) + 1e-6))
    # whole or from a carried state
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(9, n, generator=g, dtype=P.F) for n in (4, 4, 3))
    i, f = torch.randn(9, generator=g, dtype=P.F), -torch.rand(9, generator=g, dtype=P.F)
    whole, end = P.matrix_memory(q, k, v, i, f)
    first, mid = P.matrix_memory(q[:5], k[:5], v[:5], i[:5], f[:5])
    rest, end2 = P.matrix_memory(q[5:], k[5:], v[5:], i[5:], f[5:], mid)
    assert torch.allclose(torch.cat([first, rest]), whole) and torch.allclose(end[0], end2[0]) and end[2] == end2[2]


def test_plain_layer_norms_the_sum():
    cfg = P.config([P.mlstm_layer(1, 4, 4, mlp=P.dense(8))], width=8)
    w = P.random_weights(cfg, 1)
    x = torch.randn(5, 8, dtype=P.F)
    y = P.norm_of_sum(x, 2 * x, w["l0.norm1"], 3.0, 0.0)
    assert torch.allclose((y / w["l0.norm1"]).pow(2).mean(-1), torch.ones(5, dtype=P.F)) and torch.allclose(y, P.rms(x, 0.0) * w["l0.norm1"])
    seen = []
    P.forward(cfg, w, [1, 2, 3], seen)
    assert torch.allclose((seen[0] / w["l0.norm2"]).pow(2).mean(-1), torch.ones(3, dtype=P.F), atol=1e-4)
