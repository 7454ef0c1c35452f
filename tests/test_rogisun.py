"""The Rogisun design in the layer-list engine against its plain float64 implementation (rogisun_oracle.py): every
mechanism alone, prefill against token-by-token decoding, portions, mixed batches, reused blocks and slots, far and
early tokens, borders of position chunks and recurrence chunks, long decoding, other sizes, generation through the
engine's own entry points. Every case runs on the CPU (torch twin of the executor: host logic) and, marked gpu, on the
HIP kernels."""
from __future__ import annotations

import json
import math
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import rogisun_cases as rc
import rogisun_oracle as oracle
from ollama_operator_amd.engine.sampling import SamplingOptions
from ollama_operator_amd.engine.scheduler import BatchScheduler
from ollama_operator_amd.models.config import StackConfig, UnsupportedArchitecture, load_stack_config

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
BOTH = ["float32", "bfloat16"]
GREEDY = SamplingOptions(temperature=0.0, repeat_penalty=1.0)
F64 = torch.float64


@pytest.fixture(scope="module")
def std(tmp_path_factory):
    return rc.Model(tmp_path_factory.mktemp("rogisun"), rc.standard(), seed=3)


# ------------------------------------------------------------------ configuration
def test_config_roundtrip(std):
    cfg = load_stack_config(std.path)
    assert cfg == rc.standard() and cfg.has_state
    assert StackConfig.from_rogisun(cfg.to_rogisun()) == cfg
    r = std.runner("cpu")
    # K/V pools of the pair layers' attention only
    assert r.kc[0].shape[1:] == (2, 16, 16) and r.vc[0].shape[1:] == (2, 16, 12) and r.kc[1] is None and r.vc[2] is None
    # a slot: the mixers' states and convolution windows, then a ring of 3 + 8 inputs per sublayer
    ring = 11 * 48
    assert r.states[0].shape[1] == 4 * 8 * 14 + 3 * (2 * 16 + 56) + 2 * ring
    assert r.states[1].shape[1] == 3 * 12 * 10 + 2 * ring
    assert r.states[2].shape[1] == 4 * 8 * 6 + 2 * (24 + 32) + ring
    assert r.w.head is r.w.embed


def test_bench_configurations_are_readable():
    """The sizes `bench.py --stack ... --rogisun` measures are valid configurations of the design."""
    sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
    import bench
    for z in bench.ROGISUN_SIZES.values():
        c = bench.rogisun_config(z).to_rogisun()
        assert StackConfig.from_rogisun(c).to_rogisun() == c and len(c["layers"]) == 8


def test_unknown_parts_are_refused():
    c = rc.standard().to_rogisun()
    for path, val in ((("layers", 0, "type"), "conv_mixer"), (("layers", 0, "mlp", "kind"), "dense"),
                      (("layers", 0, "mixer", "left", "kv_heads"), 4), (("layers", 0, "mixer", "left", "mask", "size"), 0),
                      (("layers", 0, "mixer", "right", "kv_heads"), 3), (("layers", 1, "mixer", "decay"), [0.5]),
                      (("layers", 1, "mlp", "router", "top"), 9), (("layers", 2, "mixer", "groups"), 3),
                      (("layers", 2, "mixer", "norm_groups"), 5), (("canon", "taps"), 0)):
        d = json.loads(json.dumps(c))
        node = d
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = val
        with pytest.raises(UnsupportedArchitecture):
            StackConfig.from_rogisun(d)


def test_oracle_mechanisms_by_hand():
    """The plain implementation on numbers worked out by hand."""
    one = torch.ones(1, 1, dtype=F64)
    # blocks of 2 positions: row 2 starts a new block
    assert oracle.visible(4, 2).tolist() == [[True, False, False, False], [True, True, False, False], [False, False, True, False],
                                             [False, False, True, True]]
    # causal convolution: the last tap is the current token's
    x = torch.tensor([[1.0], [10.0], [100.0]], dtype=F64)
    assert oracle.causal_conv(x, torch.tensor([[2.0, 3.0]], dtype=F64)).flatten().tolist() == [3.0, 32.0, 320.0]
    # delta rule, one head, D = Dv = 1, k = q = 1 (positive inputs, unit norm), decay 1/2, beta 1/2: S1 = v/2, and the
    # second write sees S = v/4: u = (v - v/4) / 2, S2 = v/4 + 3v/8 = 5v/8; the read-out is RMS-normed to its sign
    W = {k: one for k in ("q", "k", "q.conv", "k.conv", "v.conv", "o")}
    W.update({"v": 2 * one, "b": 0 * one, "A_log": torch.zeros(1, dtype=F64), "a1": 0 * one, "a2": one, "g1": 0 * one, "g2": one,
              "dt_bias": torch.tensor([math.log(math.expm1(math.log(2.0)))], dtype=F64), "norm": torch.ones(1, dtype=F64)})
    m = dict(heads=1, kv_heads=1, dim=1, vdim=1, conv=1)
    v = 2 / (1 + math.exp(-2.0))
    q = v2 = 1 / (1 + math.exp(-1.0))
    q = q / math.sqrt(q * q + 1e-6)
    k, eps = q, 0.25
    S1 = 0.5 * v * k
    S2 = 0.5 * S1 + k * 0.5 * (v - k * 0.5 * S1)
    got = oracle.gated_delta(torch.ones(2, 1, dtype=F64), W, m, eps).flatten()
    for s, g in zip((S1, S2), got.tolist()):
        assert abs(g - 0.5 * (q * s) / math.sqrt((q * s) ** 2 + eps)) < 1e-12 and v2
    # experts: the weight acts on the input; both clamps
    e = {"gate": 4 * one, "up": -9 * one, "down": one}
    assert abs(float(oracle.expert(0.25 * one, e, 2.0)) - 1.0 / (1 + math.exp(-1.702)) * -1.0) < 1e-12
    assert abs(float(oracle.expert(one, e, 2.0)) - 2.0 / (1 + math.exp(-3.404)) * -1.0) < 1e-12
    got = oracle.route(torch.tensor([0.0, 2.0, 1.0], dtype=F64), 2)
    assert [i for i, _ in got] == [1, 2] and abs(got[0][1] - 1 / (1 + math.exp(-2))) < 1e-12


# ------------------------------------------------------------------ each mechanism alone
MECHANISMS = {
    "linear": ([(rc.linear(), None)], {}),
    "linear_one_head_vdim_wider": ([(rc.linear(decay=(0.95,), dim=5, vdim=33), None)], {}),
    "linear_forgets_all": ([(rc.linear(decay=(0.0, 1e-3, 0.99), dim=8, vdim=8), None)], {}),
    "mamba": ([(rc.mamba(), None)], {}),
    "mamba_group_each_one_tap": ([(rc.mamba(heads=3, vdim=7, state=5, groups=3, conv=1, norm_groups=1), None)], {}),
    "mamba_one_group_five_taps": ([(rc.mamba(heads=2, vdim=16, state=40, groups=1, conv=5, norm_groups=2), None)], {}),
    "pair": ([(rc.pair(), None)], {}),
    "pair_attention_only": ([(rc.pair(right=0.0), None)], {}),
    "pair_delta_only": ([(rc.pair(left=0.0), None)], {}),
    "pair_chunk_of_one": ([(rc.pair(chunk=1, right=0.0), None)], {}),
    "pair_chunk_of_two_head_each": ([(rc.pair(heads=3, kv_heads=3, dim=6, vdim=7, chunk=2, right=0.1), None)], {}),
    "pair_one_chunk_for_all": ([(rc.pair(heads=5, kv_heads=1, dim=12, vdim=70, chunk=1000, right=0.2), None)], {}),
    "delta_head_each_one_tap": ([(rc.pair(left=0.0, r=rc.delta(heads=2, kv_heads=2, dim=5, vdim=9, conv=1, decay_rank=3,
                                                                gate_rank=11)), None)], {}),
    "delta_wide_keys": ([(rc.pair(left=0.0, r=rc.delta(heads=2, kv_heads=1, dim=70, vdim=17, conv=3, decay_rank=16)), None)], {}),
    "delta_one_head_wide_values": ([(rc.pair(left=0.0, r=rc.delta(heads=1, kv_heads=1, dim=16, vdim=100)), None)], {}),
    "experts": ([(rc.linear(), rc.moe())], {}),
    "experts_top_one": ([(rc.mamba(), rc.moe(experts=5, top=1, ff=13, limit=0.5))], {}),
    "experts_all_of_them": ([(rc.linear(), rc.moe(experts=3, top=3, ff=8, limit=30.0))], {}),
    "input_convolution_one_tap": ([(rc.linear(), rc.moe())], dict(taps=1)),
    "input_convolution_eight_taps": ([(rc.mamba(), rc.moe())], dict(taps=8)),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_alone(tmp_path, device, name):
    layers, kw = MECHANISMS[name]
    m = rc.Model(tmp_path, rc.config(layers, **kw), seed=11)
    toks = rc.tokens(45, 96, seed=1)
    want, trail = m.oracle(toks)
    r = m.runner(device)
    got_trail = rc.layer_trail(r, toks)
    assert got_trail.shape == trail.shape
    assert np.abs(got_trail - trail).max() < 1e-4 * max(1.0, np.abs(trail).max()), "residual after the layer"
    rc.check(rc.run_cuts(r, toks, [len(toks)]), want, "float32", name)
    rc.check(rc.run_cuts(r, toks, [20, 21, 23, 25, 45]), want, "float32", name + " in portions")


@pytest.mark.parametrize("device", DEVICES)
def test_router_against_the_plain_choice(tmp_path, device):
    """The engine's routing (ids and weights it leaves behind) equals the plain choice, for shapes on both sides of a wave."""
    for i, f in enumerate([rc.moe(experts=6, top=3), rc.moe(experts=7, top=1), rc.moe(experts=4, top=4), rc.moe(experts=70, top=5)]):
        m = rc.Model(tmp_path, rc.config([(rc.linear(), f)], width=32, vocab=40), seed=20 + i, name=f"r{i}")
        toks = rc.tokens(40, 40, seed=i)
        r = m.runner(device)
        rc.check(rc.run_cuts(r, toks, [17, 40]), m.oracle(toks)[0], "float32", f"router shape {i}")
        z = r.proj[:23, :f.experts].double().cpu()
        for b in (0, 5, 22):
            want = oracle.route(z[b], f.top)
            assert r.eids[b, :f.top].tolist() == [e for e, _ in want]
            assert np.allclose(r.ew[b, :f.top].cpu().numpy(), [w for _, w in want], rtol=1e-5)


# ------------------------------------------------------------------ whole prompts, decoding, portions
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", BOTH)
def test_whole_prompt_and_layers(std, device, dtype):
    toks = rc.tokens(60, 96, seed=2)
    want, trail = std.oracle(toks)
    r = std.runner(device, dtype)
    got_trail = rc.layer_trail(r, toks)
    for i in range(trail.shape[0]):
        d = got_trail[i] - trail[i]
        if dtype == "float32":
            assert np.abs(d).max() < 1e-4 * max(1.0, np.abs(trail[i]).max()), f"residual after layer {i}"
        else:
            e = np.sqrt((d ** 2).mean(-1)) / np.sqrt((trail[i] ** 2).mean(-1))
            assert np.median(e) < 0.03, f"residual after layer {i}"
    rc.check(rc.run_cuts(r, toks, [len(toks)]), want, dtype, "whole prompt")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", BOTH)
def test_prefill_then_token_by_token(std, device, dtype):
    toks = rc.tokens(80, 96, seed=4)
    rc.check(rc.run_cuts(std.runner(device, dtype), toks, [40] + list(range(41, 81))), std.oracle(toks)[0], dtype,
             "prefill 40, then one by one")


@pytest.mark.parametrize("device", DEVICES)
def test_every_token_alone_from_the_start(std, device):
    toks = rc.tokens(37, 96, seed=5)
    rc.check(rc.run_cuts(std.runner(device), toks, list(range(1, 38))), std.oracle(toks)[0], "float32", "one by one from 0")


@pytest.mark.parametrize("device", DEVICES)
def test_portions_of_many_sizes(std, device):
    """Portions of 2, 3, 1, 17, ... tokens across block borders (16), recurrence chunks (32) and position chunks (11, 24);
    portions of 2 to 9 tokens on the kernels for few rows; more rows than one forward holds (max_batch 32)."""
    toks = rc.tokens(150, 96, seed=6)
    want, _ = std.oracle(toks)
    r = std.runner(device, max_batch=32)
    cuts = [2, 5, 6, 8, 10, 27, 31, 32, 33, 35, 64, 66, 127, 129, 131, 150]
    rc.check(rc.run_cuts(r, toks, cuts), want, "float32", "portions")
    r = std.runner(device, max_batch=128)
    rc.check(rc.run_cuts(r, toks, [1, 3, 34, 35, 99, 150]), want, "float32", "portions over several chunks")
    for n in (2, 3, 7, 8, 9):
        cuts = list(range(n, 60, n)) + [60]
        rc.check(rc.run_cuts(r, toks[:60], cuts), want[:60], "float32", f"portions of {n}")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", BOTH)
def test_mixed_batch_equals_each_alone(std, device, dtype):
    """Five requests on four slots and a ten-block pool: portions of some beside single tokens of others, one
    sitting out a step, one ending early and its slot and blocks taken by a newcomer; steps of a few rows that hold
    portions of two tokens beside single ones."""
    V = 96
    reqs = {k: rc.tokens(n, V, seed=30 + i) for i, (k, n) in enumerate([("a", 50), ("b", 7), ("c", 33), ("d", 21), ("e", 40)])}
    if dtype == "float32":
        want = {k: std.oracle(t)[0] for k, t in reqs.items()}
    else:   # rounding apart, a request's logits do not depend on its company
        want = {k: rc.run_cuts(std.runner(device, dtype), t, [len(t)]) for k, t in reqs.items()}
    r = std.runner(device, dtype, kv_tokens=160, max_seqs=4)
    plan = [[("a", 20), ("b", 2)], [("a", 1), ("b", 2), ("c", 3)], [("a", 2), ("b", 3), ("c", 14)], [("a", 1), ("c", 1), ("d", 16)],
            [("c", 15), ("d", 5)], [("a", 26), ("e", 3)], [("e", 30)], [("e", 1)], [("e", 6)]]
    at = {k: 0 for k in reqs}
    sid, got = {}, {k: [] for k in reqs}
    for step in plan:
        entries = []
        for k, n in step:
            if k not in sid:
                sid[k] = r.new_sequence()
            entries.append((sid[k], reqs[k][at[k]:at[k] + n], list(range(n))))
        out = r.step_entries(entries).float().cpu().numpy()
        o = 0
        for k, n in step:
            got[k].append(out[o:o + n])
            o += n
            at[k] += n
            if at[k] == len(reqs[k]):
                r.free_sequence(sid.pop(k))
    assert all(at[k] == len(reqs[k]) for k in reqs)
    for k in reqs:
        rc.check(np.concatenate(got[k]), want[k], dtype, f"request {k} in the mixed batch")


@pytest.mark.parametrize("device", DEVICES)
def test_freed_blocks_and_slots_are_clean(std, device):
    """One slot and a pool for one request: the next request gets the previous one's slot and blocks and must see
    nothing of them, neither in the states nor in the convolutions' windows. The second one starts with a single token."""
    r = std.runner(device, kv_tokens=64, max_seqs=1)
    for seed, cuts in ((40, [33, 34, 60]), (41, [1, 2, 3, 60]), (42, [2, 4, 50, 60])):
        toks = rc.tokens(60, 96, seed=seed)
        rc.check(rc.run_cuts(r, toks, cuts), std.oracle(toks)[0], "float32", f"request {seed} on a reused slot")
    assert r.kv.alloc.n_free == r.kv.alloc.n_blocks and len(r.kv.rows_free) == 1


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(std, device):
    for n in (1, 2, 3):
        toks = rc.tokens(n, 96, seed=50 + n)
        rc.check(rc.run_cuts(std.runner(device), toks, [n]), std.oracle(toks)[0], "float32", f"{n} token prompt")


# ------------------------------------------------------------------ position chunks, far tokens
def _one_key_model(tmp_path, chunk):
    """One pair layer whose second mixer is switched off: queries and keys depend on the token alone, and the query of
    token B points along the key of token A; the last head's distance slope is small (2^-8), so a far key still counts."""
    m = rc.Model(tmp_path, rc.config([(rc.pair(heads=4, kv_heads=1, dim=16, vdim=16, scale=1.0, chunk=chunk, right=0.0), None)],
                                     width=32, vocab=50, taps=1), seed=9)
    A, B = 7, 11
    T = {k: v.double() for k, v in m.tensors.items()}
    ha, hb = (oracle.rms_norm(T["embed"][t], T["l0.norm1"], 1e-5) * (1 + T["l0.canon1"][:, 0]) for t in (A, B))
    ka = T["l0.mix.left.k"] @ ha
    m.set_tensor("l0.mix.left.q", (6.0 * ka[:, None] * hb[None, :] / (hb @ hb)).repeat(4, 1).float())
    return m, A, B


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("where", ["inside", "outside"])
def test_one_key_at_the_chunks_edge(tmp_path, device, where):
    """The last token's query points along the key of ONE earlier token, which is the first of its block of positions
    (inside) or the last of the block before (outside). Decoded alone, as the last row of a prompt portion that starts
    before the block's start, and of a portion of two tokens."""
    chunk = 41
    m, A, B = _one_key_model(tmp_path, chunk)
    body = [t for t in rc.tokens(400, 49, seed=8) if t not in (A, B)]
    n, start = 3 * chunk + 30, 3 * chunk           # the last token sits 29 into the fourth block
    at = start if where == "inside" else start - 1
    toks = body[:at] + [A] + body[at + 1:n - 1] + [B]
    want, _ = m.oracle(toks)
    without = m.oracle(toks[:at] + [body[300]] + toks[at + 1:])[0][-1]
    if where == "inside":
        assert rc.rel_err(want[-1], without) > 0.05, "the key at the edge must matter in this construction"
    else:
        assert rc.rel_err(want[-1], without) < 1e-9, "a key of the block before must not matter"
    r = m.runner(device, max_batch=64, kv_tokens=256)
    rc.check(rc.run_cuts(r, toks, [n - 1, n])[-1:], want[-1:], "float32", "decoded token")
    rc.check(rc.run_cuts(r, toks, [100, n])[-1:], want[-1:], "float32", "prompt portion")
    rc.check(rc.run_cuts(r, toks, [n - 2, n])[-1:], want[-1:], "float32", "portion of two tokens")


@pytest.mark.parametrize("device", DEVICES)
def test_attention_finds_a_far_key_in_a_wide_chunk(tmp_path, device):
    """All the weight of the last token on the FIRST token of a wide chunk, 1600 positions back (the decode attention
    then shares the row's keys among several blocks): the distance penalty of head 3 is 6, its score far above."""
    m, A, B = _one_key_model(tmp_path, 2000)
    body = [t for t in rc.tokens(1800, 49, seed=8) if t not in (A, B)][:1599]
    toks = [A] + body + [B]
    want, _ = m.oracle(toks)
    without = m.oracle([body[0]] + body + [B])[0][-1]
    assert rc.rel_err(want[-1], without) > 0.05, "the far key must matter in this construction"
    r = m.runner(device, max_batch=512, kv_tokens=1680)
    n = len(toks)
    rc.check(rc.run_cuts(r, toks, [n - 1, n])[-1:], want[-1:], "float32", "decoded token asking for a far key")
    rc.check(rc.run_cuts(r, toks, [1400, n])[-1:], want[-1:], "float32", "prompt portion asking for a far key")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["linear", "mamba", "delta"])
def test_state_keeps_the_first_token(tmp_path, device, kind):
    """Recurrences that do not forget: the last logits still depend on the first token, 200 positions back, and the
    engine agrees however the prompt is cut (a state that is lost or taken from a neighbour would show)."""
    mx = {"linear": rc.linear(decay=(1.0, 0.9995)), "mamba": rc.mamba(),
          # (many key directions: writes overlap little)
          "delta": rc.pair(left=0.0, r=rc.delta(heads=2, kv_heads=1, dim=128, vdim=8))}[kind]
    m = rc.Model(tmp_path, rc.config([(mx, None)], width=32, vocab=50), seed=12)
    if kind == "mamba":
        m.set_tensor("l0.mix.A_log", torch.full((4,), -12.0))
        m.set_tensor("l0.mix.dt_bias", torch.full((4,), -3.0))
    elif kind == "delta":
        m.set_tensor("l0.mix.right.A_log", torch.full((2,), -12.0))
    toks = rc.tokens(201, 50, seed=13)
    want, _ = m.oracle(toks)
    other = m.oracle([(toks[0] + 1) % 50] + toks[1:])[0]
    assert rc.rel_err(other[-1], want[-1]) > 2e-3, "the first token must matter in this construction"
    r = m.runner(device, max_batch=128, kv_tokens=256)
    for cuts in ([201], [1, 201], [100, 102, 200, 201], [64, 128] + list(range(129, 202))):
        e = rc.rel_err(rc.run_cuts(r, toks, cuts), want)
        assert e.max() < 5e-5, f"{kind} cut at {cuts[:4]}: {e.max():.3g}"


@pytest.mark.parametrize("device", DEVICES)
def test_strong_and_weak_decays_side_by_side(tmp_path, device):
    """Delta-rule channels that forget within a token (log decays of -50 and less) beside channels that keep for hundreds:
    the chunked form's exponents must not overflow, its running sums must not lose the weak ones."""
    mx = rc.pair(left=0.0, r=rc.delta(heads=2, kv_heads=1, dim=16, vdim=16))
    m = rc.Model(tmp_path, rc.config([(mx, None)], width=32, vocab=50), seed=14)
    m.set_tensor("l0.mix.right.A_log", torch.tensor([2.5, -2.0]))
    m.set_tensor("l0.mix.right.dt_bias", torch.linspace(-8.0, 6.0, 32))
    toks = rc.tokens(150, 50, seed=15)
    want, _ = m.oracle(toks)
    r = m.runner(device, max_batch=256, kv_tokens=256)
    for cuts in ([150], [33, 70, 150], [140] + list(range(141, 151))):
        rc.check(rc.run_cuts(r, toks, cuts), want, "float32", "strong and weak decays")


@pytest.mark.parametrize("device", DEVICES)
def test_long_context_decode(tmp_path, device):
    """Single tokens after 1300 rows, a long row beside short ones, a chunk wider than a split's share of the keys."""
    layers = [(rc.pair(heads=4, kv_heads=2, dim=16, vdim=24, scale=0.4, chunk=5000), None),
              (rc.mamba(), None), (rc.pair(heads=2, kv_heads=1, chunk=650), None)]
    m = rc.Model(tmp_path, rc.config(layers, width=32, vocab=60), seed=21)
    toks = rc.tokens(1306, 60, seed=22)
    want, _ = m.oracle(toks)
    r = m.runner(device, max_batch=512, kv_tokens=1400)
    got = rc.run_cuts(r, toks, [1298] + list(range(1299, 1307)))
    rows = list(range(1298, 1306))                  # 1300 is a border of the 650 chunks
    rc.check(got[rows], want[rows], "float32", "decoded after a long context")
    short = rc.tokens(9, 60, seed=23)
    ws = m.oracle(short)[0]
    a, b = r.new_sequence(), r.new_sequence()
    r.step_entries([(a, toks[:1200], []), (b, short[:5], [])])
    out = r.step_entries([(a, toks[1200:1201], [0]), (b, short[5:7], [0, 1])]).float().cpu().numpy()
    rc.check(out[:1], want[1200:1201], "float32", "long row of a mixed step")
    rc.check(out[1:], ws[5:7], "float32", "short rows of a mixed step")


# ------------------------------------------------------------------ other sizes
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", BOTH)
def test_other_sizes(tmp_path, device, dtype):
    """Widths, head sizes and hidden sizes that are not multiples of 8 (no vector loads), a vocabulary wider than a tile,
    an eps of its own, three heads per key/value head."""
    layers = [(rc.linear(decay=(0.8, 0.99, 0.5, 0.999, 0.9), dim=14, vdim=22), rc.moe(experts=9, top=3, ff=22, limit=0.7)),
              (rc.pair(heads=6, kv_heads=2, dim=20, vdim=18, scale=0.3, chunk=29, r=rc.delta(heads=6, kv_heads=2, dim=10, vdim=12,
                                                                                               decay_rank=5, gate_rank=9)), None),
              (rc.mamba(heads=6, vdim=9, state=21, groups=3, conv=2, norm_groups=3), rc.moe(experts=5, top=5, ff=6))]
    m = rc.Model(tmp_path, rc.config(layers, width=52, vocab=300, eps=1e-3, taps=3), seed=17)
    toks = rc.tokens(90, 300, seed=18)
    want, _ = m.oracle(toks)
    rc.check(rc.run_cuts(m.runner(device, dtype, max_batch=128), toks, [70, 71, 72, 90]), want, dtype, "odd sizes")


@pytest.mark.parametrize("device", DEVICES)
def test_large_heads(tmp_path, device):
    """Heads whose state fills many registers per thread (128 x 200, 256 x 72, 160 x 130) and keys wider than the chunked
    forms take (walked token by token), in a prompt and decoding."""
    layers = [(rc.mamba(heads=2, vdim=200, state=128, groups=1, norm_groups=1), None),
              (rc.linear(decay=(0.9, 0.99), dim=256, vdim=72), None),
              (rc.pair(left=0.5, r=rc.delta(heads=2, kv_heads=1, dim=160, vdim=130)), None),
              (rc.pair(heads=2, kv_heads=1, dim=200, vdim=150, scale=0.07, left=0.5,
                       r=rc.delta(heads=1, kv_heads=1, dim=128, vdim=256)), None)]
    m = rc.Model(tmp_path, rc.config(layers, width=64, vocab=80), seed=27)
    toks = rc.tokens(70, 80, seed=28)
    want, _ = m.oracle(toks)
    rc.check(rc.run_cuts(m.runner(device, max_batch=64), toks, [60] + list(range(61, 71))), want, "float32", "large heads")


@pytest.mark.parametrize("device", DEVICES)
def test_matrix_core_sizes(tmp_path, device):
    """Sizes the matrix-core products and vector loads take, in both dtypes; a prompt portion over several tiles, position
    chunks and recurrence chunks, then single tokens; experts sorted and multiplied together."""
    layers = [(rc.linear(decay=(0.7, 0.98, 0.995, 0.999), dim=64, vdim=64), rc.moe(experts=8, top=2, ff=64, limit=2.0)),
              (rc.pair(heads=4, kv_heads=2, dim=64, vdim=64, scale=0.125, chunk=70, r=rc.delta(heads=4, kv_heads=2, dim=64, vdim=128,
                                                                                                  decay_rank=16, gate_rank=24)),
               rc.moe(experts=6, top=3, ff=96)),
              (rc.mamba(heads=8, vdim=32, state=64, groups=2, conv=4, norm_groups=2), rc.moe(experts=4, top=1, ff=128)),
              (rc.pair(heads=2, kv_heads=1, dim=128, vdim=128, scale=0.09, chunk=130, r=rc.delta(heads=2, kv_heads=2, dim=128, vdim=64,
                                                                                                   decay_rank=32, gate_rank=8)), None)]
    m = rc.Model(tmp_path, rc.config(layers, width=128, vocab=256), seed=19)
    toks = rc.tokens(200, 256, seed=20)
    want, _ = m.oracle(toks)
    for dtype in BOTH:
        r = m.runner(device, dtype, max_batch=256)
        rc.check(rc.run_cuts(r, toks, [190] + list(range(191, 201))), want, dtype, "matrix-core sizes")
        rc.check(rc.run_cuts(r, toks, [45, 130, 200])[120:], want[120:], dtype, "matrix-core sizes, a portion from the middle")


# ------------------------------------------------------------------ generation through the engine's entry points
def greedy_oracle(m, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(np.argmax(m.oracle(toks)[0][-1])))
    return toks[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generate_and_long_decode(std, device):
    """`Runner.generate` (prefill, the on-device sampler, the decode graph on a GPU) produces the oracle's greedy
    continuation over several block and chunk borders; the next turn extends the cached sequence, a prompt that shares
    only a part starts anew (a recurrent state cannot be cut back)."""
    prompt = rc.tokens(12, 96, seed=60)
    want = greedy_oracle(std, prompt, 40)
    r = std.runner(device, use_graphs=None)
    sid = r.new_sequence()
    got = list(r.generate(sid, prompt, GREEDY, max_tokens=40))
    assert got == want
    more = list(r.generate(sid, prompt + got + [5, 6], GREEDY, max_tokens=4))
    assert more == greedy_oracle(std, prompt + got + [5, 6], 4)
    other = prompt[:6] + [1, 2, 3]
    assert list(r.generate(sid, other, GREEDY, max_tokens=3)) == greedy_oracle(std, other, 3)


@pytest.mark.parametrize("device", DEVICES)
def test_scheduler_batches_requests(std, device):
    r = std.runner(device, max_seqs=5, kv_tokens=1024, use_graphs=None)
    sch = BatchScheduler(r, max_parallel=3)
    try:
        prompts = [rc.tokens(n, 96, seed=70 + i) for i, n in enumerate((9, 20, 14))]
        lens = (12, 5, 9)
        its = [sch.submit(p, GREEDY, max_tokens=k) for p, k in zip(prompts, lens)]
        got = [list(it) for it in its]
        for p, k, g in zip(prompts, lens, got):
            assert g == greedy_oracle(std, p, k)
    finally:
        sch.close()


def test_command_line_generates_token_ids(std, capsys):
    from ollama_operator_amd import cli
    prompt = rc.tokens(9, 96, seed=90)
    cli.main(["tokens", std.path, "--ids", " ".join(map(str, prompt)), "--num-predict", "5", "--device", "cpu",
              "--dtype", "float32"])
    out = capsys.readouterr().out.strip().splitlines()[-1]
    assert [int(t) for t in out.split()] == greedy_oracle(std, prompt, 5)


def test_trace_replay_program(std, tmp_path):
    """bin/trace_run on the CPU twin: a request that sits out a step, one that ends and gives its slot back."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b = rc.tokens(30, 96, seed=91), rc.tokens(12, 96, seed=92)
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:20], want=[0, 19])], end=[]),
             dict(step=1, entries=[dict(id="b", tokens=b, want=[11])], end=["b"]),
             dict(step=2, entries=[dict(id="a", tokens=a[20:], want=[9]), dict(id="c", tokens=b[:2], want=[])], end=["a", "c"])]
    out = tmp_path / "out"
    p = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", std.path, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "64", "--device", "cpu"], input="".join(json.dumps(x) + "\n" for x in steps),
                       capture_output=True, text=True, timeout=300, env={**os.environ, "PYTHON": sys.executable})
    assert p.returncode == 0, p.stderr[-2000:]
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(3)]
    wa, wb = std.oracle(a)[0], std.oracle(b)[0]
    rc.check(np.fromfile(out / "0.f32", "<f4").reshape(2, 96), wa[[0, 19]], "float32", "step 0")
    rc.check(np.fromfile(out / "1.f32", "<f4").reshape(1, 96), wb[[11]], "float32", "step 1")
    rc.check(np.fromfile(out / "2.f32", "<f4").reshape(1, 96), wa[[29]], "float32", "step 2")


# ------------------------------------------------------------------ the HIP executor against its twin
@pytest.mark.gpu
def test_gpu_matches_twin_layer_by_layer(std):
    toks = rc.tokens(50, 96, seed=95)
    for dtype, tol in (("float32", 1e-4), ("bfloat16", 0.05)):
        a = rc.layer_trail(std.runner("cpu", dtype), toks)
        b = rc.layer_trail(std.runner("cuda", dtype), toks)
        for i in range(a.shape[0]):
            assert np.abs(a[i] - b[i]).max() < tol * max(1.0, np.abs(a[i]).max()), f"{dtype}: layer {i}"


@pytest.mark.gpu
@pytest.mark.parametrize("seed", [0, 1, 2, 3, 4, 5])
def test_random_configurations(tmp_path, seed):
    """Configurations drawn at the scale of a small real model, 300-token prompts in portions and whole, then single
    tokens: float32 sharply, bfloat16 by the typical row."""
    rng = random.Random(3000 + seed)
    cfg = rc.random_config(rng)
    m = rc.Model(tmp_path, cfg, seed=seed)
    toks = rc.tokens(300, cfg.n_vocab, seed=seed)
    want, _ = m.oracle(toks)
    cuts = [rng.randint(1, 100), rng.randint(101, 250), 290] + list(range(291, 301))
    rc.check(rc.run_cuts(m.runner("cuda", "float32", max_batch=512, kv_tokens=512), toks, cuts), want, "float32", f"configuration {seed}")
    r = m.runner("cuda", "bfloat16", max_batch=512, kv_tokens=512)
    e = rc.rel_err(rc.run_cuts(r, toks, cuts), want)
    assert np.isfinite(e).all() and np.median(e) < 0.05, f"configuration {seed}: typical row off by {np.median(e):.3g}"
