"""The Gavasun design in the layer-list engine against its plain float64 implementation (gavasun_oracle.py): every
mechanism alone, prefill against token-by-token decoding, portions, mixed batches, reused blocks and slots, far and
early tokens, edges of windows, position chunks and recurrence chunks, long decoding, other sizes, generation through the
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

import gavasun_cases as gc
import gavasun_oracle as oracle
from ollama_operator_amd.engine.sampling import SamplingOptions
from ollama_operator_amd.engine.scheduler import BatchScheduler
from ollama_operator_amd.models.config import (StackConfig, UnsupportedArchitecture, load_stack_config, rotary_amplitude,
                                               rotary_inv_freq)

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
BOTH = ["float32", "bfloat16"]
GREEDY = SamplingOptions(temperature=0.0, repeat_penalty=1.0)
F64 = torch.float64


@pytest.fixture(scope="module")
def std(tmp_path_factory):
    return gc.Model(tmp_path_factory.mktemp("gavasun"), gc.standard(), seed=3)


# ------------------------------------------------------------------ configuration
def test_config_roundtrip(std):
    cfg = load_stack_config(std.path)
    assert cfg == gc.standard() and cfg.has_state
    assert StackConfig.from_gavasun(cfg.to_gavasun()) == cfg
    assert [(li, ps, first) for li, ps, first in cfg.runs()] == [(0, 0, False), (1, 0, False), (2, 0, False), (1, 1, False), (2, 1, False),
                                                                 (3, 0, False), (4, 0, False), (5, 0, False)]
    r = std.runner("cpu")
    assert r.w.loop_in is None and len(r.states) == 8
    # K/V pools of the attention layers, one row per token of the latent ones, none of the delta rule
    assert r.kc[0].shape[1:] == (2, 16, 16) and r.vc[0].shape[1:] == (2, 16, 12) and r.kc[2].shape[1:] == (1, 16, 26)
    assert r.vc[2] is None and r.kc[1] is None and r.states[2] is None
    # carried convolution inputs: rings of taps - 1 + 8 rows (q | k | v), behind the delta rule's state matrices
    assert r.states[0].shape[1] == (2 + 8) * (6 * 16 + 2 * 16 + 2 * 12)
    assert r.states[1].shape[1] == 4 * 8 * 14 + (3 + 8) * (2 * 2 * 8 + 4 * 14)
    assert r.states[1].data_ptr() != r.states[3].data_ptr(), "every pass of the looped span has its own state"


def test_norm_weights_are_distances_from_one(std):
    r = std.runner("cpu")
    assert torch.allclose(r.w.layers[0]["norm_w"], 1.0 + std.tensors["l0.norm1"].float())
    assert torch.allclose(r.w.final_w, 1.0 + std.tensors["final.norm"].float())


def test_bench_configurations_are_readable():
    """The sizes `bench.py --stack ... --gavasun` measures are valid configurations of the design."""
    sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
    import bench
    for z in bench.GAVASUN_SIZES.values():
        c = bench.gavasun_config(z).to_gavasun()
        assert StackConfig.from_gavasun(c).to_gavasun() == c and len(c["layers"]) == 8


def test_unknown_parts_are_refused():
    c = gc.standard().to_gavasun()
    for path, val in ((("layers", 0, "type"), "conv_mixer"), (("layers", 0, "mlp", "kind"), "sparse"),
                      (("layers", 0, "mixer", "kv_heads"), 4), (("layers", 0, "mixer", "mask", "size"), 0),
                      (("layers", 0, "mixer", "rot", "dims"), 7), (("layers", 0, "mixer", "conv"), 0),
                      (("layers", 0, "mixer", "rot", "scaling", "factor"), 0.0), (("layers", 1, "mixer", "kv_heads"), 3),
                      (("layers", 2, "mixer", "q_rank"), 0), (("layers", 1, "mlp", "router", "top"), 9),
                      (("loop", "stop"), 9)):
        d = json.loads(json.dumps(c))
        node = d
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = val
        with pytest.raises(UnsupportedArchitecture):
            StackConfig.from_gavasun(d)


def test_frequencies_against_the_plain_ones():
    for dims, base, sc in ((16, 500.0, None), (8, 100.0, dict(factor=3.0, fast=8.0, slow=1.0, original=64)),
                           (64, 1e6, dict(factor=2.0, fast=32.0, slow=1.0, original=512)),
                           (4, 10.0, dict(factor=40.0, fast=1.0, slow=1.0, original=4096)),   # ramp over no index at all
                           (6, 1e4, dict(factor=8.0, fast=1e6, slow=1e-6, original=100))):    # ramp over every index
        want, amp = oracle.frequencies(dict(dims=dims, base=base, scaling=sc))
        scaling = ("yarn", sc["factor"], sc["fast"], sc["slow"], sc["original"]) if sc else ()
        assert np.allclose(rotary_inv_freq(dims, base, scaling), want, rtol=1e-13) and rotary_amplitude(scaling) == pytest.approx(amp)


def test_oracle_mechanisms_by_hand():
    """The plain implementation on numbers worked out by hand."""
    one = torch.ones(1, 1, dtype=F64)
    assert oracle.in_window(4, 2).tolist() == [[True, False, False, False], [True, True, False, False], [False, True, True, False],
                                               [False, False, True, True]]
    assert oracle.in_chunk(4, 2).tolist() == [[True, False, False, False], [True, True, False, False], [False, False, True, False],
                                              [False, False, True, True]]
    x = torch.tensor([[1.0], [10.0], [100.0]], dtype=F64)
    assert oracle.causal_conv(x, torch.tensor([[2.0, 3.0]], dtype=F64)).flatten().tolist() == [3.0, 32.0, 320.0]
    # base 100, dims 4: frequencies 1 and 1/10; an index is log10(original / (2 pi t)): 0.3 for fast, 0.7 for slow, so the
    # ramp runs from index 0 to 1; both at 1.5 (from 1 to 2): nothing is divided yet at index 1
    def turns(index):
        return 1000.0 / (2 * math.pi * 10.0 ** index)
    for fast, slow, want in ((0.3, 0.7, [1.0, 0.1 / math.e]), (1.5, 1.5, [1.0, 0.1])):
        sc = dict(factor=math.e, fast=turns(fast), slow=turns(slow), original=1000)
        f, amp = oracle.frequencies(dict(dims=4, base=100.0, scaling=sc))
        assert np.allclose(f, want) and abs(amp - 1.1) < 1e-12
    # a turn by one: adjacent pairs against halves
    v = torch.zeros(2, 1, 4, dtype=F64)
    v[1, 0] = torch.tensor([1.0, 2.0, 3.0, 4.0])
    rot = dict(dims=2, base=1.0)
    c, s = math.cos(1.0), math.sin(1.0)
    assert torch.allclose(oracle.rotate(v, rot, True)[1, 0], torch.tensor([c - 2 * s, 2 * c + s, 3.0, 4.0], dtype=F64))
    rot = dict(dims=4, base=1.0)
    assert torch.allclose(oracle.rotate(v, rot, False)[1, 0], torch.tensor([c - 3 * s, 2 * c - 4 * s, 3 * c + s, 4 * c + 2 * s], dtype=F64))
    # delta rule, one head, D = Dv = 1, decay 1/2, beta 1/2, v = silu(2), k = q near 1: the second write sees half of S1
    W = {k: one for k in ("q", "k", "q.conv", "k.conv", "v.conv", "o")}
    W.update({"v": 2 * one, "b": 0 * one, "A_log": torch.zeros(1, dtype=F64), "a": 0 * one, "g": one,
              "dt_bias": torch.tensor([math.log(math.expm1(math.log(2.0)))], dtype=F64), "norm": torch.ones(1, dtype=F64)})
    v = 2 / (1 + math.exp(-2.0))
    k = 1 / (1 + math.exp(-1.0))
    k = k / math.sqrt(k * k + 1e-6)
    S1 = 0.5 * v * k
    S2 = 0.5 * S1 + k * 0.5 * (v - k * 0.5 * S1)
    got = oracle.gated_delta(torch.ones(2, 1, dtype=F64), W, dict(heads=1, kv_heads=1, dim=1, vdim=1), 0.25).flatten()
    for S, g in zip((S1, S2), got.tolist()):
        assert abs(g - (k * S) / math.sqrt((k * S) ** 2 + 0.25) / (1 + math.exp(-1.0))) < 1e-12
    # router: softmax over all, the two largest, divided by their sum
    got = oracle.route(torch.tensor([0.0, 2.0, 1.0], dtype=F64), 2)
    assert [i for i, _ in got] == [1, 2] and abs(got[0][1] - math.e / (math.e + 1.0)) < 1e-12
    assert abs(float(oracle.gelu(torch.tensor(1.0, dtype=F64))) - 0.8413447460685429) < 1e-12
    # a span of two layers three times
    assert oracle.order(dict(layers=[0] * 4, loop=dict(start=1, stop=3, times=3))) == [0, 1, 2, 1, 2, 1, 2, 3]


# ------------------------------------------------------------------ each mechanism alone
MECHANISMS = {
    "delta": ([(gc.delta(), None)], {}),
    "delta_one_head_one_tap": ([(gc.delta(heads=1, kv_heads=1, dim=5, vdim=33, conv=1), None)], {}),
    "delta_head_each_six_taps": ([(gc.delta(heads=3, kv_heads=3, dim=16, vdim=16, conv=6), None)], {}),
    "delta_wide_keys": ([(gc.delta(heads=2, kv_heads=1, dim=70, vdim=17, conv=3), None)], {}),
    "delta_wide_values": ([(gc.delta(heads=4, kv_heads=1, dim=16, vdim=100, conv=2), None)], {}),
    "latent": ([(gc.latent(), None)], {}),
    "latent_window_of_one": ([(gc.latent(window=1), None)], {}),
    "latent_window_of_two_one_head": ([(gc.latent(heads=1, window=2, q_rank=1), None)], {}),
    "latent_no_window": ([(gc.latent(window=0, vdim=70), None)], {}),
    "latent_plain_frequencies": ([(gc.latent(scaling=()), None)], {}),
    "latent_two_rotated": ([(gc.latent(dim=33, rot_dim=2, kv_rank=17, q_rank=30), None)], {}),
    "latent_unrotated_part": ([(gc.latent(rot=False), None)], {}),
    "attention": ([(gc.attn(), None)], {}),
    "attention_chunk_of_one": ([(gc.attn(chunk=1), None)], {}),
    "attention_chunk_of_two_head_each": ([(gc.attn(heads=3, kv_heads=3, dim=6, vdim=7, chunk=2, rot_dims=6), None)], {}),
    "attention_one_chunk_for_all": ([(gc.attn(heads=5, kv_heads=1, dim=12, vdim=70, chunk=1000), None)], {}),
    "attention_no_mask_no_rotation": ([(gc.attn(chunk=0, rot_dims=0), None)], {}),
    "attention_one_tap": ([(gc.attn(conv=1), None)], {}),
    "attention_two_taps": ([(gc.attn(conv=2), None)], {}),
    "attention_four_taps": ([(gc.attn(heads=4, dim=24, vdim=20, rot_dims=16, conv=4), None)], {}),
    "attention_four_taps_wide_row": ([(gc.attn(heads=33, kv_heads=3, dim=64, vdim=8, rot_dims=64, conv=4), None)], {}),
    "attention_seven_taps": ([(gc.attn(conv=7, chunk=20), None)], {}),
    "attention_one_head": ([(gc.attn(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=8), None)], {}),
    "dense": ([(gc.delta(), gc.dense())], {}),
    "experts": ([(gc.latent(), gc.moe())], {}),
    "experts_none_shared": ([(gc.attn(), gc.moe(shared=0))], {}),
    "experts_top_one": ([(gc.delta(), gc.moe(experts=5, top=1, ff=13, shared=300))], {}),
    "experts_all_of_them": ([(gc.latent(), gc.moe(experts=3, top=3, ff=8, shared=5))], {}),
    "one_expert": ([(gc.delta(), gc.moe(experts=1, top=1, ff=8))], {}),
    "loop_from_the_start": ([(gc.delta(), gc.dense()), (gc.attn(), None)], dict(loop=(0, 2, 3))),
    "loop_of_one_layer_at_the_end": ([(gc.attn(), None), (gc.latent(), gc.moe())], dict(loop=(1, 2, 4))),
    "loop_once": ([(gc.latent(), None), (gc.delta(), None)], dict(loop=(0, 1, 1))),
    "embedding_scale_one": ([(gc.attn(), gc.dense())], dict(scale=1.0)),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_alone(tmp_path, device, name):
    layers, kw = MECHANISMS[name]
    m = gc.Model(tmp_path, gc.config(layers, **kw), seed=11)
    toks = gc.tokens(45, 96, seed=1)
    want, trail = m.oracle(toks)
    r = m.runner(device)
    got_trail = gc.layer_trail(r, toks)
    assert got_trail.shape == trail.shape
    assert np.abs(got_trail - trail).max() < 1e-4 * max(1.0, np.abs(trail).max()), "residual after the layer"
    gc.check(gc.run_cuts(r, toks, [len(toks)]), want, "float32", name)
    gc.check(gc.run_cuts(r, toks, [20, 21, 23, 25, 45]), want, "float32", name + " in portions")


@pytest.mark.parametrize("device", DEVICES)
def test_router_against_the_plain_choice(tmp_path, device):
    """The engine's routing (ids and weights it leaves behind) equals the plain choice, for shapes on both sides of a wave."""
    for i, f in enumerate([gc.moe(experts=6, top=3), gc.moe(experts=7, top=1, shared=0), gc.moe(experts=4, top=4),
                           gc.moe(experts=70, top=5)]):
        m = gc.Model(tmp_path, gc.config([(gc.delta(), f)], width=32, vocab=40), seed=20 + i, name=f"r{i}")
        toks = gc.tokens(40, 40, seed=i)
        r = m.runner(device)
        gc.check(gc.run_cuts(r, toks, [17, 40]), m.oracle(toks)[0], "float32", f"router shape {i}")
        z = r.proj[:23, :f.experts].double().cpu()
        for b in (0, 5, 22):
            want = oracle.route(z[b], f.top)
            assert r.eids[b, :f.top].tolist() == [e for e, _ in want]
            assert np.allclose(r.ew[b, :f.top].cpu().numpy(), [w for _, w in want], rtol=1e-5)


# ------------------------------------------------------------------ whole prompts, decoding, portions
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", BOTH)
def test_whole_prompt_and_layers(std, device, dtype):
    toks = gc.tokens(60, 96, seed=2)
    want, trail = std.oracle(toks)
    r = std.runner(device, dtype)
    got_trail = gc.layer_trail(r, toks)
    for i in range(trail.shape[0]):
        d = got_trail[i] - trail[i]
        if dtype == "float32":
            assert np.abs(d).max() < 1e-4 * max(1.0, np.abs(trail[i]).max()), f"residual after layer run {i}"
        else:
            e = np.sqrt((d ** 2).mean(-1)) / np.sqrt((trail[i] ** 2).mean(-1))
            assert np.median(e) < 0.03, f"residual after layer run {i}"
    gc.check(gc.run_cuts(r, toks, [len(toks)]), want, dtype, "whole prompt")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", BOTH)
def test_prefill_then_token_by_token(std, device, dtype):
    toks = gc.tokens(80, 96, seed=4)
    gc.check(gc.run_cuts(std.runner(device, dtype), toks, [40] + list(range(41, 81))), std.oracle(toks)[0], dtype,
             "prefill 40, then one by one")


@pytest.mark.parametrize("device", DEVICES)
def test_every_token_alone_from_the_start(std, device):
    toks = gc.tokens(50, 96, seed=5)
    gc.check(gc.run_cuts(std.runner(device), toks, list(range(1, 51))), std.oracle(toks)[0], "float32", "one by one from 0")


@pytest.mark.parametrize("device", DEVICES)
def test_portions_of_many_sizes(std, device):
    """Portions of 2, 3, 1, 17, ... tokens across block borders (16), recurrence chunks (32), windows (13, 40) and position
    chunks (11, 24); portions of 2 to 9 tokens around the size up to which a step writes the carried inputs in the launch
    that reads them (8 rows); more rows than one forward holds (max_batch 32)."""
    toks = gc.tokens(150, 96, seed=6)
    want, _ = std.oracle(toks)
    r = std.runner(device, max_batch=32)
    cuts = [2, 5, 6, 8, 10, 27, 31, 32, 33, 35, 64, 66, 127, 129, 131, 150]
    gc.check(gc.run_cuts(r, toks, cuts), want, "float32", "portions")
    r = std.runner(device, max_batch=128)
    gc.check(gc.run_cuts(r, toks, [1, 3, 34, 35, 99, 150]), want, "float32", "portions over several chunks")
    for n in (2, 3, 7, 8, 9, 16, 17):
        cuts = list(range(n, 60, n)) + [60]
        gc.check(gc.run_cuts(r, toks[:60], cuts), want[:60], "float32", f"portions of {n}")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", BOTH)
def test_mixed_batch_equals_each_alone(std, device, dtype):
    """Five requests on four slots and a ten-block pool: portions of some beside single tokens of others, one
    sitting out a step, one ending early and its slot and blocks taken by a newcomer; steps of a few rows that hold
    portions of two tokens beside single ones."""
    V = 96
    reqs = {k: gc.tokens(n, V, seed=30 + i) for i, (k, n) in enumerate([("a", 50), ("b", 7), ("c", 33), ("d", 21), ("e", 40)])}
    if dtype == "float32":
        want = {k: std.oracle(t)[0] for k, t in reqs.items()}
    else:   # rounding apart, a request's logits do not depend on its company
        want = {k: gc.run_cuts(std.runner(device, dtype), t, [len(t)]) for k, t in reqs.items()}
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
        gc.check(np.concatenate(got[k]), want[k], dtype, f"request {k} in the mixed batch")


@pytest.mark.parametrize("device", DEVICES)
def test_freed_blocks_and_slots_are_clean(std, device):
    """One slot and a pool for one request: the next request gets the previous one's slot and blocks and must see
    nothing of them, neither in the states nor in the convolutions' rings. The second one starts with a single token."""
    r = std.runner(device, kv_tokens=64, max_seqs=1)
    for seed, cuts in ((40, [33, 34, 60]), (41, [1, 2, 3, 60]), (42, [2, 4, 50, 60])):
        toks = gc.tokens(60, 96, seed=seed)
        gc.check(gc.run_cuts(r, toks, cuts), std.oracle(toks)[0], "float32", f"request {seed} on a reused slot")
    assert r.kv.alloc.n_free == r.kv.alloc.n_blocks and len(r.kv.rows_free) == 1


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(std, device):
    for n in (1, 2, 3):
        toks = gc.tokens(n, 96, seed=50 + n)
        gc.check(gc.run_cuts(std.runner(device), toks, [n]), std.oracle(toks)[0], "float32", f"{n} token prompt")


# ------------------------------------------------------------------ edges of windows and position chunks, far tokens
A, B = 7, 11   # the query of token B points along the key of token A


def _one_key_model(tmp_path, kind, size):
    """One layer whose queries and keys depend on the token alone (no rotation, convolutions switched to the current token)
    and whose score for (B, A) stands out."""
    if kind == "latent":
        mx = gc.latent(heads=2, dim=16, rot_dim=4, vdim=16, kv_rank=24, q_rank=20, scale=1.0, window=size, rot=False)
    else:
        mx = gc.attn(heads=4, kv_heads=1, dim=16, vdim=16, scale=1.0, chunk=size, conv=2, rot_dims=0)
    m = gc.Model(tmp_path, gc.config([(mx, None)], width=32, vocab=50), seed=9)
    if kind == "attention":
        for k, n in (("q", 64), ("k", 16), ("v", 16)):
            m.set_tensor(f"l0.mix.{k}.b", torch.zeros(n))
            m.set_tensor(f"l0.mix.{k}.conv", torch.tensor([[0.0, 1.0]]).repeat(n, 1))
    T = {k: v.double() for k, v in m.tensors.items()}
    ha, hb = (oracle.centred_norm(T["embed"][t] * 1.7, T["l0.norm1"], 1e-5) for t in (A, B))
    W = oracle.sub(T, "l0.mix.")
    if kind == "latent":
        c = oracle.unit_rms(W["dkv"][:24] @ ha, 1e-5) * W["dkv.norm"]
        k = (W["uk"] @ c).view(2, 16)
        cq = oracle.unit_rms(W["dq"] @ hb, 1e-5) * W["dq.norm"]
        target = torch.cat([k, torch.zeros(2, 4, dtype=F64)], 1).reshape(-1)
        m.set_tensor("l0.mix.uq", (0.4 * target[:, None] * cq[None, :] / (cq @ cq)).float())
    else:
        k = oracle.unit_rms(W["k"] @ ha, 1e-5) * W["k.norm"]
        m.set_tensor("l0.mix.q.norm", torch.ones(64))
        m.set_tensor("l0.mix.q", (k[:, None] * hb[None, :] / (hb @ hb)).repeat(4, 1).float())
    return m


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("where", ["inside", "outside"])
@pytest.mark.parametrize("kind", ["latent", "attention"])
def test_one_key_at_the_edge(tmp_path, device, kind, where):
    """The last token's query points along the key of ONE earlier token, the oldest one that its window (the first of its
    block of positions) still holds, or the one before that. Decoded alone, as the last row of a prompt portion that starts
    before the edge, and of a portion of two tokens."""
    size = 41
    m = _one_key_model(tmp_path, kind, size)
    body = [t for t in gc.tokens(400, 49, seed=8) if t not in (A, B)]
    n = 3 * size + 30                              # the last token sits 29 into the fourth block
    edge = n - size if kind == "latent" else 3 * size
    at = edge if where == "inside" else edge - 1
    toks = body[:at] + [A] + body[at + 1:n - 1] + [B]
    want, _ = m.oracle(toks)
    without = m.oracle(toks[:at] + [body[300]] + toks[at + 1:])[0][-1]
    if where == "inside":
        assert gc.rel_err(want[-1], without) > 0.05, "the key at the edge must matter in this construction"
    else:
        assert gc.rel_err(want[-1], without) < 1e-9, "a key past the edge must not matter"
    r = m.runner(device, max_batch=64, kv_tokens=256)
    gc.check(gc.run_cuts(r, toks, [n - 1, n])[-1:], want[-1:], "float32", "decoded token")
    gc.check(gc.run_cuts(r, toks, [100, n])[-1:], want[-1:], "float32", "prompt portion")
    gc.check(gc.run_cuts(r, toks, [n - 2, n])[-1:], want[-1:], "float32", "portion of two tokens")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["latent", "attention"])
def test_finds_a_far_key(tmp_path, device, kind):
    """All the weight of the last token on the FIRST token of a wide window or chunk, 1600 positions back (the decode
    attention then shares the row's keys among several blocks)."""
    m = _one_key_model(tmp_path, kind, 2000)
    body = [t for t in gc.tokens(1800, 49, seed=8) if t not in (A, B)][:1599]
    toks = [A] + body + [B]
    want, _ = m.oracle(toks)
    without = m.oracle([body[0]] + body + [B])[0][-1]
    assert gc.rel_err(want[-1], without) > 0.05, "the far key must matter in this construction"
    r = m.runner(device, max_batch=512, kv_tokens=1680)
    n = len(toks)
    gc.check(gc.run_cuts(r, toks, [n - 1, n])[-1:], want[-1:], "float32", "decoded token asking for a far key")
    gc.check(gc.run_cuts(r, toks, [1400, n])[-1:], want[-1:], "float32", "prompt portion asking for a far key")


@pytest.mark.parametrize("device", DEVICES)
def test_rotation_at_far_positions(tmp_path, device):
    """Fast rotations 1200 positions from the start: an angle worked out in float32 would show."""
    m = gc.Model(tmp_path, gc.config([(gc.attn(heads=2, kv_heads=1, dim=16, vdim=8, scale=1.0, chunk=400, rot_dims=16, base=1.5), None),
                                      (gc.latent(rot_dim=16, base=1.5, scale=0.5, window=30), None)], width=32, vocab=50), seed=31)
    toks = gc.tokens(1230, 50, seed=32)
    want, _ = m.oracle(toks)
    r = m.runner(device, max_batch=512, kv_tokens=1300)
    got = gc.run_cuts(r, toks, [1220] + list(range(1221, 1231)))
    gc.check(got[1190:], want[1190:], "float32", "far positions")


@pytest.mark.parametrize("device", DEVICES)
def test_state_keeps_the_first_token(tmp_path, device):
    """A delta rule that does not forget: the last logits still depend on the first token, 200 positions back, and the
    engine agrees however the prompt is cut (a state that is lost or taken from a neighbour would show)."""
    m = gc.Model(tmp_path, gc.config([(gc.delta(heads=2, kv_heads=1, dim=128, vdim=8), None)], width=32, vocab=50), seed=12)
    m.set_tensor("l0.mix.A_log", torch.full((2,), -12.0))
    toks = gc.tokens(201, 50, seed=13)
    want, _ = m.oracle(toks)
    other = m.oracle([(toks[0] + 1) % 50] + toks[1:])[0]
    assert gc.rel_err(other[-1], want[-1]) > 2e-3, "the first token must matter in this construction"
    r = m.runner(device, max_batch=128, kv_tokens=256)
    for cuts in ([201], [1, 201], [100, 102, 200, 201], [64, 128] + list(range(129, 202))):
        e = gc.rel_err(gc.run_cuts(r, toks, cuts), want)
        assert e.max() < 5e-5, f"cut at {cuts[:4]}: {e.max():.3g}"


@pytest.mark.parametrize("device", DEVICES)
def test_strong_and_weak_decays_side_by_side(tmp_path, device):
    """Heads that forget within a token (log decays of -80 and less) beside heads that keep for hundreds: the chunked form's
    exponents must not overflow, its running sums must not lose the weak ones."""
    m = gc.Model(tmp_path, gc.config([(gc.delta(heads=4, kv_heads=2, dim=16, vdim=16), None)], width=32, vocab=50), seed=14)
    m.set_tensor("l0.mix.A_log", torch.tensor([4.0, -3.0, 0.0, -8.0]))
    m.set_tensor("l0.mix.dt_bias", torch.tensor([3.0, -4.0, -1.0, 1.0]))
    toks = gc.tokens(150, 50, seed=15)
    want, _ = m.oracle(toks)
    r = m.runner(device, max_batch=256, kv_tokens=256)
    for cuts in ([150], [33, 70, 150], [140] + list(range(141, 151))):
        gc.check(gc.run_cuts(r, toks, cuts), want, "float32", "strong and weak decays")


@pytest.mark.parametrize("device", DEVICES)
def test_convolutions_reach_back_over_cuts(tmp_path, device):
    """Layers whose convolutions take only their OLDEST tap: every output comes from a carried input, across portions of
    every size around the ring's spare rows and across single tokens."""
    m = gc.Model(tmp_path, gc.config([(gc.attn(conv=4, chunk=50), None), (gc.delta(conv=3), None)], width=32, vocab=50), seed=33)
    for li, taps, rows in ((0, 4, dict(q=96, k=32, v=24)), (1, 3, dict(q=16, k=16, v=56))):
        for k, n in rows.items():
            w = torch.zeros(n, taps)
            w[:, 0] = 1.0
            m.set_tensor(f"l{li}.mix.{k}.conv", w)
    toks = gc.tokens(90, 50, seed=34)
    want, _ = m.oracle(toks)
    r = m.runner(device, max_batch=128)
    for cuts in ([90], [1, 2, 3, 4, 5, 90], [7, 14, 15, 23, 24, 33, 34, 60, 61, 90], [40] + list(range(41, 91))):
        gc.check(gc.run_cuts(r, toks, cuts)[5:], want[5:], "float32", f"cut at {cuts[:4]}")


@pytest.mark.parametrize("device", DEVICES)
def test_long_context_decode(tmp_path, device):
    """Single tokens after 1300 rows, a long row beside short ones, windows and chunks wider than a split's share of the
    keys beside ones that begin 1200 keys in."""
    layers = [(gc.attn(heads=4, kv_heads=2, dim=16, vdim=24, scale=0.4, chunk=5000), None), (gc.delta(), None),
              (gc.latent(window=1200), None), (gc.attn(heads=2, kv_heads=1, chunk=650), None), (gc.latent(window=100), None)]
    m = gc.Model(tmp_path, gc.config(layers, width=32, vocab=60), seed=21)
    toks = gc.tokens(1306, 60, seed=22)
    want, _ = m.oracle(toks)
    r = m.runner(device, max_batch=512, kv_tokens=1400)
    got = gc.run_cuts(r, toks, [1298] + list(range(1299, 1307)))
    rows = list(range(1298, 1306))                  # 1300 is a border of the 650 chunks
    gc.check(got[rows], want[rows], "float32", "decoded after a long context")
    short = gc.tokens(9, 60, seed=23)
    ws = m.oracle(short)[0]
    a, b = r.new_sequence(), r.new_sequence()
    r.step_entries([(a, toks[:1200], []), (b, short[:5], [])])
    out = r.step_entries([(a, toks[1200:1201], [0]), (b, short[5:7], [0, 1])]).float().cpu().numpy()
    gc.check(out[:1], want[1200:1201], "float32", "long row of a mixed step")
    gc.check(out[1:], ws[5:7], "float32", "short rows of a mixed step")


# ------------------------------------------------------------------ other sizes
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", BOTH)
def test_other_sizes(tmp_path, device, dtype):
    """Widths, head sizes and hidden sizes that are not multiples of 8 (no vector loads), a vocabulary wider than a tile,
    an eps of its own, three heads per key/value head."""
    layers = [(gc.delta(heads=6, kv_heads=2, dim=10, vdim=12, conv=2), gc.moe(experts=9, top=3, ff=22, shared=21)),
              (gc.attn(heads=6, kv_heads=2, dim=20, vdim=18, scale=0.3, chunk=29, rot_dims=10), gc.dense(ff=27)),
              (gc.latent(heads=5, dim=9, rot_dim=2, vdim=11, kv_rank=13, q_rank=15, window=17), gc.moe(experts=5, top=5, ff=6, shared=3))]
    m = gc.Model(tmp_path, gc.config(layers, width=52, vocab=300, eps=1e-3, loop=(1, 3, 2)), seed=17)
    toks = gc.tokens(90, 300, seed=18)
    want, _ = m.oracle(toks)
    gc.check(gc.run_cuts(m.runner(device, dtype, max_batch=128), toks, [70, 71, 72, 90]), want, dtype, "odd sizes")


@pytest.mark.parametrize("device", DEVICES)
def test_large_heads(tmp_path, device):
    """Heads whose state fills many registers per thread and keys wider than the chunked form takes (walked token by token),
    wide attention heads, latent rows wider than 256, many query rows."""
    layers = [(gc.delta(heads=2, kv_heads=1, dim=160, vdim=130), None), (gc.delta(heads=1, kv_heads=1, dim=128, vdim=256), None),
              (gc.attn(heads=2, kv_heads=1, dim=200, vdim=150, scale=0.07, rot_dims=200), None),
              (gc.attn(heads=40, kv_heads=8, dim=64, vdim=32, scale=0.1, rot_dims=32, chunk=50), None),
              (gc.latent(heads=2, dim=200, rot_dim=40, vdim=180, kv_rank=240, q_rank=300, scale=0.05), None)]
    m = gc.Model(tmp_path, gc.config(layers, width=64, vocab=80), seed=27)
    toks = gc.tokens(70, 80, seed=28)
    want, _ = m.oracle(toks)
    gc.check(gc.run_cuts(m.runner(device, max_batch=64), toks, [60] + list(range(61, 71))), want, "float32", "large heads")


@pytest.mark.parametrize("device", DEVICES)
def test_matrix_core_sizes(tmp_path, device):
    """Sizes the matrix-core products and vector loads take, in both dtypes; a prompt portion over several tiles, windows,
    position chunks and recurrence chunks, then single tokens; experts sorted and multiplied together."""
    layers = [(gc.delta(heads=4, kv_heads=2, dim=64, vdim=128), gc.moe(experts=8, top=2, ff=64, shared=64)),
              (gc.attn(heads=4, kv_heads=2, dim=64, vdim=64, scale=0.06, chunk=70, rot_dims=32), gc.moe(experts=6, top=3, ff=96, shared=0)),
              (gc.latent(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=96, q_rank=64, scale=0.1, window=75), gc.dense(ff=192)),
              (gc.attn(heads=2, kv_heads=1, dim=128, vdim=128, scale=0.04, chunk=130, rot_dims=128), gc.moe(experts=4, top=1, ff=128)),
              (gc.delta(heads=2, kv_heads=2, dim=128, vdim=64), None)]
    m = gc.Model(tmp_path, gc.config(layers, width=128, vocab=256, loop=(1, 3, 2)), seed=19)
    toks = gc.tokens(200, 256, seed=20)
    want, _ = m.oracle(toks)
    for dtype in BOTH:
        r = m.runner(device, dtype, max_batch=256)
        gc.check(gc.run_cuts(r, toks, [190] + list(range(191, 201))), want, dtype, "matrix-core sizes")
        gc.check(gc.run_cuts(r, toks, [45, 130, 200])[120:], want[120:], dtype, "matrix-core sizes, a portion from the middle")


# ------------------------------------------------------------------ generation through the engine's entry points
def greedy_oracle(m, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(np.argmax(m.oracle(toks)[0][-1])))
    return toks[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generate_and_long_decode(std, device):
    """`Runner.generate` (prefill, the on-device sampler, the decode graph on a GPU) produces the oracle's greedy
    continuation over several block, window and chunk borders; the next turn extends the cached sequence, a prompt that
    shares only a part starts anew (a recurrent state cannot be cut back)."""
    prompt = gc.tokens(12, 96, seed=60)
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
        prompts = [gc.tokens(n, 96, seed=70 + i) for i, n in enumerate((9, 20, 14))]
        lens = (12, 5, 9)
        its = [sch.submit(p, GREEDY, max_tokens=k) for p, k in zip(prompts, lens)]
        got = [list(it) for it in its]
        for p, k, g in zip(prompts, lens, got):
            assert g == greedy_oracle(std, p, k)
    finally:
        sch.close()


def test_command_line_generates_token_ids(std, capsys):
    from ollama_operator_amd import cli
    prompt = gc.tokens(9, 96, seed=90)
    cli.main(["tokens", std.path, "--ids", " ".join(map(str, prompt)), "--num-predict", "5", "--device", "cpu",
              "--dtype", "float32"])
    out = capsys.readouterr().out.strip().splitlines()[-1]
    assert [int(t) for t in out.split()] == greedy_oracle(std, prompt, 5)


def test_trace_replay_program(std, tmp_path):
    """bin/trace_run on the CPU twin: a request that sits out a step, one that ends and gives its slot back."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b = gc.tokens(30, 96, seed=91), gc.tokens(12, 96, seed=92)
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
    gc.check(np.fromfile(out / "0.f32", "<f4").reshape(2, 96), wa[[0, 19]], "float32", "step 0")
    gc.check(np.fromfile(out / "1.f32", "<f4").reshape(1, 96), wb[[11]], "float32", "step 1")
    gc.check(np.fromfile(out / "2.f32", "<f4").reshape(1, 96), wa[[29]], "float32", "step 2")


# ------------------------------------------------------------------ the HIP executor against its twin
@pytest.mark.gpu
def test_gpu_matches_twin_layer_by_layer(std):
    toks = gc.tokens(50, 96, seed=95)
    for dtype, tol in (("float32", 1e-4), ("bfloat16", 0.05)):
        a = gc.layer_trail(std.runner("cpu", dtype), toks)
        b = gc.layer_trail(std.runner("cuda", dtype), toks)
        for i in range(a.shape[0]):
            assert np.abs(a[i] - b[i]).max() < tol * max(1.0, np.abs(a[i]).max()), f"{dtype}: layer run {i}"


@pytest.mark.gpu
@pytest.mark.parametrize("seed", [0, 1, 2, 3, 4, 5, 6, 7])
def test_random_configurations(tmp_path, seed):
    """Configurations drawn at the scale of a small real model, 300-token prompts in portions and whole, then single
    tokens: float32 sharply, bfloat16 by the typical row."""
    rng = random.Random(4000 + seed)
    cfg = gc.random_config(rng)
    m = gc.Model(tmp_path, cfg, seed=seed)
    toks = gc.tokens(300, cfg.n_vocab, seed=seed)
    want, _ = m.oracle(toks)
    cuts = [rng.randint(1, 100), rng.randint(101, 250), 290] + list(range(291, 301))
    gc.check(gc.run_cuts(m.runner("cuda", "float32", max_batch=512, kv_tokens=512), toks, cuts), want, "float32", f"configuration {seed}")
    r = m.runner("cuda", "bfloat16", max_batch=512, kv_tokens=512)
    e = gc.rel_err(gc.run_cuts(r, toks, cuts), want)
    assert np.isfinite(e).all() and np.median(e) < 0.05, f"configuration {seed}: typical row off by {np.median(e):.3g}"
