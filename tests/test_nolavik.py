"""Nolavik through the framework (config reader, checkpoint loader, engine, scheduler, paged cache, state slots, kernels)
against the plain float64 definition in nolavik_oracle.py. Every scenario runs on the CPU path in fp32 and, on a GPU box,
through the HIP kernels in fp32 and bf16. Small configurations made here, with sizes that differ between layers and values
that obvious choices would make equal or 1: grouped and single heads, value sizes unlike key sizes, odd sizes, one tap and
many, one expert and all of them chosen, with and without a shared expert and of another width, layers without a feed-forward,
repeated stretches at the start, in the middle and at the end, of one pass and of several, and no repetition at all."""
import json
import os

import numpy as np
import pytest
import torch

import nolavik_oracle as oracle
from llmss_amd.engine import LLMEngine, SamplingParams, build_model
from llmss_amd.models.config import ModelConfig
from llmss_amd.models.weights import nolavik_shapes, nolavik_state_dict

gpu = pytest.mark.gpu
RUNS = [pytest.param("cpu", "float32", id="cpu-fp32"), pytest.param("cuda", "float32", marks=gpu, id="gpu-fp32"),
        pytest.param("cuda", "bfloat16", marks=gpu, id="gpu-bf16")]


def moe(experts, top, ff, shared=0):
    d = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))
    if shared:
        d["shared"] = dict(ff=shared)
    return d


def delta(heads, kv, dim, vdim, conv, mlp=None):
    return dict(type="delta", mixer=dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv), mlp=mlp)


def par(left, right, scales, mlp=None):
    """left: heads, kv, dim, vdim, scale, rotated dims, base, scaling (factor, low, high, original); right: inner, state,
    dt_rank, taps."""
    H, G, dim, vdim, scale, rot, base, sc = left
    m = dict(heads=H, kv_heads=G, dim=dim, vdim=vdim, scale=scale)
    if rot:
        m["rot"] = dict(base=base, dims=rot)
        if sc:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), sc))
    return dict(type="parallel", mlp=mlp, mixer=dict(
        left=m, right=dict(zip(("inner", "state", "dt_rank", "conv"), right)), left_scale=scales[0], right_scale=scales[1]))


def lat(heads, dim, rd, vdim, q_rank, kv_rank, scale, base, mlp=None):
    return dict(type="latent_attention", mlp=mlp, mixer=dict(
        heads=heads, dim=dim, rot_dim=rd, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale, rot=dict(base=base, dims=rd)))


def model(vocab, width, eps, loop, layers):
    d = dict(architecture="Nolavik", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers)
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


CONFIGS = {
    # every mechanism, the repeated stretch in the middle, a layer without a feed-forward inside it
    "mixed": model(97, 48, 1e-5, (1, 4, 2), [
        lat(3, 8, 4, 12, 20, 24, 0.3, 500.0, mlp=moe(5, 2, 20, 12)),
        delta(4, 2, 8, 12, 4, mlp=moe(4, 1, 16)),
        par((4, 2, 12, 8, 1.5, 8, 300.0, (4.0, 1.0, 3.0, 40)), (40, 6, 5, 3), (0.7, 1.2)),
        lat(2, 16, 6, 8, 12, 10, 0.25, 90.0, mlp=moe(3, 3, 10, 24)),
        delta(3, 3, 6, 10, 2, mlp=moe(6, 2, 12, 8)),
    ]),
    # nothing optional: no repetition, one tap, no rotation on the attention branch, one expert
    "plain": model(61, 24, 1e-6, None, [
        delta(1, 1, 8, 8, 1, mlp=moe(1, 1, 10)),
        par((1, 1, 8, 8, 1.0, 0, 1.0, None), (16, 1, 1, 1), (1.0, 1.0), mlp=moe(3, 3, 10)),
        lat(1, 4, 2, 4, 8, 8, 0.5, 100.0),
    ]),
    # sizes the 16-byte paths and the matrix cores take; the stretch at the start, three passes
    "wide": model(83, 64, 1e-6, (0, 2, 3), [
        par((4, 1, 64, 32, 0.9, 32, 1000.0, (8.0, 1.0, 4.0, 100)), (96, 16, 8, 4), (0.8, 0.5), mlp=moe(8, 2, 32, 64)),
        delta(4, 2, 32, 64, 4, mlp=moe(4, 2, 48, 48)),
        lat(4, 32, 16, 32, 40, 48, 0.15, 10000.0, mlp=moe(5, 2, 32, 16)),
        delta(2, 2, 64, 64, 3),
    ]),
    # odd sizes everywhere, the stretch at the end, a single pass (whose vector is added all the same)
    "odd": model(51, 35, 1e-5, (1, 3, 1), [
        lat(5, 7, 6, 9, 11, 13, 0.4, 77.0, mlp=moe(7, 3, 9, 11)),
        par((6, 3, 10, 7, 2.0, 6, 20.0, None), (37, 9, 3, 6), (1.1, -0.6), mlp=moe(5, 4, 9)),
        delta(6, 2, 5, 7, 6, mlp=moe(3, 1, 7, 5)),
    ]),
    # one layer of each mixer alone, repeated
    "delta": model(43, 32, 1e-5, (0, 1, 4), [delta(2, 1, 16, 24, 3, mlp=moe(4, 2, 16, 8))]),
}


class Case:
    def __init__(self, name, tmp, device, dtype, seed=0):
        self.cfg = CONFIGS[name] if name in CONFIGS else BROAD
        mc = ModelConfig.from_hf_dict(self.cfg)
        self.sd = nolavik_state_dict(mc, seed=seed)
        if dtype == "bfloat16":
            # a close call of a router would send a token to another expert under bf16 rounding, and states and caches carry
            # that on: here the biases decide which experts are chosen, the token how they are weighted
            for n in self.sd:
                if n.endswith(".router"):
                    self.sd[n] = self.sd[n] * 0.25
                elif n.endswith(".router.b"):
                    g = torch.Generator().manual_seed(len(n) + int(n[1]))
                    self.sd[n] = (torch.randperm(self.sd[n].numel(), generator=g) * 1.5).to(torch.bfloat16)
        d = tmp / f"{name}-{seed}"
        d.mkdir(exist_ok=True)
        from safetensors.torch import save_file

        save_file({k: v.contiguous() for k, v in self.sd.items()}, str(d / "model.safetensors"))
        (d / "config.json").write_text(json.dumps(self.cfg))
        self.path, self.device, self.dtype = str(d), device, dtype
        self.model = build_model(self.path, dtype=dtype, device=device)
        self.V = self.cfg["vocab"]
        self._ref = {}

    bf16_limits = (4e-2, 0.4)

    def engine(self, tokens=512, slots=4, block=16, **kw):
        return LLMEngine(self.model, max_num_seqs=slots, block_size=block, num_blocks=-(-tokens // block),
                         max_model_len=tokens, max_batched_tokens=tokens, use_graphs=kw.pop("use_graphs", False),
                         autotune=False, **kw)

    def ref(self, tokens):
        key = tuple(tokens)
        if key not in self._ref:
            self._ref[key] = oracle.forward(self.cfg, self.sd, list(tokens)).float()
        return self._ref[key]

    def close(self, got, want, what=""):
        got, want = got.float().cpu(), want.float()
        d = (got - want) - (got - want).mean(-1, keepdim=True)
        err = d.pow(2).mean(-1).sqrt() / want.std(-1).clamp_min(1e-3)
        if self.dtype == "float32":
            assert float(err.max()) < 2e-4, f"{what}: relative error {float(err.max()):.3g} at row {int(err.argmax())}"
            return
        # (a head whose recurrence returns next to nothing - a first token whose key and query are nearly orthogonal - is
        # blown up by its norm, rounding and all: single rows may stand out)
        mid, top = self.bf16_limits
        assert float(err.median()) < (mid if len(err) >= 8 else 0.25) and float(err.max()) < top, \
            f"{what}: relative error median {float(err.median()):.3g}, max {float(err.max()):.3g} at row {int(err.argmax())}"


def toks(n, V, seed):
    return np.random.default_rng(seed).integers(0, V, n).tolist()


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("nolavik")
    made = {}

    def get(name, device, dtype):
        k = (name, device, dtype)
        if k not in made:
            made[k] = Case(name, tmp, device, dtype)
        return made[k]
    return get


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_every_position(cases, name, device, dtype):
    c = cases(name, device, dtype)
    t = toks(75, c.V, 1)  # more than a chunk of 64, five pages
    eng = c.engine()
    got = eng.replay_step([(0, t, list(range(len(t))))], end=[0])
    c.close(got, c.ref(t), "whole prompt")
    for n in (1, 2, 3):  # the first tokens of a sequence on their own, in the slot and pages the last request left
        got = eng.replay_step([(n, t[:n], list(range(n)))], end=[n])
        c.close(got, c.ref(t[:n]), f"first {n} token(s)")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_residual_stream_after_every_layer_run(cases, name, device, dtype):
    c = cases(name, device, dtype)
    t = toks(19, c.V, 2)
    want = []
    oracle.forward(c.cfg, c.sd, t, lambda r, x: want.append(x.clone()))
    assert len(want) == len(c.model.cfg.layer_runs())
    seen = {}
    c.model.tap = lambda i, x: seen.__setitem__(i, x.detach().float().cpu().clone())
    try:
        tapped = c.engine().replay_step([(0, t, [len(t) - 1])], end=[0])
    finally:
        c.model.tap = None
    assert sorted(seen) == list(range(len(want)))
    for i, w in enumerate(want):
        rel = (seen[i] - w.float()).abs().amax(-1) / w.abs().max()  # per token
        if dtype == "float32":
            assert float(rel.max()) < 2e-4, f"layer run {i}: {float(rel.max()):.3g}"
        else:
            assert float(rel.max()) < 0.06, f"layer run {i}: {[round(float(r), 3) for r in rel]}"
    # the tap takes the closing ops apart; fused they give the same row
    fused = c.engine().replay_step([(0, t, [len(t) - 1])], end=[0])
    assert float((fused - tapped).abs().max()) < (1e-4 if dtype == "float32" else 0.2)


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prefill_against_token_by_token_decoding(cases, name, device, dtype):
    c = cases(name, device, dtype)
    t = toks(40, c.V, 3)
    eng = c.engine()
    rows = [eng.replay_step([(0, [tok], [0])]) for tok in t]  # every token decoded alone, from position 0 on
    eng.replay_step([], end=[0])
    c.close(torch.cat(rows), c.ref(t), "token by token")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", ["mixed", "wide"])
@pytest.mark.parametrize("cuts", [(2, 2, 2, 3, 5, 16, 17, 2, 1, 1, 9), (15, 1, 16, 1, 17, 6), (33, 2, 21),
                                  (1, 2, 70, 2, 33, 1, 1, 30), (9, 1, 10, 10, 1, 19, 2)])
def test_portions_of_several_sizes(cases, cuts, name, device, dtype):
    # portions that end one before, at and one after the edges of pages (16) and chunks (64)
    c = cases(name, device, dtype)
    t = toks(sum(cuts), c.V, 4)
    eng = c.engine()
    got, at = [], 0
    for n in cuts:
        got.append(eng.replay_step([(7, t[at:at + n], list(range(n)))]))
        at += n
    eng.replay_step([], end=[7])
    c.close(torch.cat(got), c.ref(t), f"portions {cuts}")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", ["mixed", "plain", "odd", "wide"])
def test_mixed_batch_of_unequal_requests_equals_each_alone(cases, name, device, dtype):
    c = cases(name, device, dtype)
    seqs = {0: toks(50, c.V, 5), 1: toks(23, c.V, 6), 2: toks(9, c.V, 7), 3: toks(37, c.V, 8)}
    # per step: how many tokens of each request (0 = sits the step out); single tokens ride beside portions
    plan = [{0: 17, 1: 2}, {0: 1, 1: 5, 2: 9}, {0: 1, 1: 16, 3: 30}, {0: 31, 3: 1}, {3: 1, 1: 0}, {3: 5}]
    eng = c.engine(tokens=256)
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    for step in plan:
        entries, end = [], []
        for k, n in step.items():
            if n == 0:
                continue
            entries.append((k, seqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(seqs[k]):
                end.append(k)
        out = eng.replay_step(entries, end)
        r = 0
        for k, tk, _ in entries:
            got[k].append(out[r:r + len(tk)])
            r += len(tk)
    assert at == {k: len(v) for k, v in seqs.items()}
    for k, t in seqs.items():
        c.close(torch.cat(got[k]), c.ref(t), f"request {k} in the mixed batch")


@pytest.mark.parametrize("device,dtype", RUNS)
def test_pages_and_state_slots_are_used_again(cases, device, dtype):
    c = cases("mixed", device, dtype)
    eng = c.engine(tokens=64, slots=2, block=16)  # 4 pages, 2 sequences with their state slots
    assert eng.sched.num_free_blocks() == 4
    used = set()
    for r in range(6):  # every round takes the pages and slots that finished requests gave back
        a, b = toks(30 + r, c.V, 10 + r), toks(17, c.V, 20 + r)
        o1 = eng.replay_step([(2 * r, a[:20], [19]), (2 * r + 1, b, [16])], end=[2 * r + 1])
        used.add(eng.sched.state_slot(2 * r))
        assert eng.sched.num_free_blocks() == 2
        o2 = eng.replay_step([(2 * r, a[20:], list(range(len(a) - 20)))], end=[2 * r])
        assert eng.sched.num_free_blocks() == 4 and eng.sched.num_running() == 0
        c.close(o1, torch.stack([c.ref(a)[19], c.ref(b)[16]]), f"round {r}, first step")
        c.close(o2, c.ref(a)[20:], f"round {r}, second step")
    assert used <= {0, 1}
    with pytest.raises(RuntimeError):  # a third live request has no slot
        eng.replay_step([(100, [1], []), (101, [1], []), (102, [1], [])])
    assert eng.sched.num_free_blocks() == 4 and eng.sched.num_running() == 0


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_long_decoding_across_pages_and_chunks(cases, name, device, dtype):
    c = cases(name, device, dtype)
    t = toks(150, c.V, 30)
    eng = c.engine()
    got = [eng.replay_step([(0, t[:5], [4])])]
    got += [eng.replay_step([(0, [tok], [0])]) for tok in t[5:]]
    c.close(torch.cat(got), c.ref(t)[4:], "long decoding")


@pytest.mark.parametrize("device,dtype", RUNS)
def test_a_token_far_back_decides_the_logits(cases, device, dtype):
    """The latent attention's queries are made larger and the attention branch's scale is: single keys - the sequence's first, a
    page's first or last row - then carry a row's result, and one that is lost or doubled shows. Prompts and decoded tokens."""
    c = cases("mixed", device, dtype)
    sd = dict(c.sd)
    cfg = json.loads(json.dumps(c.cfg))
    for i, L in enumerate(cfg["layers"]):
        if L["type"] == "latent_attention":
            sd[f"l{i}.mix.uq"] = (sd[f"l{i}.mix.uq"].float() * 5).to(torch.bfloat16)
        elif L["type"] == "parallel":
            L["mixer"]["left"]["scale"] = 6.0
    sharp = Case.__new__(Case)
    sharp.__dict__.update(c.__dict__)
    sharp.cfg, sharp.sd, sharp._ref = cfg, sd, {}
    sharp.bf16_limits = (0.15, 0.5)  # scores several times larger: so is what their rounding does
    from llmss_amd.models.weights import _nolavik_finish

    mc = ModelConfig.from_hf_dict(cfg)
    sharp.model = type(c.model)(mc, _nolavik_finish(mc, lambda n: sd[n].float(), c.device, c.model.dtype))
    t = toks(230, c.V, 31)
    eng = sharp.engine()
    want = list(range(0, 200, 37)) + [15, 16, 17, 199]
    got = [eng.replay_step([(0, t[:200], want)])]
    got += [eng.replay_step([(0, [tok], [0])]) for tok in t[200:]]
    sharp.close(torch.cat(got), torch.cat([sharp.ref(t)[want], sharp.ref(t)[200:]]), "sharp attention")
    # the oracle itself: other first tokens change the last row by more than the tolerance
    moved = oracle.forward(cfg, sd, t[3:6] + t[3:])[-1].float() - sharp.ref(t)[-1]
    assert float(moved.std() / sharp.ref(t)[-1].std()) > 0.01


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_greedy_generation_through_the_engine(cases, name, device, dtype):
    c = cases(name, device, dtype)
    prompts = [toks(11, c.V, 40), toks(3, c.V, 41), toks(26, c.V, 42)]
    eng = LLMEngine(c.model, max_num_seqs=4, block_size=16, num_blocks=32, max_model_len=128, max_batched_tokens=24,
                    prefill_chunk=7, autotune=False)  # its own scheduler cuts the prompts and batches the decodes
    out = eng.generate(prompts, SamplingParams(max_new_tokens=12, is_greedy=True, ignore_eos=True))
    for p, o in zip(prompts, out):
        want = oracle.greedy(c.cfg, c.sd, p, 12)
        if dtype == "float32":
            assert o == want
        else:  # bf16 may flip a near-tie; the tokens before the first difference must then be a true near-tie
            k = next((i for i, (x, y) in enumerate(zip(o, want)) if x != y), None)
            if k is not None:
                lg = oracle.forward(c.cfg, c.sd, p + want[:k])[-1]
                assert float(lg[want[k]] - lg[o[k]]) < 0.1 * float(lg.std())


@pytest.mark.parametrize("device,dtype", RUNS)
def test_preempted_requests_start_over_from_an_empty_state(cases, device, dtype):
    """A pool too small for all requests: the scheduler preempts (pages and state slot go back) and recomputes."""
    c = cases("mixed", device, dtype)
    prompts = [toks(20, c.V, 80), toks(18, c.V, 81), toks(22, c.V, 82)]
    eng = LLMEngine(c.model, max_num_seqs=3, block_size=8, num_blocks=9, max_model_len=64, max_batched_tokens=32,
                    autotune=False)
    out = eng.generate(prompts, SamplingParams(max_new_tokens=14, is_greedy=True, ignore_eos=True))
    assert eng.stats["preemptions"] > 0
    if dtype == "float32":
        for p, o in zip(prompts, out):
            assert o == oracle.greedy(c.cfg, c.sd, p, 14)


def test_config_reader_rejects_what_the_design_does_not_have():
    def broken(name, edit):
        bad = json.loads(json.dumps(CONFIGS[name]))
        edit(bad)
        with pytest.raises(ValueError):
            ModelConfig.from_hf_dict(bad)
    broken("plain", lambda d: d["layers"][0].__setitem__("type", "convolution"))
    broken("mixed", lambda d: d["layers"][1]["mixer"].__setitem__("kv_heads", 3))
    broken("mixed", lambda d: d["layers"][2]["mixer"]["left"].__setitem__("kv_heads", 3))
    broken("mixed", lambda d: d["layers"][2]["mixer"]["left"]["rot"].__setitem__("dims", 14))  # more than the head holds
    broken("mixed", lambda d: d["layers"][0]["mixer"]["rot"].__setitem__("dims", 6))  # more than the rotated part
    broken("plain", lambda d: d["layers"][1]["mlp"]["router"].__setitem__("top", 4))  # more than there are experts
    broken("plain", lambda d: d["layers"][1]["mlp"].__setitem__("kind", "conv"))
    broken("mixed", lambda d: d["loop"].__setitem__("stop", 6))
    broken("mixed", lambda d: d["loop"].__setitem__("times", 0))
    broken("plain", lambda d: d.__setitem__("layers", []))


def test_config_reader_takes_every_size_and_constant_from_the_file():
    mc = ModelConfig.from_hf_dict(CONFIGS["mixed"])
    assert (mc.model_type, mc.vocab_size, mc.hidden_size, mc.norm_eps, mc.tie_word_embeddings, mc.loop, mc.loop_step) == \
        ("nolavik", 97, 48, 1e-5, False, (1, 4, 2), True)
    assert mc.layer_runs() == [0, 1, 2, 3, 1, 2, 3, 4]
    assert [mc.pass_before(r) for r in range(8)] == [None, 0, None, None, 1, None, None, None]
    a, b, p = (mc.layer_specs[i].mixer for i in (0, 1, 2))
    assert (a.kind, a.heads, a.dim, a.rot_dim, a.vdim, a.q_rank, a.kv_rank, a.scale, a.rot.dims, a.rot.base, a.gate, a.window) == \
        ("latent_attention", 3, 8, 4, 12, 20, 24, 0.3, 4, 500.0, False, 0)
    assert (b.kind, b.heads, b.kv_heads, b.dim, b.vdim, b.conv) == ("gated_delta", 4, 2, 8, 12, 4)
    lf, rt = p.left, p.right
    assert (p.kind, p.scales, lf.heads, lf.kv_heads, lf.dim, lf.vdim, lf.scale, lf.rot.dims, lf.rot.base, lf.rot.llama3, lf.unit_qk,
            lf.unit_sink, lf.window, lf.softcap) == \
        ("pair", (0.7, 1.2), 4, 2, 12, 8, 1.5, 8, 300.0, (4.0, 1.0, 3.0, 40.0), True, True, 0, 0.0)
    assert (rt.kind, rt.inner, rt.state, rt.dt_rank, rt.conv) == ("mamba", 40, 6, 5, 3)
    f = mc.layer_specs[0].mlp
    assert (f.kind, f.experts, f.top, f.expert.ff, f.shared.ff, f.act, f.score, f.bias, f.shared_gate, f.weight_input) == \
        ("moe", 5, 2, 20, 12, "silu", "chosen", True, True, False)
    assert mc.layer_specs[2].mlp is None and mc.layer_specs[1].mlp.shared is None and not mc.layer_specs[1].mlp.shared_gate
    plain = ModelConfig.from_hf_dict(CONFIGS["plain"])
    assert plain.loop is None and plain.layer_runs() == [0, 1, 2] and plain.layer_specs[1].mixer.left.rot is None
    assert "loop.step" not in nolavik_shapes(plain)
    odd = ModelConfig.from_hf_dict(CONFIGS["odd"])  # one pass: nothing repeats, its vector is still added
    assert odd.layer_runs() == [0, 1, 2] and [odd.pass_before(r) for r in range(3)] == [None, 0, None]
    assert nolavik_shapes(odd)["loop.step"] == (1, 35) and odd.layer_specs[1].mixer.left.rot.llama3 is None
    assert mc.num_params() == sum(int(np.prod(s)) for s in nolavik_shapes(mc).values())


def test_loader_checks_shapes_against_the_config(cases, tmp_path):
    c = cases("plain", "cpu", "float32")
    cfg = json.loads(json.dumps(c.cfg))
    cfg["layers"][1]["mixer"]["right"]["state"] = 2
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    os.symlink(os.path.join(c.path, "model.safetensors"), tmp_path / "model.safetensors")
    with pytest.raises(ValueError):
        build_model(str(tmp_path), dtype="float32", device="cpu")


def test_every_pass_has_a_cache_and_a_state_of_its_own(cases):
    c = cases("mixed", "cpu", "float32")
    kv = c.model.allocate_kv_cache(4, 16, num_slots=3)
    assert len(kv) == 8
    assert len({k[0].data_ptr() for k in kv if k[0] is not None}) == 5  # three latent runs, two attention branches
    assert kv[0][0].shape == (4, 16, 24 + 4) and kv[3][0].shape == kv[6][0].shape == (4, 16, 10 + 6)
    for r in (2, 5):
        assert kv[r][0].shape == (4, 16, 2 * 12) and kv[r][1].shape == (4, 16, 2 * 8)
        assert kv[r][2]["S"].shape == (3, 40, 6) and kv[r][2]["tail"].shape == (3, 2, 40)
    for r in (1, 4):
        assert kv[r][:2] == (None, None) and kv[r][2]["S"].shape == (3, 4, 8, 12)
        assert kv[r][2]["tail"].shape == (3, 3, 2 * 16 + 48)
    assert kv[1][2]["S"].data_ptr() != kv[4][2]["S"].data_ptr()
    assert c.model.kv_bytes_per_block(16) == 16 * 4 * (28 + 2 * 16 + 2 * 2 * (12 + 8))
    assert c.model.needs_state
    assert c.model.state_bytes_per_slot() == 4 * (2 * (4 * 96 + 3 * 80) + 2 * 40 * (6 + 2) + 3 * 60 + 1 * (36 + 30))


def test_trace_runner_replays_steps_on_the_cpu_path(cases, tmp_path):
    import subprocess
    import sys

    c = cases("odd", "cpu", "float32")
    t = toks(21, c.V, 50)
    steps = [dict(step=0, entries=[dict(id="a", tokens=t[:9], want=[0, 8])], end=[]),
             dict(step=1, entries=[dict(id="b", tokens=t[:2], want=[])], end=[]),
             dict(step=2, entries=[dict(id="a", tokens=t[9:], want=[11]), dict(id="b", tokens=t[2:3], want=[0])],
                  end=["a", "b"])]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", c.path, "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "64", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    g0 = torch.from_numpy(np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, c.V))
    g2 = torch.from_numpy(np.fromfile(tmp_path / "2.f32", dtype="<f4").reshape(2, c.V))
    c.close(g0, c.ref(t)[[0, 8]], "step 0")
    c.close(g2, torch.stack([c.ref(t)[20], c.ref(t[:3])[2]]), "step 2")


# A wider model than the others here, for the GPU: rows of hundreds of tokens, the 16-byte forms of the row kernels,
# the matrix-core projections and grouped expert products, the chunked recurrence over many chunks.
BROAD = model(600, 384, 1e-5, (1, 3, 2), [
    lat(6, 48, 16, 40, 136, 112, 0.12, 5000.0, mlp=moe(6, 2, 160, 192)),
    delta(6, 3, 64, 96, 4, mlp=moe(5, 3, 96)),
    par((6, 2, 48, 64, 0.5, 24, 20000.0, (8.0, 1.0, 4.0, 300)), (456, 20, 24, 4), (0.6, 0.9), mlp=moe(4, 1, 128, 64)),
    delta(2, 1, 128, 64, 2),
    lat(4, 32, 32, 64, 96, 96, 0.15, 300.0, mlp=moe(8, 2, 64, 320)),
])


@gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner_replays_long_requests_on_the_gpu(cases, tmp_path, dtype):
    """bin/trace_run as a user runs it, on the GPU in both precisions: a request of 400 tokens alone in portions of
    changing size and then token by token, then - in the pages and the slot it gave back - three requests side by
    side, portions of some beside single tokens of others. Every position's logits against the float64 definition."""
    import subprocess
    import sys

    c = cases("broad", "cuda", dtype)
    reqs = {"a": toks(400, c.V, 31), "b": toks(230, c.V, 32), "c": toks(130, c.V, 33), "d": toks(5, c.V, 34)}
    steps, at = [], {k: 0 for k in reqs}

    def feed(pairs):
        ent = []
        for k, n in pairs:
            ent.append(dict(id=k, tokens=reqs[k][at[k]:at[k] + n], want=list(range(n))))
            at[k] += n
        steps.append(dict(step=len(steps), entries=ent, end=[k for k, _ in pairs if at[k] == len(reqs[k])], rows=[
            (k, at[k] - n + j) for k, n in pairs for j in range(n)]))

    cuts = [100, 2, 133, 3, 33, 2, 17, 78, 64, 1, 1, 1, 37]
    i = 0
    while at["a"] < len(reqs["a"]):
        left = len(reqs["a"]) - at["a"]
        feed([("a", min(left, cuts[i % len(cuts)]) if left > 20 else 1)])
        i += 1
    pat = {"b": [150, 1, 60, 1, 1, 2], "c": [2, 1, 1, 30, 1], "d": [1, 1, 3]}
    i = 0
    while any(at[k] < len(reqs[k]) for k in pat):
        pairs = [(k, min(len(reqs[k]) - at[k], pat[k][i % len(pat[k])])) for k in pat
                 if at[k] < len(reqs[k]) and (i + ord(k)) % 5 != 4]
        if pairs:
            feed(pairs)
        i += 1
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", c.path, "--dtype", dtype,
                        "--out", str(tmp_path), "--max-tokens", "448"],
                       input="".join(json.dumps({k: v for k, v in s.items() if k != "rows"}) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert sum(ln.startswith("done") for ln in r.stdout.splitlines()) == len(steps)
    ref = {k: c.ref(v).double() for k, v in reqs.items()}
    every = torch.cat(list(ref.values()))
    spread = float((every - every.mean(-1, keepdim=True)).pow(2).mean().sqrt())
    errs = []
    for s in steps:
        got = torch.from_numpy(np.fromfile(tmp_path / f"{s['step']}.f32", dtype="<f4").reshape(-1, c.V)).double()
        want = torch.stack([ref[k][p] for k, p in s["rows"]])
        d = (got - want) - (got - want).mean(-1, keepdim=True)
        errs.append(d.pow(2).mean(-1).sqrt() / spread)
    errs = torch.cat(errs)
    if dtype == "float32":
        assert float(errs.max()) < 5e-5, f"row {int(errs.argmax())}: {float(errs.max()):.3g} of the logits' spread"
    else:  # bf16 products and activations: the model's own rounding noise
        assert float(errs.median()) < 0.02 and float(errs.max()) < 0.1, (float(errs.median()), float(errs.max()))


def test_registry_facade_runs_the_design(cases):
    """MODEL_REGISTRY["nolavik"](config, weights): HF-style calls with a growing paged past and a state slot."""
    from llmss_amd.models.registry import MODEL_REGISTRY, Weights
    from llmss_amd.utils.checkpoint import weight_files

    c = cases("mixed", "cpu", "float32")
    cfg = ModelConfig.from_pretrained(c.path)
    lm = MODEL_REGISTRY[cfg.model_type](cfg, Weights(weight_files(c.path), "cpu", torch.float32), max_blocks=16)
    t = toks(21, c.V, 60)
    out = lm(torch.tensor([t[:13]]), use_cache=True)
    c.close(out.logits[0], c.ref(t[:13]), "prompt through the facade")
    out2 = lm(torch.tensor([t[13:]]), past_key_values=out.past_key_values, use_cache=True)
    c.close(out2.logits[0], c.ref(t)[13:], "continuation through the facade")
    lm.release(out2.past_key_values)
    assert len(lm._free_state) == 16


def test_preset_builds_and_steps():
    m = build_model("tiny-nolavik", dtype="float32", device="cpu")
    eng = LLMEngine(m, max_num_seqs=2, block_size=16, num_blocks=8, max_model_len=64, max_batched_tokens=64,
                    autotune=False)
    out = eng.generate([[1, 2, 3]], SamplingParams(max_new_tokens=4, is_greedy=True, ignore_eos=True))
    assert len(out[0]) == 4


@gpu
def test_decode_graphs_and_autotuned_projections_decode_right(cases):
    """Serving defaults on a GPU: GEMM plans timed per decode bucket, decode steps replayed from captured graphs
    (state slots ride in the graphs' static buffers), pipelined decode."""
    c = cases("wide", "cuda", "bfloat16")
    assert c.model.gemm_shapes()
    eng = LLMEngine(c.model, max_num_seqs=4, block_size=16, num_blocks=32, max_model_len=96, max_batched_tokens=64)
    assert eng.graphs
    prompts = [toks(9, c.V, 70), toks(17, c.V, 71), toks(2, c.V, 72)]
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=10, is_greedy=True, ignore_eos=True))
    for p, out in zip(prompts, outs):
        want = oracle.greedy(c.cfg, c.sd, p, 10)
        k = next((i for i, (x, y) in enumerate(zip(out, want)) if x != y), None)
        if k is not None:
            lg = oracle.forward(c.cfg, c.sd, p + want[:k])[-1]
            assert float(lg[want[k]] - lg[out[k]]) < 0.1 * float(lg.std())


@gpu
def test_fp32_decode_graphs_reproduce_the_oracle_exactly(cases):
    c = cases("mixed", "cuda", "float32")
    eng = LLMEngine(c.model, max_num_seqs=4, block_size=16, num_blocks=32, max_model_len=96, max_batched_tokens=64,
                    autotune=False)
    assert eng.graphs
    prompts = [toks(9, c.V, 73), toks(30, c.V, 74), toks(1, c.V, 75)]
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=20, is_greedy=True, ignore_eos=True))
    for p, out in zip(prompts, outs):
        assert out == oracle.greedy(c.cfg, c.sd, p, 20)
