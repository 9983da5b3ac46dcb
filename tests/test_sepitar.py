"""Sepitar (looped layered decoder of parallel blocks: attention with a bucketed distance bias, soft-capped attention with a
sink, latent attention with a sink, routed clamped units) against the plain oracle of tests/sepitar_oracle.py.

Small configurations with random weights made here; the framework side always runs through the engine
(scheduler admission, pages, runner) or the ops' public entry points.  CPU tensors exercise the ops' PyTorch forms,
``cuda`` ones the HIP kernels (marked gpu).
"""
import copy
import math

import numpy as np
import pytest
import torch

import sepitar_oracle as oracle
from financial_chatbot_llm_amd.config import EngineConfig
from financial_chatbot_llm_amd.engine import LLMEngine, SamplingParams
from financial_chatbot_llm_amd.models.configs import layered_config
from financial_chatbot_llm_amd.models.layered import layer_runs
from financial_chatbot_llm_amd.models.mixers import RoutedFF
from financial_chatbot_llm_amd.models.sepitar import SepitarModel, example_config
from financial_chatbot_llm_amd.ops import mixers as mx

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 3e-4, torch.bfloat16: 8e-2}


def random_weights(model, seed):
    g = torch.Generator().manual_seed(seed)
    sd = {}
    for name, shape in model.full_shapes().items():
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g)
        if leaf == "norm1" or name == "final.norm":          # stored around zero
            t = 0.2 * r
        elif leaf == "norm":
            t = 1.0 + 0.2 * r
        elif leaf == "b":
            t = 0.2 * r
        elif leaf in ("sink", "embed"):
            t = r
        elif leaf == "rel":
            t = 1.5 * r
        else:
            t = r * shape[-1] ** -0.5 * 1.5
        sd[name] = t.to(torch.bfloat16)
    return sd


def small_config(pattern="LRC", loop=(0, 2, 2), **over):
    return example_config(width=over.pop("width", 96), vocab=over.pop("vocab", 168), pattern=pattern, loop=loop)


def build(cfgd, device, dtype, seed=1, blocks_=24, seqs=4, graphs=False, async_=False, max_len=1024, prefix=False, sd=None):
    mc = layered_config(cfgd, "sepitar-test")
    model = SepitarModel(mc, device=device, dtype=dtype)
    sd = sd if sd is not None else random_weights(model, seed)
    model.load_state(sd)
    eng = LLMEngine(EngineConfig(model="sepitar-test", device=device, dtype="fp32" if dtype == torch.float32 else "bf16",
                                 num_kv_blocks=blocks_, max_num_seqs=seqs, max_model_len=max_len,
                                 max_num_batched_tokens=512, enable_prefix_caching=prefix, use_cuda_graph=graphs,
                                 async_scheduling=async_, graph_batch_sizes=(1, 2, 4)), model=model)
    return eng, sd


def poison(eng):
    """Pages as a previous owner might have left them: nothing may depend on their content."""
    for lay in eng.kv.layers:
        lay[1].fill_(float("nan"))


def close(got, want, dtype, routed=False):
    """``routed``: in bf16 a router's near-tie may fall the other way at a few positions."""
    got, want = torch.as_tensor(got).double().cpu(), torch.as_tensor(want).double()
    assert torch.isfinite(got).all()
    err = (got - want).abs().flatten(1).max(-1).values / max(want.abs().max().item(), 1e-9)
    over = int((err > TOL[dtype]).sum())
    allowed = 0.05 * err.numel() if routed and dtype == torch.bfloat16 else 0
    assert over <= allowed, f"{over} of {err.numel()} positions over: worst {err.max():.3e}"


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def run_whole(eng, rid, toks):
    return eng.replay_step([(rid, toks, list(range(len(toks))))], [rid])


def i32(x, device="cpu"):
    return torch.tensor(x, dtype=torch.int32, device=device)


# ---------------------------------------------------------------------------------------------------
# whole models, layer kinds, loops, sizes
# ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("pattern", ["l", "r", "c", "L", "R", "C", "LRC", "cRlCLr"])
def test_layer_kinds_against_oracle(device, dtype, pattern):
    """Each mixer alone, with the routed feed-forward beside it, and mixes in other orders, no loop."""
    cfgd = small_config(pattern, loop=None)
    eng, sd = build(cfgd, device, dtype)
    poison(eng)
    toks = tokens(90, cfgd["vocab"], 3)          # crosses a 64-token page and leaves the 21- and 37-token windows
    close(run_whole(eng, "r", toks), oracle.forward(cfgd, sd, toks), dtype, routed=pattern != pattern.lower())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("loop", [(0, 3, 2), (1, 2, 3), (1, 3, 2), (0, 1, 4), (2, 3, 2), (0, 3, 1), None])
def test_loops(device, loop):
    """Spans at the start, in the middle, at the end and over the whole model, one to four passes; prompt portions and
    decoded tokens (each pass reads its own rows), the residual stream after every layer run."""
    cfgd = small_config("LRC", loop=loop)
    eng, sd = build(cfgd, device, torch.float32)
    n_runs = 3 if loop is None else 3 + (loop[2] - 1) * (loop[1] - loop[0])
    assert len(eng.kv.layers) == n_runs
    poison(eng)
    toks = tokens(80, cfgd["vocab"], 4)
    layers = []
    want = oracle.forward(cfgd, sd, toks, layers)
    got = [eng.replay_step([("r", toks[a:b], list(range(b - a)))], ["r"] if b == 80 else [])
           for a, b in ((0, 41), (41, 43), (43, 70), *((i, i + 1) for i in range(70, 80)))]
    close(torch.cat(got), want, torch.float32)
    eng.model.capture = []
    close(run_whole(eng, "again", toks), want, torch.float32)
    assert len(eng.model.capture) == len(layers) == n_runs
    for x, ref in zip(eng.model.capture, layers):
        close(x, ref, torch.float32)


def test_loop_faults_show():
    """The mistakes are planted in the oracle's configuration: a pass too few, and a loop one layer off, change the
    logits far beyond the tolerance."""
    cfgd = small_config("LRC", loop=(0, 2, 2))
    eng, sd = build(cfgd, "cpu", torch.float32)
    toks = tokens(40, cfgd["vocab"], 5)
    got = run_whole(eng, "r", toks).double().numpy()
    for bad in ({"start": 0, "stop": 2, "times": 1}, {"start": 1, "stop": 3, "times": 2}):
        assert np.abs(got - oracle.forward({**cfgd, "loop": bad}, sd, toks)).max() > 0.1


def test_layer_order():
    assert [r.layer for r in layer_runs(4)] == [0, 1, 2, 3]
    runs = layer_runs(4, {"start": 1, "stop": 3, "times": 3})
    assert [r.layer for r in runs] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [i for i, r in enumerate(runs) if r.again] == [3, 5]
    assert [i for i, r in enumerate(layer_runs(2, {"start": 0, "stop": 1, "times": 2})) if r.again] == [1]
    for bad in ({"start": 2, "stop": 2, "times": 2}, {"start": 0, "stop": 5, "times": 2}, {"start": 0, "stop": 2, "times": 0}):
        with pytest.raises(ValueError):
            layer_runs(4, bad)


@pytest.mark.parametrize("device", DEVICES)
def test_absent_entries_and_single_sizes(device):
    """No mask, no cap, no rotation, no scaling, no shared expert, one expert, one head, as many key/value heads as
    heads (also by an absent entry), a window of one key, a bias table of two rows, scales of 0 and 1, sizes that only a
    tensor gives, a loop over layers without a feed-forward."""
    cfgd = small_config("lrcLRC", loop=(0, 3, 2))
    L = cfgd["layers"]
    del L[0]["mixer"]["mask"], L[0]["mixer"]["rot"]["scaling"]
    L[0]["mixer"].update(heads=1)
    del L[1]["mixer"]["mask"], L[1]["mixer"]["kv_heads"]
    L[1]["mixer"].update(buckets=2, bias_max=4, scale=0.0)
    del L[2]["mixer"]["softcap"], L[2]["mixer"]["rot"]
    L[2]["mixer"].update(heads=1, kv_heads=1, mask={"size": 5})
    L[3]["mixer"].update(mask={"size": 1})
    del L[3]["mlp"]["shared"]
    L[3]["mlp"]["router"].update(experts=1, top=1)
    L[4]["mixer"].update(mask={"size": 1}, kv_heads=1, scale=1.0)
    L[4]["mlp"]["router"].update(top=7)
    del L[5]["mixer"]["rot"]["scaling"]
    L[5]["mixer"].update(kv_heads=4, scale=1.0)
    sd = random_weights(SepitarModel(layered_config(cfgd, "t"), device="cpu"), 6)
    assert "l0.mlp.router" not in sd and "l3.mlp.shared.up" not in sd and sd["l1.mix.rel"].shape == (2, 6)
    for l in L:
        l["mixer"].pop("buckets", None)                # the tensor gives it
    eng, _ = build(cfgd, device, torch.float32, sd=sd)
    poison(eng)
    toks = tokens(90, cfgd["vocab"], 5)
    close(run_whole(eng, "r", toks), oracle.forward(cfgd, sd, toks), torch.float32)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_other_sizes(device, dtype):
    """Sizes unlike the small default: odd head counts, key and value sizes that fill no wave and differ, rotated
    parts of a head, ranks that are no multiple of anything, windows longer than a page and very short ones, bias
    tables of odd and large row counts, expert widths of 1, 9 and 133, 70 experts top 5, a width that is no multiple of
    the wide accesses, a large norm eps, other constants."""
    cfgd = small_config("LRCLRC", loop=(1, 4, 2), width=82, vocab=97)
    cfgd["norm"]["eps"] = 0.02
    L = cfgd["layers"]
    L[0]["mixer"].update(dim=13, heads=5, kv_rank=35, q_rank=9, rot_dim=6, vdim=7, scale=0.31, mask={"size": 70},
                         rot={"base": 50.0, "dims": 6, "scaling": {"factor": 1.7, "fast": 3.0, "original": 40, "slow": 0.3}})
    L[1]["mixer"].update(dim=9, heads=6, kv_heads=3, vdim=33, bias_max=64, buckets=7, mask={"size": 65}, scale=0.4)
    L[2]["mixer"].update(dim=34, heads=6, kv_heads=2, vdim=17, softcap=1.3, scale=0.6,
                         rot={"base": 77.0, "dims": 6, "scaling": {"factor": 2.5, "high": 3.0, "low": 1.0, "original": 30}})
    L[3]["mixer"].update(dim=64, heads=2, kv_rank=136, q_rank=100, rot_dim=16, vdim=48, scale=0.1, mask={"size": 3},
                         rot={"base": 500.0, "dims": 16, "scaling": {"factor": 8.0, "fast": 2.0, "original": 700, "slow": 1.9}})
    L[4]["mixer"].update(dim=132, heads=5, kv_heads=5, vdim=20, bias_max=91.5, buckets=40, mask={"size": 130}, scale=0.07)
    L[5]["mixer"].update(dim=48, heads=12, kv_heads=4, vdim=136, softcap=50.0, scale=0.15, mask={"size": 64},
                         rot={"base": 10.0, "dims": 48, "scaling": {"factor": 3.0, "high": 8.0, "low": 2.0, "original": 500}})
    L[0]["mlp"].update(router={"experts": 70, "top": 5}, expert={"ff": 9, "limit": 2.2})
    L[1]["mlp"].update(router={"experts": 3, "top": 1}, expert={"ff": 133, "limit": 0.3})
    L[1]["mlp"]["shared"].update(ff=1, limit=3.0)
    L[2]["mlp"].update(router={"experts": 2, "top": 2}, expert={"ff": 1, "limit": 10.0})
    L[3]["mlp"]["shared"].update(ff=50, limit=0.4)
    eng, sd = build(cfgd, device, dtype, blocks_=8)
    poison(eng)
    toks = tokens(150, cfgd["vocab"], 7)
    close(run_whole(eng, "r", toks), oracle.forward(cfgd, sd, toks), dtype, routed=True)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_wide_heads(device, dtype):
    """Head sizes and ranks beyond what the matrix-core attention covers (bf16 then takes the f32-lane kernels), even
    and odd."""
    cfgd = small_config("lrcl", width=64, loop=(0, 2, 2))
    L = cfgd["layers"]
    L[0]["mixer"].update(heads=2, kv_rank=300, rot_dim=40, scale=0.05, rot={"base": 100.0, "dims": 40})
    L[1]["mixer"].update(dim=264, vdim=300, heads=2, kv_heads=1, scale=0.06)
    L[2]["mixer"].update(dim=261, vdim=41, heads=2, kv_heads=2, scale=0.05)
    L[3]["mixer"].update(heads=2, kv_rank=259, scale=0.05)
    eng, sd = build(cfgd, device, dtype, blocks_=4)
    toks = tokens(80, cfgd["vocab"], 8)
    close(run_whole(eng, "r", toks), oracle.forward(cfgd, sd, toks), dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(device):
    """Sequences of one and two tokens, and the first tokens of a longer one, each request alone."""
    cfgd = small_config("LRC")
    eng, sd = build(cfgd, device, torch.float32)
    poison(eng)
    for n in (1, 2, 5):
        toks = tokens(n, cfgd["vocab"], 60 + n)
        close(run_whole(eng, f"r{n}", toks), oracle.forward(cfgd, sd, toks), torch.float32)


def test_norms_are_stored_around_zero():
    """Zero norm weights are norms without a weight; the random initialisation follows."""
    cfgd = small_config("LRC")
    eng, sd = build(cfgd, "cpu", torch.float32)
    m = eng.model
    for n in ("l0.norm1", "l2.norm1", "final.norm"):
        sd[n] = torch.zeros_like(sd[n])
    m.load_state(sd)
    assert (m.layers[0].norm1 == 1).all() and (m.final_norm == 1).all()
    m.init_random(seed=3)
    assert abs(m.final_norm.mean() - 1) < 0.1 and abs(m.layers[1].norm1.mean() - 1) < 0.1


# ---------------------------------------------------------------------------------------------------
# cache, batching
# ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_prefill_then_token_by_token(device, dtype):
    cfgd = small_config("LRC", loop=(1, 3, 2))
    eng, sd = build(cfgd, device, dtype)
    poison(eng)
    toks = tokens(140, cfgd["vocab"], 11)
    want = oracle.forward(cfgd, sd, toks)
    got = [eng.replay_step([("r", toks[:30], list(range(30)))])]
    for i in range(30, len(toks)):               # long decoding: the windows pass over decoded tokens and page borders
        got.append(eng.replay_step([("r", toks[i:i + 1], [0])], ["r"] if i == len(toks) - 1 else []))
    close(torch.cat(got), want, dtype, routed=True)
    assert eng.bm.num_free() == eng.bm.num_blocks and eng.state_slots is None


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("sizes", [[2, 2, 3, 60, 2, 1, 1, 64, 5], [63, 1, 1, 2, 70], [1, 1, 1, 130], [2] * 20, [20, 2, 15, 2, 37]])
def test_portions(device, sizes):
    """Portions cut inside pages and inside windows, down to two tokens."""
    cfgd = small_config("LRC")
    eng, sd = build(cfgd, device, torch.float32)
    poison(eng)
    toks = tokens(sum(sizes), cfgd["vocab"], 13)
    want = oracle.forward(cfgd, sd, toks)
    got, at = [], 0
    for n in sizes:
        got.append(eng.replay_step([("r", toks[at:at + n], list(range(n)))]))
        at += n
    close(torch.cat(got), want, torch.float32)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_and_reuse(device, dtype):
    """Unequal requests in one batch (portions beside single tokens) and a pool that only fits what is live: pages
    are freed and used again."""
    cfgd = small_config("LRC")
    eng, sd = build(cfgd, device, dtype, blocks_=7, seqs=3)
    poison(eng)
    V = cfgd["vocab"]
    reqs = {f"q{i}": tokens(n, V, 20 + i) for i, n in enumerate([150, 70, 33, 100, 5, 64])}
    want = {k: torch.as_tensor(oracle.forward(cfgd, sd, t)) for k, t in reqs.items()}
    got = {k: [] for k in reqs}
    at = {k: 0 for k in reqs}
    sched = [
        [("q0", 50), ("q1", 3), ("q2", 33)],            # q2 complete at once
        [("q0", 1), ("q1", 60), ("q3", 2)],             # q3 takes q2's pages
        [("q0", 30), ("q1", 1), ("q3", 62)],
        [("q1", 1), ("q0", 69), ("q3", 1)],
        [("q1", 5), ("q3", 35)],                        # q1, q3, q0 complete
        [("q4", 5), ("q5", 2)],
        [("q5", 62)],
    ]
    for step in sched:
        entries, end = [], []
        for k, n in step:
            entries.append((k, reqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                end.append(k)
        out = eng.replay_step(entries, end)
        o = 0
        for k, t, _ in entries:
            got[k].append(out[o:o + len(t)])
            o += len(t)
    assert all(at[k] == len(reqs[k]) for k in reqs) and eng.bm.num_free() == eng.bm.num_blocks
    close(torch.cat([torch.cat(got[k]) for k in reqs]), torch.cat([want[k] for k in reqs]), dtype, routed=True)


@pytest.mark.parametrize("device", DEVICES)
def test_batch_rows_do_not_depend_on_their_neighbours(device):
    """The same request alone and between two others gives the same logits (f32)."""
    cfgd = small_config("LRC")
    eng, sd = build(cfgd, device, torch.float32)
    V = cfgd["vocab"]
    a, b, c = tokens(45, V, 1), tokens(20, V, 2), tokens(70, V, 3)
    alone = run_whole(eng, "x", b)
    poison(eng)
    out = eng.replay_step([("a", a, []), ("b", b, list(range(len(b)))), ("c", c, [])], ["a", "b", "c"])
    assert (out - alone).abs().max() <= 4e-6 * alone.abs().max()


# ---------------------------------------------------------------------------------------------------
# mechanisms alone, with inputs in which a fault stands out
# ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W", [(3, 8), (70, 132), (5, 7), (33, 516), (4, 2056), (2, 4100), (2, 8196)])
def test_residual_update_with_embedding_rows(device, dtype, T, W):
    """The stream's start from the table, the update with two outputs (column slices), the table's row on top, the
    norm: against numpy in f64; ids outside the vocabulary are clamped; each part alone."""
    g = torch.Generator().manual_seed(W)
    table = torch.randn(11, W, generator=g).to(dtype)
    ids = torch.randint(0, 11, (T,), generator=g)
    w = torch.randn(W, generator=g)
    pad = 4 if W % 4 == 0 else 3
    buf = torch.randn(T, 2 * W + pad, generator=g).to(dtype)
    bd = buf.to(device)
    a, b = bd[:, pad:pad + W], bd[:, pad + W:]
    tol = 5e-6 if dtype == torch.float32 else 4e-2
    e = table.double().numpy()[ids.numpy()]
    norm = lambda x: oracle.rms(x, 1e-3) * w.double().numpy()  # noqa: E731
    x, h = mx.embed_norm(ids.to(device), table.to(device), w.to(device), 1e-3, dtype)
    assert np.array_equal(x.double().cpu().numpy(), e) and h.dtype == dtype
    assert np.abs(h.double().cpu().numpy() - norm(e)).max() < tol * max(1.0, np.abs(norm(e)).max())
    x0 = torch.randn(T, W, generator=g)
    for with_a, with_b, with_e in ((1, 1, 1), (1, 0, 1), (0, 0, 1), (1, 1, 0), (0, 1, 0)):
        xd = x0.clone().to(device)
        h = mx.residual_norm(xd, w.to(device), 1e-3, a if with_a else None, b if with_b else None, out_dtype=dtype,
                             ids=ids.to(device) if with_e else None, table=table.to(device) if with_e else None)
        want = x0.double().numpy() + with_a * buf[:, pad:pad + W].double().numpy() \
            + with_b * buf[:, pad + W:].double().numpy() + with_e * e
        assert np.abs(xd.double().cpu().numpy() - want).max() < 3e-6
        assert np.abs(h.double().cpu().numpy() - norm(want)).max() < tol * max(1.0, np.abs(norm(want)).max())
    xd = x0.clone().to(device)
    assert mx.residual_norm(xd, None, 1e-3, a, b) is None                        # the update alone
    far = mx.embed_norm(i32([-5, 99], device), table.to(device), w.to(device), 1e-3, dtype)[0].cpu()
    assert torch.equal(far, table[[0, 10]].float())
    with pytest.raises(ValueError):
        mx.residual_norm(xd, None, 1e-3, a, b, ids=ids[:1].to(device), table=table.to(device))


def test_frequency_scaling():
    """Both scalings against the oracle's formulas; pairs on either side of both wavelength limits; a factor of one."""
    for base, dims, sc in ((1000.0, 24, {"factor": 5.0, "high": 6.0, "low": 1.5, "original": 96}),
                           (5e5, 128, {"factor": 8.0, "high": 4.0, "low": 1.0, "original": 8192}),
                           (20.0, 6, {"factor": 1.0, "high": 2.0, "low": 1.0, "original": 64}), (77.0, 10, None)):
        rot = {"base": base, "dims": dims, "scaling": sc}
        f, m = mx.rope_freqs(dims, base, sc)
        want = oracle.wavelength_freqs(rot)
        assert m == 1.0 and np.abs(f.double().numpy() - want).max() < 1e-6 * want.max()
        if sc and sc["factor"] > 1 and dims >= 24:
            r = want / oracle.base_freqs(rot)
            assert np.isclose(r, 1).any() and np.isclose(r, 1 / sc["factor"]).any()
            assert ((r < 0.999) & (r > 1.001 / sc["factor"])).any()
    for base, dims, sc in ((1e4, 8, {"factor": 3.0, "fast": 8.0, "original": 128, "slow": 0.5}),
                           (5e3, 64, {"factor": 16.0, "fast": 32.0, "original": 4096, "slow": 1.0}),
                           (10.0, 16, {"factor": 2.0, "fast": 1.0, "original": 64, "slow": 0.999})):
        rot = {"base": base, "dims": dims, "scaling": sc}
        f, m = mx.rope_freqs(dims, base, sc)
        want, wm = oracle.ramp_freqs(rot)
        assert abs(m - wm) < 1e-12 and wm > 1 and np.abs(f.double().numpy() / want - 1).max() < 1e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,P,rot,layout", [(4, 2, 32, 28, 24, "half"), (3, 3, 64, 16, 64, "half"), (5, 1, 9, 7, 6, "half"),
                                                (2, 2, 128, 128, 128, "half"), (6, 2, 24, 8, 8, "pairs"), (4, 1, 40, 16, 16, "half"),
                                                (3, 1, 10, 4, 2, "half")])
def test_norm_rotation_and_cache_rows(device, dtype, H, G, D, P, rot, layout):
    """Norms over whole projections and the rotation in one pass: queries returned, keys and values in scattered cache
    rows, a row that is not cached, positions far into a sequence, column slices; each part without the other."""
    T, eps = 37, 1e-3
    g = torch.Generator().manual_seed(D)
    nq, nk, nv = H * D, G * D, G * P
    off = 8 if D % 8 == 0 else 3
    buf = torch.randn(T, off + nq + nk + nv, generator=g).to(dtype)
    qw, kw = 1 + 0.3 * torch.randn(nq, generator=g), 1 + 0.3 * torch.randn(nk, generator=g)
    pos = torch.randint(0, 3000, (T,), generator=g)
    pos[0] = 0
    freq, _ = mx.rope_freqs(rot, 100.0)
    rows = torch.randperm(T + 9, generator=g)[:T].tolist()
    rows[5] = -1
    bd = buf.to(device)
    q, k, v = bd[:, off:off + nq], bd[:, off + nq:off + nq + nk], bd[:, off + nq + nk:]
    ref = buf.double().numpy()[:, off:]

    def turned(x, n, m):
        x = x.reshape(T, n, D)
        a = pos.numpy()[:, None, None] * freq.double().numpy()
        c, s, y = m * np.cos(a), m * np.sin(a), x.copy()
        u, w = (x[..., :rot // 2], x[..., rot // 2:rot]) if layout == "half" else (x[..., 0:rot:2], x[..., 1:rot:2])
        ru, rw = u * c - w * s, w * c + u * s
        if layout == "half":
            y[..., :rot // 2], y[..., rot // 2:rot] = ru, rw
        else:
            y[..., 0:rot:2], y[..., 1:rot:2] = ru, rw
        return y.reshape(T, n * D)

    for norm in (True, False):
        for turn in (True, False):
            cache = torch.full((T + 9, nk + nv), 7.0, dtype=dtype, device=device)
            out = mx.qk_norm_write(q, k, v, qw.to(device) if norm else None, kw.to(device) if norm else None, eps,
                                   i32(rows, device), cache, dim=D, freq=freq.to(device) if turn else None,
                                   pos=pos.to(torch.int32).to(device), layout=layout, mscale=1.2).double().cpu().numpy()
            qr, kr = ref[:, :nq], ref[:, nq:nq + nk]
            if norm:
                qr, kr = oracle.rms(qr, eps) * qw.double().numpy(), oracle.rms(kr, eps) * kw.double().numpy()
            if turn:
                qr, kr = turned(qr, H, 1.2), turned(kr, G, 1.2)
            tol = 1.5e-3 if dtype == torch.float32 else 4e-2          # f32 angles at position 3000
            assert np.abs(out - qr).max() < tol * max(1.0, np.abs(qr).max())
            c = cache.double().cpu().numpy()
            for t in range(T):
                if rows[t] >= 0:
                    want = np.concatenate([kr[t], ref[t, nq + nk:]])
                    assert np.abs(c[rows[t]] - want).max() < tol * max(1.0, np.abs(want).max()), t
            unused = [r for r in range(T + 9) if r not in rows]
            assert (c[unused] == 7.0).all()
    if layout == "half":
        with pytest.raises(ValueError):
            mx.qk_norm_write(q, k, v, None, None, eps, i32(rows, device), cache, dim=D + 1, freq=freq.to(device),
                             pos=pos.to(torch.int32).to(device))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R,Dr,rot,m", [(40, 8, 8, 1.11), (33, 6, 4, 1.0), (128, 64, 64, 1.3), (7, 2, 2, 1.5)])
def test_latent_rows(device, dtype, R, Dr, rot, m):
    """The normed latent and the rotated shared key part in the cache row, every head's rotated query part, cos and
    sin times a factor; the rest of a partly rotated part passes unscaled."""
    T, H, dn, eps = 19, 3, 5, 1e-2
    g = torch.Generator().manual_seed(R)
    kv = torch.randn(T, R + Dr, generator=g).to(dtype)
    q = torch.randn(T, H * (dn + Dr), generator=g).to(dtype)
    w = 1 + 0.3 * torch.randn(R, generator=g)
    freq, _ = mx.rope_freqs(rot, 60.0)
    start = 100
    cache = torch.zeros(T + 3, R + Dr, dtype=dtype, device=device)
    rows = torch.randperm(T + 3, generator=g)[:T].tolist()
    qr = mx.latent_prep(kv.to(device), w.to(device), eps, freq.to(device), rot, i32(list(range(start, start + T)), device),
                        i32(rows, device), cache, q.to(device), H, dn + Dr, dn, R, Dr, m).double().cpu().numpy()
    pad = lambda x: np.concatenate([np.zeros((start,) + x.shape[1:]), x])  # noqa: E731
    f = freq.double().numpy()
    kvn, qn = kv.double().numpy(), q.double().numpy().reshape(T, H, dn + Dr)
    want_q = oracle.rotate_pairs(pad(qn[..., dn:]), f, m)[start:]
    want_k = oracle.rotate_pairs(pad(kvn[:, None, R:]), f, m)[start:, 0]
    want_c = oracle.rms(kvn[:, :R], eps) * w.double().numpy()
    tol = 5e-5 if dtype == torch.float32 else 4e-2
    assert np.abs(qr - want_q).max() < tol
    got = cache.double().cpu().numpy()[rows]
    assert np.abs(got - np.concatenate([want_c, want_k], 1)).max() < tol


@pytest.mark.parametrize("rows,far", [(2, 5), (12, 30), (16, 128), (7, 60), (32, 1024), (40, 91.5), (4, 2.5)])
def test_distance_buckets(rows, far):
    """The table of buckets against the formula, also where a step falls on a whole distance; the last entry is the
    first distance of the last row."""
    b = mx.distance_buckets(rows, far).tolist()
    assert all(oracle.bucket(n, rows, far) == b[min(n, len(b) - 1)] for n in range(3000))
    assert b[0] == 0 and b[-1] == rows - 1 and (len(b) == 1 or b[-2] < rows - 1) and b == sorted(b)
    with pytest.raises(ValueError):
        mx.distance_buckets(rows, rows // 2)


def _paged_rows(rows, table):
    """Cache of the rows of positions 0.. under the page table; rows the sequence has not reached hold leftovers."""
    cache = torch.full((table.shape[1] * 64, rows.shape[1]), 3.0, dtype=rows.dtype)
    for j in range(rows.shape[0]):
        cache[int(table[0, j // 64]) * 64 + j % 64] = rows[j]
    return cache


def _segments(n):
    return (list(range(n // 2, n // 2 + 50)), list(range(9)), list(range(62, 67)), [n - 1], [64], [63], [0], [1])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,P,size,B,far", [(6, 2, 16, 12, 37, 12, 30), (4, 4, 24, 8, 64, 7, 64), (5, 1, 9, 7, 1 << 30, 16, 128),
                                                (12, 3, 40, 33, 130, 40, 91.5), (2, 1, 64, 272, 90, 12, 30),
                                                (32, 1, 16, 16, 900, 32, 1024), (3, 1, 136, 136, 100, 5, 70)])
def test_attention_distance_bias(device, dtype, H, G, D, P, size, B, far):
    """Distance bias and elementwise gate of chunk rows and single rows (also split over blocks) against the oracle's
    attention, with bias steps of several units from bucket to bucket -- tables held on chip and, with many heads,
    tables too large for it, saturated buckets, no window."""
    n = 260
    g = torch.Generator().manual_seed(H + D)
    table = i32([[2, 0, 4, 3, 1]])
    rows = torch.randn(n, G * (D + P), generator=g).to(dtype)
    cache = _paged_rows(rows, table).to(device)
    w = 4.0 * torch.randn(B, H, generator=g)
    rel = w[mx.distance_buckets(B, far)[:size]].t().contiguous().to(device)
    k = rows[:, :G * D].double().numpy().reshape(n, G, D)
    v = rows[:, G * D:].double().numpy().reshape(n, G, P)
    q_all = torch.randn(n, H * D, generator=g).to(dtype)
    want = oracle.attend(q_all.double().numpy().reshape(n, H, D), k, v, 0.4, oracle.visible(n, {"size": size}),
                         bias=oracle.distance_bias(n, w.double().numpy(), far))
    for seg in _segments(n):
        t = len(seg)
        gate = torch.randn(t, H * P + 4, generator=g).to(dtype)
        out = mx.window_attend(q_all[seg].to(device), cache, i32([0, t], device), i32(seg, device), table.to(device), size,
                               0.4, t, H, G, D, P, gate=gate.to(device)[:, 4:], rel=rel).double().cpu().numpy()
        ref = want[seg].reshape(t, H * P) * oracle.sigmoid(gate[:, 4:].double().numpy())
        assert np.abs(out - ref).max() < (3e-5 if dtype == torch.float32 else 4e-2), (seg[0], t)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_bucket_edges_stand_out(device, dtype):
    """All scores zero and one bias row far above the rest: exactly the keys whose distance falls into that row are
    averaged -- for every row of the table, from a chunk and from single rows."""
    H, G, D, P, n, B, far, size = 2, 1, 16, 200, 200, 8, 60, 150
    table = i32([[2, 0, 3, 1]])
    rows = torch.zeros(n, D + P)
    rows[:, D:] = torch.eye(n)[:, :P]                       # key j's value: the j-th unit vector
    cache = _paged_rows(rows.to(dtype), table).to(device)
    for b in range(B):
        w = torch.full((B, H), -30.0)
        w[b] = 10.0
        rel = w[mx.distance_buckets(B, far)[:size]].t().contiguous().to(device)
        for seg in (list(range(160, 180)), [199], [70], [3]):
            t = len(seg)
            out = mx.window_attend(torch.zeros(t, H * D, dtype=dtype, device=device), cache, i32([0, t], device),
                                   i32(seg, device), table.to(device), size, 1.0, t, H, G, D, P, rel=rel).float().cpu()
            out = out.view(t, H, P)
            for i, p in enumerate(seg):
                hit = [j for j in range(max(0, p - size + 1), p + 1) if oracle.bucket(p - j, B, far) == b]
                if hit:
                    ref = torch.zeros(P)
                    ref[hit] = 1.0 / len(hit)
                    assert (out[i] - ref).abs().max() < 4e-3, (b, p)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,P,size,cap", [(6, 2, 16, 12, 37, 2.0), (4, 4, 24, 8, 1 << 30, 50.0), (5, 1, 9, 7, 1 << 30, 0.5),
                                              (12, 3, 40, 33, 130, 5.0), (2, 1, 64, 272, 1 << 30, 3.0), (3, 1, 136, 136, 100, 4.0)])
def test_attention_cap_sink_gate(device, dtype, H, G, D, P, size, cap):
    """Soft cap, sink and head gate against the oracle's attention: raw scores far inside and far beyond the cap,
    sinks from far below to far above what the cap allows; with a distance bias as well (added after the cap)."""
    n = 260
    g = torch.Generator().manual_seed(H + D)
    table = i32([[2, 0, 4, 3, 1]])
    rows = torch.randn(n, G * (D + P), generator=g).to(dtype)
    cache = _paged_rows(rows, table).to(device)
    sink = torch.linspace(-30.0, 12.0, H) if H > 2 else torch.tensor([1.0, 4.0])
    k = rows[:, :G * D].double().numpy().reshape(n, G, D)
    v = rows[:, G * D:].double().numpy().reshape(n, G, P)
    q_all = torch.randn(n, H * D, generator=g) * torch.linspace(0.1, 30.0, n)[:, None]
    q_all = q_all.to(dtype)
    w = torch.randn(6, H, generator=g)
    rel = w[mx.distance_buckets(6, 20)].t().contiguous().to(device)
    bias = oracle.distance_bias(n, w.double().numpy(), 20)
    for with_bias in (False, True):
        want = oracle.attend(q_all.double().numpy().reshape(n, H, D), k, v, 0.4, oracle.visible(n, {"size": size}), cap=cap,
                             sink=sink.double().numpy(), bias=bias if with_bias else None)
        for seg in _segments(n):
            t = len(seg)
            gate = torch.randn(t, H, generator=g).to(dtype)
            out = mx.window_attend(q_all[seg].to(device), cache, i32([0, t], device), i32(seg, device), table.to(device), size,
                                   0.4, t, H, G, D, P, gate=gate.to(device), sink=sink.to(device), softcap=cap,
                                   rel=rel if with_bias else None).double().cpu().numpy()
            ref = (want[seg] * oracle.sigmoid(gate.double().numpy())[:, :, None]).reshape(t, H * P)
            assert np.abs(out - ref).max() < (5e-5 if dtype == torch.float32 else 4e-2), (seg[0], t)


@pytest.mark.gpu
def test_option_combinations_beside_the_matrix_cores():
    """bf16 combinations the matrix-core forms do not take (they run on the f32-lane kernel): a table with slopes,
    with kept first tokens, a cap on sigmoid weights; against the PyTorch form."""
    H, G, D, P, n, size = 4, 2, 16, 16, 150, 40
    g = torch.Generator().manual_seed(1)
    table = i32([[2, 0, 1]])
    cache = _paged_rows(torch.randn(n, G * (D + P), generator=g).bfloat16(), table)
    rel, sl = torch.randn(H, 30, generator=g), torch.rand(H, generator=g)
    q = torch.randn(n, H * D, generator=g).bfloat16()
    for kw in (dict(rel=rel, slopes=sl), dict(rel=rel, keep_first=5), dict(softcap=3.0, head_bias=sl), dict(softcap=3.0, slopes=sl),
               dict(softcap=3.0, keep_first=5)):
        for seg in (list(range(90, 140)), [149]):
            t = len(seg)
            args = lambda d: (q[seg].to(d), cache.to(d), i32([0, t], d), i32(seg, d), table.to(d), size, 0.3, t, H, G, D, P)  # noqa: E731
            dev = {k: v.cuda() if torch.is_tensor(v) else v for k, v in kw.items()}
            a, b = mx.window_attend(*args("cpu"), **kw).float(), mx.window_attend(*args("cuda"), **dev).float().cpu()
            assert (a - b).abs().max() < 4e-2 * max(1.0, a.abs().max().item()), kw.keys()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [1, 5, 64, 70])
def test_window_edges_stand_out(device, dtype, size):
    """One key per query gets an overwhelming score, distance bias and all: the oldest key of the window is seen,
    the one before it is not.  Chunk rows and single rows around page borders; row cache and latent cache."""
    H, G, D, P, n = 6, 2, 16, 12, 200
    g = torch.Generator().manual_seed(size)
    table = i32([[2, 0, 3, 1]])
    rel = torch.randn(H, min(40, size), generator=g).to(device)
    chunks = [list(range(p0, p0 + 8)) for p0 in (size, 60, 124, 188)]
    chunks += [[p] for p in (size - 1, size, size + 1, 63, 64, 65, 127, 128, 199)]
    base = torch.zeros(n, G * (D + P))
    base[:, G * D:] = torch.randn(n, G * P, generator=g)
    lat = torch.randn(n, 32 + 4, generator=g)          # latent rows: 16 value entries, 16 that answer queries, 4 rotated
    lat[:, 16:] = 0.0
    for kind in ("oldest", "before"):
        for seg in chunks:
            t = len(seg)
            rows, lrows, q, ql, target = base.clone(), lat.clone(), torch.zeros(t, H, D), torch.zeros(t, H, 32), []
            for i, p in enumerate(seg):
                j = max(p - size + 1, 0) if kind == "oldest" else p - size
                target.append(j)
                if j >= 0:
                    for kvh in range(G):
                        rows[j, kvh * D + i] = 60.0
                    lrows[j, 16 + i] = 60.0
                q[i, :, i] = 5.0
                ql[i, :, 16 + i] = 5.0
            rows, lrows = rows.to(dtype), lrows.to(dtype)
            cu, pos, bt = i32([0, t], device), i32(seg, device), table.to(device)
            out = mx.window_attend(q.to(dtype).reshape(t, -1).to(device), _paged_rows(rows, table).to(device), cu, pos, bt, size,
                                   1.0, t, H, G, D, P, rel=rel).float().cpu().view(t, H, P)
            lo = mx.latent_attend(ql.to(dtype).to(device), torch.zeros(t, H, 4, dtype=dtype, device=device),
                                  _paged_rows(lrows, table).to(device), cu, pos, bt, size, 1.0, t,
                                  sink=torch.zeros(H, device=device), exact_weights=True).float().cpu()
            for i, p in enumerate(seg):
                if target[i] < 0:
                    continue
                seen = kind == "oldest"
                for h in range(H):
                    kvh = h // (H // G)
                    tv = rows[target[i], G * D + kvh * P:G * D + (kvh + 1) * P].float()
                    assert bool((out[i, h] - tv).abs().max() < 0.05) == seen, (kind, seg, i, h)
                    assert bool((lo[i, h, :16] - lrows[target[i], :16].float()).abs().max() < 0.05) == seen, (kind, seg, i, h)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,R,Dr,size", [(3, 40, 8, 21), (8, 72, 24, 150), (5, 35, 6, 1 << 30), (16, 136, 16, 64), (2, 300, 8, 100),
                                         (70, 32, 8, 90)])
def test_latent_attention_with_sink(device, dtype, H, R, Dr, size):
    """Sinks from far below to far above the scores, chunk rows and single rows (also split over blocks), with one and
    two terms per softmax weight, with and without a head gate."""
    n = 260
    g = torch.Generator().manual_seed(H + R)
    table = i32([[2, 0, 4, 3, 1]])
    rows = torch.randn(n, R + Dr, generator=g).to(dtype)
    cache = _paged_rows(rows, table).to(device)
    sink = torch.linspace(-30.0, 12.0, H)
    ql, qr = torch.randn(n, H, R, generator=g).to(dtype), torch.randn(n, H, Dr, generator=g).to(dtype)
    kv = rows.double().numpy()[:, None]
    q = torch.cat([ql, qr], -1).double().numpy()
    vis = oracle.visible(n, {"size": size})
    for sk in (sink, None):
        want = oracle.attend(q, kv, kv[..., :R], 0.3, vis, sink=None if sk is None else sk.double().numpy())
        for seg in _segments(n):
            t = len(seg)
            gate = torch.randn(t, H, generator=g).to(dtype)
            for exact in (True, False):
                out = mx.latent_attend(ql[seg].to(device), qr[seg].to(device), cache, i32([0, t], device), i32(seg, device),
                                       table.to(device), size, 0.3, t, gate=gate.to(device) if not exact else None,
                                       sink=None if sk is None else sk.to(device), exact_weights=exact).double().cpu().numpy()
                ref = want[seg] * (1.0 if exact else oracle.sigmoid(gate.double().numpy())[:, :, None])
                assert np.abs(out - ref).max() < (3e-5 if dtype == torch.float32 else 4e-2), (seg[0], t, exact)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_sinks_count_once(device, dtype):
    """Keys and scores all zero: the output is (number of visible keys) / (that number + exp(sink)) times the common
    value -- once per query, not once per tile or per block of a split row, neither scaled nor capped."""
    H, D, P, R, n = 2, 16, 16, 16, 500
    table = i32([[7, 1, 0, 2, 6, 3, 5, 4]])
    rows = torch.zeros(n, D + P)
    rows[:, D:] = 2.0
    lrows = torch.zeros(n, R + 4)
    lrows[:, :R] = 2.0
    cache, lcache = _paged_rows(rows.to(dtype), table).to(device), _paged_rows(lrows.to(dtype), table).to(device)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    for sink in (0.0, math.log(100.0), -80.0, 90.0):
        sk = torch.full((H,), sink, device=device)
        for size, seg in ((1 << 30, [499]), (320, [499]), (320, list(range(300, 400))), (1 << 30, [0]), (5, [2, 3, 4, 5, 6])):
            t = len(seg)
            cu, pos, bt = i32([0, t], device), i32(seg, device), table.to(device)
            out = mx.window_attend(torch.zeros(t, H * D, dtype=dtype, device=device), cache, cu, pos, bt, size, 0.1, t, H, 1, D, P,
                                   sink=sk, softcap=2.0).float().cpu()
            lo = mx.latent_attend(torch.zeros(t, H, R, dtype=dtype, device=device), torch.zeros(t, H, 4, dtype=dtype, device=device),
                                  lcache, cu, pos, bt, size, 0.1, t, sink=sk, exact_weights=True).float().cpu()
            for i, p in enumerate(seg):
                c = min(p + 1, size)
                want = 2.0 * c / (c + math.exp(sink))
                assert (out[i] - want).abs().max() < tol and (lo[i] - want).abs().max() < tol, (sink, size, p)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key_under_the_cap(device, dtype):
    """A key hundreds of tokens back whose raw score is far beyond the cap weighs exactly as the capped score says:
    with a cap of 9 against 400 keys of score 0, not all of the weight."""
    H, D, P, n, far, cap = 2, 16, 4, 400, 9, 9.0
    table = i32([[3, 0, 6, 1, 5, 2, 4]])
    rows = torch.zeros(n, D + P)
    rows[far, 0] = 100.0
    rows[far, D:] = 1.0
    cache = _paged_rows(rows.to(dtype), table).to(device)
    for seg in (list(range(380, 400)), [399], [333], [9], [8]):
        t = len(seg)
        for raw, q0 in ((300.0, 3.0), (9.0, 0.09), (-300.0, -3.0), (2.0, 0.02)):
            q = torch.zeros(t, H, D)
            q[:, :, 0] = q0
            raw = float(torch.tensor(q0).to(dtype)) * 100.0
            out = mx.window_attend(q.reshape(t, -1).to(dtype).to(device), cache, i32([0, t], device), i32(seg, device),
                                   table.to(device), 1 << 30, 1.0, t, H, 1, D, P, softcap=cap).float().cpu()
            for i, p in enumerate(seg):
                e = math.exp(cap * math.tanh(raw / cap)) if p >= far else 0.0
                want = e / (e + p + (0 if p >= far else 1))
                assert (out[i] - want).abs().max() < (1e-4 if dtype == torch.float32 else 6e-3), (p, q0)


@pytest.mark.parametrize("device", DEVICES)
def test_routing(device):
    """The bias is part of the logits: it decides who is chosen and enters the weights; the weights are the softmax
    over the chosen; large logits; ties go to the lower index; bucketed rows and every expert over every row agree,
    also when one expert gets no row, with and without a shared expert."""
    from financial_chatbot_llm_amd.models import mixers as mm
    for shared in (None, {"ff": 24, "limit": 0.8}):
        spec = {"kind": "moe", "expert": {"ff": 20, "limit": 1.1}, "router": {"experts": 6, "top": 3}}
        if shared:
            spec["shared"] = shared
        ff = RoutedFF(spec, 32, score="softmax_top")
        g = torch.Generator().manual_seed(2)
        sd = {k: torch.randn(s, generator=g) * s[-1] ** -0.5 for k, s in ff.shapes().items()}
        sd["router.b"] = torch.tensor([0.0, 1.0, -50.0, 0.3, 80.0, 0.0])          # 2 never chosen, 4 always
        w_in = ff.load(lambda k: sd[k].to(device), torch.float32)
        h = torch.randn(37, 32, generator=g)
        hd = h.to(device)
        proj = torch.nn.functional.linear(hd, w_in) if w_in is not None else None
        want = oracle.experts_ff(h.double().numpy(), oracle.as_arrays(sd), "", spec)
        old = mm.DENSE_MAX_PAIRS
        try:
            for limit in (512, 1):
                mm.DENSE_MAX_PAIRS = limit
                got = ff.forward(hd, proj).cpu().double().numpy()
                assert np.abs(got - want).max() < 1e-4 * np.abs(want).max()
        finally:
            mm.DENSE_MAX_PAIRS = old
    z = torch.zeros(2, 9, device=device)
    w, i = mx.route_scores(z, 4, "softmax_top")
    assert i.tolist() == [[0, 1, 2, 3]] * 2 and (w.cpu() - 0.25).abs().max() < 1e-6


# ---------------------------------------------------------------------------------------------------
# generation through the engine's own scheduler
# ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device,graphs", [("cpu", False), pytest.param("cuda", False, marks=pytest.mark.gpu),
                                           pytest.param("cuda", True, marks=pytest.mark.gpu)])
@pytest.mark.parametrize("async_", [False, True])
def test_greedy_generation(device, graphs, async_):
    cfgd = small_config("LRC", vocab=256)
    eng, sd = build(cfgd, device, torch.float32, blocks_=12, seqs=2, graphs=graphs, async_=async_)
    poison(eng)
    prompts = [tokens(70, 256, 41), tokens(9, 256, 42), tokens(30, 256, 43)]     # three requests, two at a time
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert o == oracle.greedy(cfgd, sd, p, 12)
    assert eng.bm.num_free() == eng.bm.num_blocks
    if graphs:
        assert eng.runner.stats["graph_steps"] > 0


@pytest.mark.parametrize("device", DEVICES)
def test_prefix_reuse(device):
    """A second request on the same two pages of prompt reuses them in every pass of the loop."""
    cfgd = small_config("LRC", vocab=256)
    eng, sd = build(cfgd, device, torch.float32, blocks_=12, seqs=2, prefix=True)
    head = tokens(128, 256, 61)
    for tail in (tokens(7, 256, 62), tokens(20, 256, 63)):
        out = eng.generate([head + tail], SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))[0]
        assert out == oracle.greedy(cfgd, sd, head + tail, 6)
    assert eng.bm.hit_rate() > 0


@pytest.mark.gpu
def test_sampling_with_the_fused_head():
    """A width the fused LM-head sampler accepts, bf16, decode graphs."""
    cfgd = small_config("LRC", width=256, vocab=512)
    eng, sd = build(cfgd, "cuda", torch.bfloat16, graphs=True)
    outs = eng.generate([tokens(20, 512, 1)], SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))
    assert len(outs[0]) == 6


@pytest.mark.gpu
def test_graph_replays_match_eager_steps():
    """bf16 decoding through captured graphs and eagerly: the same greedy tokens, with eager prompt steps between the
    replays."""
    cfgd = small_config("LRC", vocab=256)
    got = []
    for graphs in (False, True):
        eng, _ = build(cfgd, "cuda", torch.bfloat16, blocks_=16, seqs=2, graphs=graphs)
        got.append(eng.generate([tokens(n, 256, n) for n in (70, 9, 30, 64)],
                                SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True)))
        assert (eng.runner.stats["graph_steps"] > 0) == graphs
    same = sum(a == b for a, b in zip(*got))
    assert same >= 3, got                              # at most one greedy near-tie in bf16


def test_preemption():
    """A pool too small for both sequences: the younger one is preempted and recomputed from its first token."""
    cfgd = small_config("LRC", vocab=256)
    eng, sd = build(cfgd, "cpu", torch.float32, blocks_=3, seqs=2)
    prompts = [tokens(60, 256, 51), tokens(62, 256, 52)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True))
    assert eng.scheduler.num_preemptions > 0
    for p, o in zip(prompts, outs):
        assert o == oracle.greedy(cfgd, sd, p, 10)


def test_registry_and_config_errors():
    from financial_chatbot_llm_amd.models import get_model_config
    from financial_chatbot_llm_amd.models.fanotar import FanotarModel
    from financial_chatbot_llm_amd.models.fanotar import example_config as fanotar_config
    c = get_model_config("sepitar-tiny")
    assert c.arch == "sepitar" and len(c.layers) == c.num_layers == 3 and c.loop["times"] == 2

    def bad(change, error=ValueError):
        cfgd = copy.deepcopy(example_config())
        change(cfgd)
        with pytest.raises(error):
            SepitarModel(layered_config(cfgd, "bad"), device="cpu")

    bad(lambda c: c["layers"][0].update(type="window_attention"))                # another design's mixer
    bad(lambda c: c["layers"][0]["mlp"].update(kind="other"))
    bad(lambda c: c["layers"][1]["mixer"].update(heads=5))                       # heads must split into kv_heads
    bad(lambda c: c["layers"][1]["mixer"].pop("bias_max"), KeyError)
    bad(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10))                # more than the rotated part
    bad(lambda c: c["layers"][2]["mixer"]["rot"].update(dims=7))
    bad(lambda c: c["layers"][1]["mlp"]["router"].update(top=8))
    bad(lambda c: c["loop"].update(stop=4))
    bad(lambda c: c["loop"].update(times=0))
    other = fanotar_config()
    other["loop"] = {"start": 0, "stop": 1, "times": 2}                          # a design that runs every layer once
    with pytest.raises(ValueError):
        FanotarModel(layered_config(other, "bad"), device="cpu")
    m = SepitarModel(layered_config(example_config(), "ok"), device="cpu")
    assert not m.has_state and len(m.cache_specs()) == 5
    sd = random_weights(m, 0)
    assert "l0.mix.g" not in sd and sd["l2.mix.g"].shape == (4, 160) and sd["l1.mix.g"].shape == (120, 160)
    assert "l1.mix.o.b" in sd and "l2.mix.o.b" not in sd and "l0.mlp.router.b" in sd and "l0.mlp.correction" not in sd
    m.load_state(sd)
    short = dict(sd)
    short["l1.mix.rel"] = sd["l1.mix.rel"][:, :3]
    with pytest.raises(ValueError):
        m.load_state(short)
    short = dict(sd)
    short.pop("l2.mix.sink")
    with pytest.raises(KeyError):
        m.load_state(short)
    m.init_random(seed=3)                            # registry examples run with random weights
    rows = torch.zeros(64, 8)
    args = (torch.zeros(1, 4), rows, i32([0, 1]), i32([0]), i32([[0]]), 4, 1.0, 1, 1, 1, 4, 4)
    with pytest.raises(ValueError):
        mx.window_attend(*args, rel=torch.zeros(2, 3))
    with pytest.raises(ValueError):
        mx.latent_attend(torch.zeros(1, 2, 4), torch.zeros(1, 2, 4), rows, *args[2:5], 4, 1.0, 1, sink=torch.zeros(3))
