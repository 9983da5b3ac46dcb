"""Fanotar (layered decoder with elementwise norms around every sublayer, convolved attention with a distance bias,
a window and a sink, keys and values shared between layers, renormalised sigmoid routing) against the plain oracle
of tests/fanotar_oracle.py.

Small configurations with random weights made here; the framework side always runs through the engine
(scheduler admission, pages, state slots, runner) or the ops' public entry points.  CPU tensors exercise
the ops' PyTorch forms, ``cuda`` ones the HIP kernels (marked gpu).
"""
import copy
import math

import numpy as np
import pytest
import torch

import fanotar_oracle as oracle
from financial_chatbot_llm_amd.config import EngineConfig
from financial_chatbot_llm_amd.engine import LLMEngine, SamplingParams
from financial_chatbot_llm_amd.models.configs import layered_config
from financial_chatbot_llm_amd.models.fanotar import FanotarModel, example_config
from financial_chatbot_llm_amd.models.mixers import RoutedFF
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
        if leaf == "alpha":
            t = 0.3 + 0.6 * torch.rand((), generator=g)
        elif leaf in ("norm1", "norm2", "norm1b", "norm2b", "norm"):
            t = 1.0 + 0.2 * r
        elif leaf == "b":
            t = 0.2 * r
        elif leaf == "sink":
            t = r
        elif leaf == "conv":
            t = r * shape[1] ** -0.5
        elif leaf == "correction":
            t = 0.1 * r
        elif leaf == "embed":
            t = 0.4 * r
        else:
            t = r * shape[-1] ** -0.5 * 1.5
        sd[name] = t.to(torch.bfloat16)
    return sd


def small_config(pattern="AEkK", **over):
    return example_config(width=over.pop("width", 96), vocab=over.pop("vocab", 168), pattern=pattern)


def build(cfgd, device, dtype, seed=1, blocks_=24, seqs=4, graphs=False, async_=False, max_len=1024):
    mc = layered_config(cfgd, "fanotar-test")
    model = FanotarModel(mc, device=device, dtype=dtype)
    sd = random_weights(model, seed)
    model.load_state(sd)
    eng = LLMEngine(EngineConfig(model="fanotar-test", device=device, dtype="fp32" if dtype == torch.float32 else "bf16",
                                 num_kv_blocks=blocks_, max_num_seqs=seqs, max_model_len=max_len,
                                 max_num_batched_tokens=512, enable_prefix_caching=False, use_cuda_graph=graphs,
                                 async_scheduling=async_, graph_batch_sizes=(1, 2, 4)), model=model)
    return eng, sd


def _poison(entry):
    for t in entry[1:]:
        if isinstance(t, dict):
            for v in t.values():
                v.fill_(float("nan"))
        elif isinstance(t, tuple):
            _poison(t)
        else:
            t.fill_(float("nan"))


def poison(eng):
    """Pages and slots as a previous owner might have left them: nothing may depend on their content."""
    for lay in eng.kv.layers:
        _poison(lay)


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
# whole models, layer kinds, sizes
# ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("pattern", ["a", "A", "e", "E", "ak", "AK", "AEkaKk"])
def test_layer_kinds_against_oracle(device, dtype, pattern):
    """Attention alone, each feed-forward, a layer on another layer's keys and values, and a mix in which two
    layers share the first source and two the second."""
    cfgd = small_config(pattern)
    eng, sd = build(cfgd, device, dtype)
    poison(eng)
    toks = tokens(90, cfgd["vocab"], 3)          # crosses a 64-token page and leaves the 37-token window twice
    close(run_whole(eng, "r", toks), oracle.forward(cfgd, sd, toks), dtype, routed=any(c in "eEK" for c in pattern))


@pytest.mark.parametrize("device", DEVICES)
def test_residual_stream_after_every_layer(device):
    cfgd = small_config("AEkK")
    eng, sd = build(cfgd, device, torch.float32)
    toks = tokens(40, cfgd["vocab"], 4)
    want = []
    oracle.forward(cfgd, sd, toks, want)
    eng.model.capture = []
    run_whole(eng, "r", toks)
    assert len(eng.model.capture) == len(want) == 4
    for got, ref in zip(eng.model.capture, want):
        close(got, ref, torch.float32)


@pytest.mark.parametrize("device", DEVICES)
def test_absent_entries_and_single_sizes(device):
    """No feed-forward, no mask, no temperature, no convolution, one tap, no shared expert, one expert, one head,
    one key/value head, as many key/value heads as heads (also by an absent entry), a window of one key, scales of
    0 and 1, a source layer's mask and temperature unlike those of the layer that reads it, no embedding scale."""
    cfgd = small_config("aAeEkK")
    del cfgd["embedding"]
    L = cfgd["layers"]
    del L[0]["mixer"]["mask"]
    del L[0]["mixer"]["conv"]
    L[0]["mixer"].update(heads=1, kv_heads=1)
    del L[1]["mixer"]["q_temp"]
    del L[1]["mixer"]["kv_heads"]
    L[1]["mixer"].update(mask={"size": 1}, conv=1)
    L[2]["mixer"].update(kv_heads=1, scale=1.0)
    L[2]["mlp"]["router"].update(experts=1, top=1, scale=1.0)
    L[3]["mixer"].update(kv_heads=6, scale=0.0)
    L[3]["mlp"]["router"].update(top=7)
    L[4]["mixer"].update(kv_heads=6, mask={"size": 50}, q_temp={"coef": 0.9, "every": 1})
    L[5]["mixer"].update(kv_heads=6, conv=2)
    del L[5]["mixer"]["mask"]
    eng, sd = build(cfgd, device, torch.float32)
    assert "l0.norm2" not in sd and "l0.mix.q.conv" not in sd and "l1.mix.q.conv" in sd
    assert "l4.mix.k" not in sd and "l4.mix.k.norm" not in sd and "l4.mix.v.conv" not in sd and "l4.mix.q.conv" in sd
    full = copy.deepcopy(cfgd)          # the oracle reads every entry: write out what absence means
    full["layers"][1]["mixer"]["kv_heads"] = 6
    w = oracle.as_arrays(sd)
    w.update({f"l0.mix.{n}.conv": np.ones((w[f"l0.mix.{n}"].shape[0], 1)) for n in "qkv"})
    poison(eng)
    toks = tokens(90, cfgd["vocab"], 5)
    close(run_whole(eng, "r", toks), oracle.forward(full, w, toks), torch.float32)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_other_sizes(device, dtype):
    """Sizes unlike the small default: odd head counts, key and value sizes that fill no wave and differ, taps from
    2 to 16, windows longer than a page and very short ones, feed-forward widths of 1, 9 and 333, 70 experts top
    5, a width that is no multiple of the wide accesses, a large norm eps, other constants."""
    cfgd = small_config("AEkAEKa", width=82, vocab=97)
    cfgd["norm"]["eps"] = 0.02
    cfgd["embedding"]["scale"] = 0.7
    L = cfgd["layers"]
    L[0]["mixer"].update(dim=40, vdim=9, heads=6, kv_heads=1, conv=2, mask={"size": 70}, scale=0.31,
                         q_temp={"coef": 1.3, "every": 64})
    L[1]["mixer"].update(dim=9, vdim=33, heads=5, kv_heads=5, conv=5, mask={"size": 3}, scale=0.6)
    L[2]["mixer"].update(dim=9, vdim=33, heads=5, kv_heads=5, conv=8, mask={"size": 64}, scale=0.9, kv_from=1)
    L[3]["mixer"].update(dim=34, vdim=20, heads=2, kv_heads=2, conv=9, mask={"size": 100}, scale=0.2)
    L[4]["mixer"].update(dim=132, vdim=17, heads=3, kv_heads=1, conv=16, scale=0.05)
    L[5]["mixer"].update(dim=132, vdim=17, heads=3, kv_heads=1, conv=4, scale=0.08, kv_from=4)
    L[6]["mixer"].update(dim=64, vdim=130, heads=12, kv_heads=4, conv=7, scale=0.1, mask={"size": 65})
    L[0]["mlp"].update(ff=333, limit=0.4)
    L[1]["mlp"].update(router={"experts": 70, "scale": 0.6, "top": 5}, expert={"ff": 9, "limit": 2.2})
    L[1]["mlp"]["shared"].update(ff=1, limit=3.0)
    L[2]["mlp"].update(ff=50, limit=1.0)
    L[3]["mlp"].update(ff=1, limit=10.0)
    L[4]["mlp"].update(router={"experts": 3, "scale": 2.0, "top": 1}, expert={"ff": 33, "limit": 0.3})
    eng, sd = build(cfgd, device, dtype, blocks_=8)
    poison(eng)
    toks = tokens(150, cfgd["vocab"], 7)
    close(run_whole(eng, "r", toks), oracle.forward(cfgd, sd, toks), dtype, routed=True)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_wide_heads(device, dtype):
    """Head sizes beyond what the matrix-core attention covers (bf16 then takes the f32-lane kernel), even and odd."""
    cfgd = small_config("akA", width=64)
    L = cfgd["layers"]
    for l in L[:2]:
        l["mixer"].update(dim=264, vdim=300, heads=2, kv_heads=1, scale=0.06)
    L[2]["mixer"].update(dim=261, vdim=41, heads=2, kv_heads=2, scale=0.05, conv=9)
    eng, sd = build(cfgd, device, dtype, blocks_=4)
    toks = tokens(80, cfgd["vocab"], 8)
    close(run_whole(eng, "r", toks), oracle.forward(cfgd, sd, toks), dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(device):
    """Sequences of one and two tokens, and the first tokens of a longer one, each request alone."""
    cfgd = small_config("AEkK")
    eng, sd = build(cfgd, device, torch.float32)
    poison(eng)
    for n in (1, 2, 5):
        toks = tokens(n, cfgd["vocab"], 60 + n)
        close(run_whole(eng, f"r{n}", toks), oracle.forward(cfgd, sd, toks), torch.float32)


@pytest.mark.parametrize("device", DEVICES)
def test_model_without_taps_holds_no_slots(device):
    cfgd = small_config("Ak")
    for l in cfgd["layers"]:
        l["mixer"]["conv"] = 1
    eng, sd = build(cfgd, device, torch.float32)
    poison(eng)
    assert eng.state_slots is None
    toks = tokens(100, cfgd["vocab"], 17)
    want = oracle.forward(cfgd, sd, toks)
    got = [eng.replay_step([("r", toks[:70], list(range(70)))])]
    got += [eng.replay_step([("r", toks[i:i + 1], [0])]) for i in range(70, 100)]
    close(torch.cat(got), want, torch.float32)


def test_shared_layers_add_no_cache_rows():
    """Layers on another layer's keys and values take no pages of their own: only their queries' convolution is
    kept per sequence."""
    one = FanotarModel(layered_config(small_config("A"), "t"), device="cpu")
    three = FanotarModel(layered_config(small_config("Akk"), "t"), device="cpu")
    assert one.kv_bytes_per_block() == three.kv_bytes_per_block() == 64 * 2 * (24 + 20) * 2
    kv = three.make_cache(2, 3)
    assert kv.layers[1][1] == ("none",) and tuple(kv.layers[1][2][1]["conv"].shape) == (3, 2, 6 * 24)


# ---------------------------------------------------------------------------------------------------
# cache, state, batching
# ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_prefill_then_token_by_token(device, dtype):
    cfgd = small_config("AEkK")
    eng, sd = build(cfgd, device, dtype)
    poison(eng)
    toks = tokens(140, cfgd["vocab"], 11)
    want = oracle.forward(cfgd, sd, toks)
    got = [eng.replay_step([("r", toks[:30], list(range(30)))])]
    for i in range(30, len(toks)):               # long decoding: the window passes over decoded tokens and a page border
        got.append(eng.replay_step([("r", toks[i:i + 1], [0])], ["r"] if i == len(toks) - 1 else []))
    close(torch.cat(got), want, dtype, routed=True)
    assert eng.bm.num_free() == eng.bm.num_blocks and eng.state_slots.num_free() == 4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps", [2, 4, 12])
@pytest.mark.parametrize("sizes", [[2, 2, 3, 60, 2, 1, 1, 64, 5], [63, 1, 1, 2, 70], [1, 1, 1, 130], [2] * 20, [36, 2, 36, 1, 37]])
def test_portions(device, sizes, taps):
    """Portions cut inside pages and inside windows, down to two tokens -- fewer than the convolution's history."""
    cfgd = small_config("AEK")
    for l in cfgd["layers"]:
        l["mixer"]["conv"] = taps
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
    """Unequal requests in one batch (portions beside single tokens), more requests than slots and a
    pool that only fits what is live: pages and slots are freed and used again."""
    cfgd = small_config("AEkK")
    eng, sd = build(cfgd, device, dtype, blocks_=7, seqs=3)
    poison(eng)
    V = cfgd["vocab"]
    reqs = {f"q{i}": tokens(n, V, 20 + i) for i, n in enumerate([150, 70, 33, 100, 5, 64])}
    want = {k: torch.as_tensor(oracle.forward(cfgd, sd, t)) for k, t in reqs.items()}
    got = {k: [] for k in reqs}
    at = {k: 0 for k in reqs}
    sched = [
        [("q0", 50), ("q1", 3), ("q2", 33)],            # q2 complete at once
        [("q0", 1), ("q1", 60), ("q3", 2)],             # q3 takes q2's slot and pages
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
    assert eng.state_slots.reuses > 0
    assert all(at[k] == len(reqs[k]) for k in reqs)
    close(torch.cat([torch.cat(got[k]) for k in reqs]), torch.cat([want[k] for k in reqs]), dtype, routed=True)


@pytest.mark.parametrize("device", DEVICES)
def test_batch_rows_do_not_depend_on_their_neighbours(device):
    """The same request alone and between two others gives the same logits (f32)."""
    cfgd = small_config("AEK")
    eng, sd = build(cfgd, device, torch.float32)
    V = cfgd["vocab"]
    a, b, c = tokens(45, V, 1), tokens(20, V, 2), tokens(70, V, 3)
    alone = run_whole(eng, "x", b)
    poison(eng)
    out = eng.replay_step([("a", a, []), ("b", b, list(range(len(b)))), ("c", c, [])], ["a", "b", "c"])
    assert (out - alone).abs().max() <= 2e-6 * alone.abs().max()


# ---------------------------------------------------------------------------------------------------
# mechanisms alone, with inputs in which a fault stands out
# ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W", [(3, 8), (70, 132), (5, 7), (2050, 12)])
def test_elementwise_norms(device, dtype, T, W):
    """The embedding's and the residual update's passes against the oracle: arguments from 1e-6 to 60 (around the
    switch of the tanh's two branches, far into saturation), sources that are column slices."""
    g = torch.Generator().manual_seed(W)
    mk = lambda a: mx.DynTanh(a, torch.randn(W, generator=g), torch.randn(W, generator=g))  # noqa: E731
    n1, n2 = mk(0.9), mk(1.7)
    dev = lambda n: mx.DynTanh(n.alpha, n.w.to(device), n.b.to(device))  # noqa: E731
    w = {}
    for k, n in (("p", n1), ("q", n2)):
        w.update({k: n.w.double().numpy(), k + ".b": n.b.double().numpy(), k + ".alpha": n.alpha})
    mag = 10.0 ** (torch.rand(T, W, generator=g) * 7.8 - 6.0) * torch.randn(T, W, generator=g).sign()
    x = torch.randn(T, W, generator=g)
    buf = torch.zeros(T, W + 4, dtype=dtype)
    buf[:, 4:] = mag.to(dtype)
    y = buf.to(device)[:, 4:]
    xd = x.clone().to(device)
    h = mx.dyn_tanh_residual(xd, y, dev(n1), dev(n2), dtype)
    xw = x.double().numpy() + oracle.dyn_tanh(buf[:, 4:].double().numpy(), w, "p")
    assert np.abs(xd.double().cpu().numpy() - xw).max() < 2e-6
    hw = oracle.dyn_tanh(xw, w, "q")
    assert h.dtype == dtype and np.abs(h.double().cpu().numpy() - hw).max() < (4e-6 if dtype == torch.float32 else 3e-2)
    only = mx.dyn_tanh_residual(xd, None, None, dev(n2), torch.float32)          # the stream's norm alone
    assert np.abs(only.double().cpu().numpy() - hw).max() < 4e-6
    x2 = x.clone().to(device)
    assert mx.dyn_tanh_residual(x2, y, dev(n1)) is None                           # the update alone
    assert torch.equal(x2, xd)
    table = torch.randn(11, W, generator=g).to(dtype)
    ids = torch.randint(0, 11, (T,), generator=g)
    xe, he = mx.dyn_tanh_embed(ids.to(device), table.to(device), 2.5, dev(n1), dev(n2), dtype)
    xw = oracle.dyn_tanh(2.5 * table.double().numpy()[ids.numpy()], w, "p")
    assert np.abs(xe.double().cpu().numpy() - xw).max() < 2e-6
    hw = oracle.dyn_tanh(xw, w, "q")
    assert np.abs(he.double().cpu().numpy() - hw).max() < (4e-6 if dtype == torch.float32 else 3e-2)


@pytest.mark.gpu
def test_tanh_relative_accuracy():
    """The kernels' tanh keeps its relative accuracy down to tiny arguments and across its switch of branches."""
    v = torch.cat([torch.logspace(-12, 1.9, 4001), torch.linspace(0.55, 0.65, 2001)])
    v = torch.cat([v, -v])[None].contiguous()
    one = mx.DynTanh(1.0, torch.ones(v.shape[1], device="cuda"), torch.zeros(v.shape[1], device="cuda"))
    got = mx.dyn_tanh_residual(v.clone().cuda(), None, None, one, torch.float32).double().cpu()
    want = torch.tanh(v.double())
    assert ((got - want).abs() / want.abs()).max() < 4e-7


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("K,D,P", [(1, 6, 4), (2, 5, 3), (4, 24, 20), (4, 128, 128), (7, 130, 9), (16, 6, 200), (13, 33, 301)])
def test_convolved_heads(device, dtype, K, D, P):
    """Convolution, per-head norms, temperature and cache rows of several segments in one call -- lengths on and
    around the kernel's tile sizes, continued and fresh ones, padding segments, pages in no order -- against the
    oracle's functions; the slots' next histories; slots not in the call untouched."""
    H, G, eps, coef, every = 3, 1 if K == 2 else 3, 1e-3, 0.7, 9
    g = torch.Generator().manual_seed(K)
    C = (H + G) * D + G * P
    lens = [1, 2, 7, 8, 9, 15, 16, 17, 33, 1, 3]
    start = [0, 5, 0, 70, 3, 0, 1, 0, 200, 0, 12]
    fresh = [p == 0 for p in start]
    S, T = len(lens), sum(lens)
    cu = np.concatenate([[0], np.cumsum(lens)]).tolist()
    pos = sum([list(range(p, p + n)) for p, n in zip(start, lens)], [])
    seg_slot = [4, 0, 9, 2, 1, 3, 11, 5, 6, -1, 8]           # the tenth is a padding row
    wq, wk = 1 + 0.3 * torch.randn(D, generator=g), 1 + 0.3 * torch.randn(D, generator=g)
    wc = torch.randn(C, K, generator=g)
    buf = torch.randn(T, C + 2, generator=g).to(dtype)
    hist = torch.randn(12, max(K - 1, 1), C, generator=g).to(dtype).float()
    state = hist.clone()
    for s in range(S):
        if fresh[s] and seg_slot[s] >= 0:
            state[seg_slot[s]] = float("nan")                 # must not be read
    rows = torch.randperm(T + 7, generator=g)[:T].tolist()
    rows[3] = -1                                              # a row that is not cached
    cache = torch.full((T + 7, G * (D + P)), 7.0, dtype=dtype)
    cd, st = cache.to(device), state.to(device)
    q = mx.conv_heads(buf.to(device)[:, 2:], wc.to(device), st if K > 1 else None, wq.to(device), wk.to(device), eps,
                      i32(cu, device), i32(seg_slot, device), i32(pos, device), i32(rows, device), cd, max(lens), H, G, D, P,
                      coef, every).float().cpu()
    cd, st = cd.float().cpu(), st.cpu()
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    u = buf[:, 2:].double().numpy()
    temp = oracle.query_temperature(max(pos) + 1, {"coef": coef, "every": every})
    used = set()
    for s in range(S):
        a, b = cu[s], cu[s + 1]
        old = np.zeros((K - 1, C)) if fresh[s] or seg_slot[s] < 0 else hist[seg_slot[s]][:K - 1].double().numpy()
        full = np.concatenate([old, u[a:b]])
        y = oracle.short_conv(full, wc.double().numpy())[K - 1:]
        qw = oracle.rms(y[:, :H * D].reshape(-1, H, D), eps) * wq.double().numpy()
        qw = (qw * temp[pos[a:b]][:, None, None]).reshape(-1, H * D)
        kw = (oracle.rms(y[:, H * D:(H + G) * D].reshape(-1, G, D), eps) * wk.double().numpy()).reshape(-1, G * D)
        scale = max(1.0, np.abs(qw).max())
        assert np.abs(q[a:b].numpy() - qw).max() < tol * scale, s
        for t in range(a, b):
            if rows[t] >= 0:
                used.add(rows[t])
                want = np.concatenate([kw[t - a], y[t - a, (H + G) * D:]])
                assert np.abs(cd[rows[t]].numpy() - want).max() < tol * max(1.0, np.abs(want).max()), (s, t)
        if K > 1 and seg_slot[s] >= 0:
            assert torch.equal(st[seg_slot[s]].double(), torch.as_tensor(full[-(K - 1):])), s
    assert all((cd[r] == 7.0).all() for r in range(T + 7) if r not in used)
    if K > 1:
        for sl in set(range(12)) - set(seg_slot):
            assert torch.equal(st[sl], state[sl])
    # queries only: the same queries, no cache row, a state record of the queries' channels
    q2 = mx.conv_heads(buf.to(device)[:, 2:], wc[:H * D].contiguous().to(device),
                       hist[:, :, :H * D].contiguous().to(device) if K > 1 else None, wq.to(device), None, eps,
                       i32(cu, device), i32(seg_slot, device), i32(pos, device), i32(rows, device), None, max(lens), H, 0, D, P,
                       coef, every).float().cpu()
    assert (q2 - q).abs().max() <= 1e-6 * q.abs().max()


@pytest.mark.parametrize("device", DEVICES)
def test_temperature_steps(device):
    """The query factor changes exactly where floor((p + 1) / every) does, also far into a sequence."""
    D = 4
    pos = [0, 8, 9, 18, 19, 98, 99, 899, 900, 1000000]
    T = len(pos)
    q = mx.conv_heads(torch.ones(T, D, device=device), torch.ones(D, 1, device=device), None, None, None, 1e-5,
                      i32(list(range(T + 1)), device), i32([-1] * T, device), i32(pos, device), i32([-1] * T, device), None, 1,
                      1, 0, D, D, 0.5, 10).cpu()
    for i, p in enumerate(pos):
        assert abs(q[i, 0].item() - (1 + 0.5 * math.log((p + 1) // 10 + 1))) < 3e-6
    assert q[0, 0] == 1.0 and q[1, 0] == 1.0 and q[2, 0] > 1.3 and q[2, 0] == q[3, 0] and q[4, 0] > q[3, 0]


def _paged_rows(rows, table):
    """Cache of the rows of positions 0.. under the page table."""
    cache = torch.full((table.shape[1] * 64, rows.shape[1]), float("nan"), dtype=rows.dtype)
    for j in range(rows.shape[0]):
        cache[int(table[0, j // 64]) * 64 + j % 64] = rows[j]
    # rows of allocated pages the sequence has not reached hold what an earlier owner left there
    return torch.where(torch.isnan(cache), torch.full_like(cache, 3.0), cache)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,P,size", [(6, 2, 16, 12, 37), (4, 4, 24, 8, 64), (5, 1, 9, 7, 1 << 30), (12, 3, 40, 33, 130),
                                          (2, 1, 64, 272, 90)])
def test_attention_bias_sink_gate(device, dtype, H, G, D, P, size):
    """Distance bias, sink and elementwise gate of chunk rows and single rows (also split over blocks) against the
    oracle's attention: head by head slopes, sinks from far below to far above the scores."""
    n = 200
    g = torch.Generator().manual_seed(H + D)
    table = i32([[2, 0, 3, 1]])
    rows = torch.randn(n, G * (D + P), generator=g).to(dtype)
    cache = _paged_rows(rows, table).to(device)
    sl = torch.tensor(oracle.slopes(H), dtype=torch.float32)
    sink = torch.linspace(-30.0, 12.0, H) if H > 2 else torch.tensor([1.0, 4.0])
    k = rows[:, :G * D].double().numpy().reshape(n, G, D)
    v = rows[:, G * D:].double().numpy().reshape(n, G, P)
    m = {"scale": 0.4, "mask": {"size": size}}
    q_all = torch.randn(n, H * D, generator=g).to(dtype)
    want = oracle.attend(q_all.double().numpy().reshape(n, H, D), k, v, m, sink.double().numpy())
    for seg in (list(range(100, 150)), list(range(0, 9)), list(range(62, 67)), [199], [64], [0], [1]):
        t = len(seg)
        gate = torch.randn(t, H * P + 3, generator=g).to(dtype)
        out = mx.window_attend(q_all[seg].to(device), cache, i32([0, t], device), i32(seg, device), table.to(device), size,
                               0.4, t, H, G, D, P, gate=gate.to(device)[:, 3:], slopes=sl.to(device),
                               sink=sink.to(device)).double().cpu().numpy()
        ref = want[seg].reshape(t, H * P) * oracle.sigmoid(gate[:, 3:].double().numpy())
        assert np.abs(out - ref).max() < (2e-5 if dtype == torch.float32 else 4e-2), (seg[0], t)
        # one gate value per head stays what it was
        gh = torch.randn(t, H, generator=g).to(dtype)
        out = mx.window_attend(q_all[seg].to(device), cache, i32([0, t], device), i32(seg, device), table.to(device), size,
                               0.4, t, H, G, D, P, gate=gh.to(device), slopes=sl.to(device),
                               sink=sink.to(device)).double().cpu().numpy()
        ref = (want[seg] * oracle.sigmoid(gh.double().numpy())[:, :, None]).reshape(t, H * P)
        assert np.abs(out - ref).max() < (2e-5 if dtype == torch.float32 else 4e-2), (seg[0], t)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_counts_once(device, dtype):
    """Keys and scores all zero: the output is (number of visible keys) / (that number + exp(sink)) times the common
    value -- once per query, not once per tile or per block of a split row -- and a sink far above the scores
    silences the head without a non-finite value."""
    H, G, D, P, n = 2, 1, 16, 16, 500
    table = i32([[7, 1, 0, 2, 6, 3, 5, 4]])
    rows = torch.zeros(n, G * (D + P))
    rows[:, D:] = 2.0
    cache = _paged_rows(rows.to(dtype), table).to(device)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    for sink in (0.0, math.log(100.0), -80.0, 90.0):
        sk = torch.full((H,), sink, device=device)
        for size, seg in ((1 << 30, [499]), (320, [499]), (320, list(range(300, 400))), (1 << 30, [0]), (5, [2, 3, 4, 5, 6])):
            t = len(seg)
            q = torch.zeros(t, H * D, dtype=dtype, device=device)
            out = mx.window_attend(q, cache, i32([0, t], device), i32(seg, device), table.to(device), size, 1.0, t, H, G, D, P,
                                   sink=sk).float().cpu()
            for i, p in enumerate(seg):
                c = min(p + 1, size)
                want = 2.0 * c / (c + math.exp(sink))
                assert (out[i] - want).abs().max() < tol, (sink, size, p)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [1, 5, 64, 70])
def test_window_edges_stand_out(device, dtype, size):
    """One key per query gets an overwhelming score, distance bias and all: the oldest key of the window is seen,
    the one before it is not, and neither is the next one.  Chunk rows and single rows around page borders."""
    H, G, D, P, n = 6, 2, 16, 12, 200
    g = torch.Generator().manual_seed(size)
    table = i32([[2, 0, 3, 1]])
    base = torch.zeros(n, G * (D + P))
    base[:, G * D:] = torch.randn(n, G * P, generator=g)
    sl = torch.tensor(oracle.slopes(H), dtype=torch.float32)
    sink = torch.zeros(H)
    chunks = [list(range(p0, p0 + 8)) for p0 in (size, 60, 124, 188)]
    chunks += [[p] for p in (size - 1, size, size + 1, 63, 64, 65, 127, 128, 199)]
    for kind in ("oldest", "before"):
        for seg in chunks:
            t = len(seg)
            rows, q, target = base.clone(), torch.zeros(t, H, D), []
            for i, p in enumerate(seg):
                j = max(p - size + 1, 0) if kind == "oldest" else p - size
                target.append(j)
                if j >= 0:
                    for kvh in range(G):
                        rows[j, kvh * D + i] = 60.0
                q[i, :, i] = 5.0
            rows, qd = rows.to(dtype), q.to(dtype)
            out = mx.window_attend(qd.reshape(t, -1).to(device), _paged_rows(rows, table).to(device), i32([0, t], device),
                                   i32(seg, device), table.to(device), size, 1.0, t, H, G, D, P, slopes=sl.to(device),
                                   sink=sink.to(device)).float().cpu().view(t, H, P)
            for i, p in enumerate(seg):
                if target[i] < 0:
                    continue
                for h in range(H):
                    kvh = h // (H // G)
                    tv = rows[target[i], G * D + kvh * P:G * D + (kvh + 1) * P].float()
                    assert bool((out[i, h] - tv).abs().max() < 0.05) == (kind == "oldest"), (kind, seg, i, h)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key_against_the_distance_bias(device, dtype):
    """A key hundreds of tokens back wins for a head exactly when its score lead exceeds that head's slope times
    the distance -- with the slopes of 8 heads from 1/2 to 1/256 -- from a chunk and from split single rows."""
    H, G, D, P, n, far, lead = 8, 1, 16, 4, 400, 9, 40.0
    table = i32([[3, 0, 6, 1, 5, 2, 4]])
    rows = torch.zeros(n, D + P)
    rows[far, 0] = lead
    rows[far, D:] = 1.0
    cache = _paged_rows(rows.to(dtype), table).to(device)
    sl = torch.tensor(oracle.slopes(H), dtype=torch.float32)
    for seg in (list(range(380, 400)), [399], [333]):
        t = len(seg)
        q = torch.zeros(t, H, D)
        q[:, :, 0] = 1.0
        out = mx.window_attend(q.reshape(t, -1).to(dtype).to(device), cache, i32([0, t], device), i32(seg, device),
                               table.to(device), 1 << 30, 1.0, t, H, G, D, P, slopes=sl.to(device)).float().cpu().view(t, H, P)
        for i, p in enumerate(seg):
            for h in range(H):
                s = float(sl[h])
                others = sum(math.exp(-s * d) for d in range(p + 1) if p - d != far)
                wt = math.exp(lead - s * (p - far))
                want = wt / (wt + others)
                assert abs(out[i, h, 0].item() - want) < (1e-4 if dtype == torch.float32 else 1e-2), (p, h)
        assert out[0, 0].abs().max() < 1e-3 and out[0, H - 1].min() > 0.99


@pytest.mark.parametrize("device", DEVICES)
def test_layers_read_the_source_layers_rows(device):
    """The reading layer's output changes with the source layer's key and value weights and with nothing of the
    layer between them."""
    cfgd = small_config("AAk")
    cfgd["layers"][2]["mixer"]["kv_from"] = 0
    eng, sd = build(cfgd, device, torch.float32)
    toks = tokens(80, cfgd["vocab"], 31)
    close(run_whole(eng, "a", toks), oracle.forward(cfgd, sd, toks), torch.float32)
    wrong = copy.deepcopy(cfgd)                       # the mistake is planted in the oracle: the other source layer
    wrong["layers"][2]["mixer"]["kv_from"] = 1
    d = np.abs(run_whole(eng, "b", toks).double().numpy() - oracle.forward(wrong, sd, toks)).max()
    assert d > 1e-2


@pytest.mark.parametrize("device", DEVICES)
def test_routing(device):
    """Sigmoid scores: the correction decides who is chosen and does not enter the weights; the weights are
    renormalised over the chosen ones and scaled; scores all near zero; ties go to the lower index."""
    g = torch.Generator().manual_seed(1)
    for E, top in ((7, 3), (70, 5), (3, 3), (130, 1)):
        z = torch.randn(40, E, generator=g) * 2.0
        c = torch.randn(E, generator=g)
        z[0] = -90.0                                  # scores around 1e-39: the sum's guard matters
        w, i = mx.route_biased(z.to(device), c.to(device), top, "sigmoid", True, 1.9)
        w, i = w.cpu().double().numpy(), i.cpu().numpy()
        differs = 0
        for t in range(1, 40):
            chosen, wt = oracle.route(z[t].double().numpy(), c.double().numpy(), top, 1.9)
            assert list(i[t]) == list(chosen) and np.abs(w[t] - wt).max() < 1e-5, t
            differs += set(chosen) != set(np.argsort(-z[t].numpy())[:top])
        assert differs > 0 or top == E
        assert np.isfinite(w).all() and w[0].max() < 1e-10
    z = torch.zeros(2, 9)
    w, i = mx.route_biased(z.to(device), torch.zeros(9, device=device), 4, "sigmoid", True, 1.0)
    assert i.tolist() == [[0, 1, 2, 3]] * 2 and (w.cpu() - 0.25).abs().max() < 1e-6
    # without renormalisation the scores themselves, as before
    w, _ = mx.route_biased(z.to(device), torch.zeros(9, device=device), 4, "sigmoid")
    assert (w.cpu() - 0.5).abs().max() < 1e-6
    w, _ = mx.route_biased(z.to(device), None, 4)
    assert (w.cpu() - 1.0 / 9).abs().max() < 1e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 9, 16, 300, 2056])
def test_clamped_unit(device, dtype, n):
    """Gate values above the limit are cut, large negative ones are not; up values are cut on both sides; column
    slices, sizes with and without wide accesses."""
    T = 5
    g = torch.Generator().manual_seed(n)
    buf = (3.0 * torch.randn(T, 2 * n + 8, generator=g)).to(dtype)
    out = mx.glu_clamp(buf.to(device)[:, 8:8 + n], buf.to(device)[:, 8 + n:], 1.3, oracle.ALPHA).double().cpu().numpy()
    a, b = buf[:, 8:8 + n].double().numpy(), buf[:, 8 + n:].double().numpy()
    gg, u = np.minimum(a, 1.3), np.clip(b, -1.3, 1.3)
    want = gg * oracle.sigmoid(oracle.ALPHA * gg) * (u + 1)
    assert np.abs(out - want).max() < (1e-5 if dtype == torch.float32 else 3e-2)


@pytest.mark.parametrize("device", DEVICES)
def test_bucketed_experts_match_dense(device, monkeypatch):
    """Rows bucketed by expert (large steps) and every expert over every row (small steps) give the same result,
    also when one expert gets no row, with and without a shared expert."""
    from financial_chatbot_llm_amd.models import mixers as mm
    for shared in (None, {"ff": 24, "limit": 0.8}):
        spec = {"kind": "moe", "expert": {"ff": 20, "limit": 1.1}, "router": {"experts": 6, "top": 2, "scale": 1.4}}
        if shared:
            spec["shared"] = shared
        ff = RoutedFF(spec, 32, score="sigmoid", renorm=True)
        g = torch.Generator().manual_seed(2)
        sd = {k: torch.randn(s, generator=g) * s[-1] ** -0.5 for k, s in ff.shapes().items()}
        sd["correction"] = torch.tensor([0.0, 0.1, -50.0, 0.0, 0.0, 0.0])          # expert 2 is never chosen
        w_in = ff.load(lambda k: sd[k].to(device), torch.float32)
        h = torch.randn(37, 32, generator=g)
        hd = h.to(device)
        proj = torch.nn.functional.linear(hd, w_in) if w_in is not None else None
        monkeypatch.setattr(mm, "DENSE_MAX_PAIRS", 512)
        a = ff.forward(hd, proj).cpu()
        monkeypatch.setattr(mm, "DENSE_MAX_PAIRS", 1)
        b = ff.forward(hd, proj).cpu()
        want = oracle.experts_ff(h.double().numpy(), oracle.as_arrays(sd), "", spec)
        for got in (a, b):
            assert np.abs(got.double().numpy() - want).max() < 1e-4 * np.abs(want).max()


# ---------------------------------------------------------------------------------------------------
# generation through the engine's own scheduler
# ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device,graphs", [("cpu", False), pytest.param("cuda", False, marks=pytest.mark.gpu),
                                           pytest.param("cuda", True, marks=pytest.mark.gpu)])
@pytest.mark.parametrize("async_", [False, True])
def test_greedy_generation(device, graphs, async_):
    cfgd = small_config("AEkK", vocab=256)
    eng, sd = build(cfgd, device, torch.float32, blocks_=12, seqs=2, graphs=graphs, async_=async_)
    poison(eng)
    prompts = [tokens(70, 256, 41), tokens(9, 256, 42), tokens(30, 256, 43)]     # three requests, two slots
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert o == oracle.greedy(cfgd, sd, p, 12)
    assert eng.state_slots.num_free() == 2 and eng.bm.num_free() == eng.bm.num_blocks
    if graphs:
        assert eng.runner.stats["graph_steps"] > 0


@pytest.mark.gpu
def test_sampling_with_the_fused_head():
    """A width the fused LM-head sampler accepts, bf16, decode graphs."""
    cfgd = small_config("AK", width=256, vocab=512)
    cfgd["layers"][1]["mixer"]["kv_from"] = 0
    eng, sd = build(cfgd, "cuda", torch.bfloat16, graphs=True)
    outs = eng.generate([tokens(20, 512, 1)], SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))
    assert len(outs[0]) == 6


def test_preemption_recomputes_state():
    """A pool too small for both sequences: the younger one is preempted, gives its slot back and is
    recomputed from its first token."""
    cfgd = small_config("Ak", vocab=256)
    eng, sd = build(cfgd, "cpu", torch.float32, blocks_=3, seqs=2)
    prompts = [tokens(60, 256, 51), tokens(62, 256, 52)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True))
    assert eng.scheduler.num_preemptions > 0
    for p, o in zip(prompts, outs):
        assert o == oracle.greedy(cfgd, sd, p, 10)


def test_registry_and_config_errors():
    from financial_chatbot_llm_amd.models import get_model_config
    c = get_model_config("fanotar-tiny")
    assert c.arch == "fanotar" and len(c.layers) == c.num_layers

    def bad(change):
        cfgd = copy.deepcopy(example_config())
        change(cfgd["layers"])
        with pytest.raises(ValueError):
            FanotarModel(layered_config(cfgd, "bad"), device="cpu")

    bad(lambda L: L[0].update(type="window_attention"))                # another design's mixer
    bad(lambda L: L[0]["mlp"].update(kind="other"))
    bad(lambda L: L[0]["mixer"].update(heads=5))                       # heads must split into kv_heads
    bad(lambda L: L[0]["mixer"].update(conv=17))
    bad(lambda L: L[1]["mlp"]["router"].update(top=8))
    bad(lambda L: L[2]["mixer"].update(kv_from=2))                     # itself, a later layer, one without its own
    bad(lambda L: L[2]["mixer"].update(kv_from=3))
    bad(lambda L: L[3]["mixer"].update(kv_from=2))
    bad(lambda L: L[2]["mixer"].update(dim=20))                        # sizes unlike the source layer's
    bad(lambda L: L[2]["mixer"].update(heads=4))
    m = FanotarModel(layered_config(example_config(), "ok"), device="cpu")
    sd = random_weights(m, 0)
    assert sd["l0.norm1b.alpha"].shape == () and "embed.norm.b" in sd and "l2.mix.v" not in sd
    m.load_state(sd)
    short = dict(sd)
    short["l0.mix.g"] = sd["l0.mix.g"][:1]
    with pytest.raises(ValueError):
        m.load_state(short)
    short = dict(sd)
    short.pop("final.norm.alpha")
    with pytest.raises(KeyError):
        m.load_state(short)
    m.init_random(seed=3)                            # registry examples run with random weights
    with pytest.raises(ValueError):
        mx.window_attend(torch.zeros(1, 4), torch.zeros(64, 8), i32([0, 1]), i32([0]), i32([[0]]), 4, 1.0, 1, 1, 1, 4, 4,
                         head_bias=torch.zeros(1), sink=torch.zeros(1))
