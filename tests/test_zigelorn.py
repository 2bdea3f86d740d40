"""The Zigelorn design in the engine against its plain whole-sequence implementation (``plain_zigelorn.py``):
every mechanism alone through the kernels' entry points, then whole models through the step function (whole
prompts, decoding token by token, portions down to two tokens, unequal requests side by side on few pages and
slots that are used again), and greedy generation through the entry point and its scheduler. Every test runs on
the CPU stand-in for the kernels (the engine's logic) and, marked ``gpu``, on the HIP kernels in both element types.
"""
import json
import math

import pytest
import torch

import plain_zigelorn as plain
import zigelorn_cases as zc
from helpers import first_difference, max_abs_diff
from nanohybrid_vlm_amd.config.model_config import ConfigError
from nanohybrid_vlm_amd.config.registry import resolve_architecture
from nanohybrid_vlm_amd.engine.replay import replay
from nanohybrid_vlm_amd.engine.runner import ModelRunner
from nanohybrid_vlm_amd.native import ops
from nanohybrid_vlm_amd.native.ops import AttentionBatch

CPU = ("cpu", "float32")
ON_GPU = [pytest.param(("cuda:0", "float32"), marks=pytest.mark.gpu, id="gpu-float32"),
          pytest.param(("cuda:0", "bfloat16"), marks=pytest.mark.gpu, id="gpu-bfloat16")]
WHERE = [pytest.param(CPU, id="cpu-stand-in")] + ON_GPU


@pytest.fixture()
def kernels(request):
    """The kernel library for the test's device: the CPU stand-in, or the HIP library (then a GPU is needed)."""
    device, _ = request.getfixturevalue("where")
    if device == "cpu":
        from emulated_kernels import EmulatedBackend
        old = ops._backend
        ops.set_backend(EmulatedBackend())
        yield
        ops.set_backend(old)
    else:
        if not torch.cuda.is_available():
            pytest.skip("no GPU here")
        old = ops._backend
        ops.set_backend(None)
        yield
        ops.set_backend(old)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: zc.write_model(str(tmp_path_factory.mktemp(f"zigelorn_{name}")), cfg, seed)
            for name, (cfg, seed) in zc.CASES.items()}


def _dt(name):
    return {"float32": torch.float32, "bfloat16": torch.bfloat16}[name]


def _tol(dtype, plain_values, fine=2e-5, coarse=4e-2):
    """Largest allowed difference, as a share of the spread of the plain values."""
    return (fine if dtype == "float32" else coarse) * float(plain_values.float().std())


def _batch(device, counts, starts):
    """An attention batch of requests that bring ``counts`` tokens from ``starts`` on."""
    cu = [0]
    for n in counts:
        cu.append(cu[-1] + n)
    positions = torch.cat([torch.arange(s, s + n) for n, s in zip(counts, starts)]).to(torch.int32)
    req = torch.repeat_interleave(torch.arange(len(counts)), torch.tensor(counts)).to(torch.int32)
    return AttentionBatch(num_tokens=cu[-1], num_requests=len(counts), token_req=req.to(device), positions=positions.to(device),
                          cu_seqlens_q=torch.tensor(cu, dtype=torch.int32).to(device),
                          context_lens=torch.tensor([s + n for n, s in zip(counts, starts)], dtype=torch.int32).to(device),
                          max_q_len=max(counts), max_context_len=max(s + n for n, s in zip(counts, starts)))


# how requests "a", "b", "c" of 75, 33 and 9 tokens are cut into steps: portions that end inside chunks of 16 and at their
# ends, single tokens, steps of up to four tokens and of more, requests that leave steps out
PLAN = [{"a": 5, "b": 1}, {"a": 1}, {"b": 2, "a": 2, "c": 3}, {"c": 1, "a": 16}, {"a": 4, "b": 4, "c": 1}, {"b": 17, "c": 2},
        {"a": 1, "b": 1, "c": 1}, {"c": 1, "b": 8, "a": 33}, {"a": 13}]
LENGTHS = {"a": 75, "b": 33, "c": 9}


def _run_in_steps(device, slot_of, plan, lengths, one_step):
    """``one_step(batch, slots, rows of {request: (first, end)})`` -> [tokens, ...] on the CPU; returns {request: rows}."""
    at, got = {r: 0 for r in lengths}, {r: [] for r in lengths}
    for step in plan:
        reqs = list(step)
        batch = _batch(device, [step[r] for r in reqs], [at[r] for r in reqs])
        slots = torch.tensor([slot_of[r] for r in reqs], dtype=torch.int32).to(device)
        y = one_step(batch, slots, {r: (at[r], at[r] + step[r]) for r in reqs})
        first = 0
        for r in reqs:
            got[r].append(y[first:first + step[r]])
            first += step[r]
            at[r] += step[r]
    assert at == lengths
    return {r: torch.cat(rows) for r, rows in got.items()}


# ------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("where", WHERE)
def test_norms_around_one(where, kernels):
    """The norm's weight is stored as its distance from one: stored zeros leave the row over its root mean square."""
    from nanohybrid_vlm_amd.parts.base import NORMS
    device, dtype = where
    g = torch.Generator().manual_seed(1)
    x = torch.randn(5, 70, generator=g) * 3
    for weight in (torch.zeros(70), 0.3 * torch.randn(70, generator=g)):
        norm = NORMS.build({"kind": "stream_rmsnorm", "size": 70, "eps": 1e-3, "zero_centred": True})
        norm.bind({"weight": weight.to(device)})
        got = norm.forward(x.to(device), _dt(dtype))
        want = plain.zero_centred_norm(x, weight, 1e-3)
        assert max_abs_diff(got.float().cpu(), want) <= _tol(dtype, want, 2e-6, 1e-2)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("W", [40, 37])
def test_token_shift(where, kernels, W):
    """Every mix of every row with the row before it, over requests cut into steps; a slot that held numbers before starts
    from zeros again."""
    device, dtype = where
    dt = _dt(dtype)
    g = torch.Generator().manual_seed(W)
    x = {r: torch.randn(n, W, generator=g).to(dt) for r, n in LENGTHS.items()}
    mu = torch.randn(3, W, generator=g)
    kept = torch.full((4, W), float("nan")).to(device)
    for slot_of in ({"a": 2, "b": 0, "c": 1}, {"a": 0, "b": 1, "c": 2}):
        def one(batch, slots, rows):
            h = torch.cat([x[r][a:b] for r, (a, b) in rows.items()]).to(device)
            return ops.token_shift(h, mu.to(device), kept, batch, slots).float().cpu().transpose(0, 1)
        got = _run_in_steps(device, slot_of, PLAN, LENGTHS, one)
        for r in LENGTHS:
            before = plain.shifted(x[r].float())
            want = torch.stack([x[r].float() + (before - x[r].float()) * m for m in mu], dim=1)
            bound = 1e-6 + (2.0 ** -8 if dtype == "bfloat16" else 1e-6) * want.abs()
            assert bool(((got[r] - want).abs() <= bound).all()), r


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("rows,band,last,K", [(1, 16, 5, 40), (8, 32, 64, 128), (16, 48, 1, 64), (5, 24, 7, 40), (3, 16, 8, 36), (40, 32, 8, 64), (17, 64, 3, 200),
                                                    (64, 32, 40, 72), (20, 48, 8, 64), (65, 32, 4, 64)])
def test_products_in_bands(where, kernels, rows, band, last, K):
    """Outputs made from several sets of rows, in one kernel for few rows and sizes that it takes, else product by product."""
    device, dtype = where
    dt = _dt(dtype)
    g = torch.Generator().manual_seed(rows)
    x = torch.randn(5, rows, K, generator=g).to(dt)
    w = (torch.randn(4 * band + last, K, generator=g) / K ** 0.5).to(dt)
    got = ops.banded_linear(x.to(device), w.to(device), band)
    assert len(got) == 5 and got[4].dtype == torch.float32
    for i in range(5):
        want = x[i].float() @ w[i * band:(4 * band + last if i == 4 else (i + 1) * band)].float().T
        assert got[i].shape == want.shape
        assert max_abs_diff(got[i].float().cpu(), want) <= _tol(dtype, want, 1e-5, 3e-2), i


def _attention_through_kernels(device, dtype, m, eps, q_in, k_in, b, wq, wk, portions, page_size):
    """q_in [T, H D], k_in [T, G D] as projected without their biases ``b``: normed, turned, stored and read back by the kernels
    in the given portions of one request, on pages handed out in a scrambled order."""
    from nanohybrid_vlm_amd.parts.positions import YarnFrequencies
    T = q_in.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    n_pages = -(-T // page_size)
    pages = torch.randperm(n_pages + 2, generator=torch.Generator().manual_seed(T)).tolist()[:n_pages]
    dt = _dt(dtype)
    k_cache = torch.full((n_pages + 2, page_size, G, D), float("nan"), dtype=dt).to(device)
    v_cache = torch.full((n_pages + 2, page_size, G, D), float("nan"), dtype=dt).to(device)
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    pos = YarnFrequencies(rot["dims"], rot["base"], 1 << 20, **(rot.get("scaling") or {}), device=device)
    packed = torch.cat((q_in, k_in), dim=1).to(dt).to(device)
    outs, at = [], 0
    for n in portions:
        batch = _batch(device, [n], [at])
        slots = torch.tensor([pages[p // page_size] * page_size + p % page_size for p in range(at, at + n)], dtype=torch.int32).to(device)
        q = ops.normed_split_write(packed[at:at + n].contiguous(), b.to(dt).to(device), wq.to(device), wk.to(device), eps,
                                   pos.frequencies() if rot["dims"] else None, pos.gain(), batch.positions, slots, k_cache, v_cache,
                                   H, G, D, D, values_from_keys=True)
        o = ops.paged_attention(q, k_cache, v_cache, batch, torch.tensor([pages], dtype=torch.int32).to(device), m["scale"],
                                (m.get("mask") or {}).get("size"))
        outs.append(o.float().cpu())
        at += n
    return torch.cat(outs)


def _plain_attention(m, eps, q_in, k_in, b, wq, wk):
    T, H, G, D = q_in.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = q_in.double() + b[:H * D].double(), k_in.double() + b[H * D:].double()
    qn = plain.turn((plain.over_rms(q, eps) * wq.double()).view(T, H, D), m.get("rot"))
    kn = plain.turn((plain.over_rms(k, eps) * wk.double()).view(T, G, D), m.get("rot"))
    return plain.windowed_softmax(qn, kn, k.view(T, G, D), m["scale"], (m.get("mask") or {}).get("size")).float()


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sizes", [(12, 3, 12), (32, 2, 16), (16, 6, 16), (64, 1, 6), (20, 2, 0)], ids=lambda s: "D%d-group%d-rot%d" % s)
@pytest.mark.parametrize("window", [7, 40, None])
def test_attention_with_projections_normed_as_a_whole(where, kernels, sizes, window):
    """Random projections with biases: the norm over all heads at once (before the split: a norm head by head gives other
    results), the scaled rotation and its gain, values that are the keys before norm and rotation, windows."""
    device, dtype = where
    D, group, rot = sizes
    m = zc.attention(2 * group, 2, D, window, 1.0 * D ** -0.5, rot, 300.0, (4.0, 50, 8.0, 0.5))["mixer"]
    g = torch.Generator().manual_seed(5)
    T, eps = 90, 1e-4
    spread = torch.linspace(0.3, 3.0, 2 * group).repeat_interleave(D)         # (heads of unequal size)
    q_in, k_in = torch.randn(T, 2 * group * D, generator=g) * spread, torch.randn(T, 2 * D, generator=g)
    b, wq, wk = 0.5 * torch.randn((2 * group + 2) * D, generator=g), torch.rand(2 * group * D, generator=g) + 0.8, torch.rand(2 * D, generator=g) + 0.8
    if dtype == "bfloat16":
        q_in, k_in, b = (t.bfloat16().float() for t in (q_in, k_in, b))
    want = _plain_attention(m, eps, q_in, k_in, b, wq, wk)
    for portions in ([T], [1] * T, [2, 5, 3, 11, 1, 2, 21, 45]):
        got = _attention_through_kernels(device, dtype, m, eps, q_in, k_in, b, wq, wk, portions, 4)
        bound = _tol(dtype, want, coarse=7e-2)
        assert max_abs_diff(got, want) <= bound, (portions, first_difference(got.flatten(1), want.flatten(1), bound))


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("D", [16, 12])
def test_one_key_that_stands_out_under_a_window(where, kernels, D):
    """Among 300 keys one is made to carry nearly all the weight of every query that sees it, and as the values are the keys
    it is also what such a query returns. So a query returns it exactly when it lies among the last ``window`` positions up
    to its own: for the marked key at the first place, at a page's border and far back, and for queries just inside and just
    outside, in a prompt and decoded one by one. No rotation, so the scores are known."""
    device, dtype = where
    window, page, T = 48, 16, 300
    m = zc.attention(2, 1, D, window, 8.0)["mixer"]
    for marked in (0, 15, 16, 47, 48, 100, 191, 240, 251):
        g = torch.Generator().manual_seed(marked)
        q_in, k_in = 0.05 * torch.randn(T, 2 * D, generator=g), 0.05 * torch.randn(T, D, generator=g)
        q_in[:, 0] = q_in[:, D] = 1.0
        k_in[:, 1] = 1.0                              # every key points along coordinate 1 ...
        k_in[marked, 0], k_in[marked, 1] = 3.0, 0.0   # ... but the marked one, which the queries ask for
        ones = torch.ones
        for portions in ([T], [marked + 1] + [1] * (T - marked - 1) if marked < 200 else [T - 60] + [1] * 60):
            got = _attention_through_kernels(device, dtype, m, 1e-6, q_in, k_in, torch.zeros(3 * D), ones(2 * D), ones(D), portions, page)
            sees = torch.tensor([0 <= i - marked < window for i in range(T)])
            hit = (got[:, 0, 0] > 2.5) & (got[:, 1, 0] > 2.5)
            assert torch.equal(hit, sees), (marked, len(portions), (hit != sees).nonzero().flatten().tolist())
            assert got[~sees][:, :, 0].abs().max() < 0.5


def test_scaled_frequencies():
    """Fast pairs keep their frequency, slow ones have it divided, and between them a ramp leads over; also where both
    borders fall together and where no pair lies on one side."""
    from nanohybrid_vlm_amd.parts.positions import YarnFrequencies
    for dims, base, scaling in ((32, 10000.0, (8.0, 4096, 32.0, 1.0)), (16, 500.0, (2.0, 64, 8.0, 8.0)), (8, 1e6, (4.0, 16, 100.0, 0.01)),
                                (64, 300.0, (40.0, 100000, 32.0, 1.0)), (10, 1000.0, None)):
        named = None if scaling is None else dict(zip(("factor", "original", "fast", "slow"), scaling))
        got = YarnFrequencies(dims, base, 1 << 20, **(named or {}))
        want, gain = plain.pair_frequencies(dims, base, named, torch.float64)
        assert torch.allclose(got.frequencies(), want, rtol=1e-12) and got.gain() == pytest.approx(gain, abs=1e-12)


def _retention_case(g, T, H, D, E):
    return {"q": torch.randn(T, H * D, generator=g), "k": torch.randn(T, H * D, generator=g), "v": torch.randn(T, H * E, generator=g),
            "g": torch.randn(T, H * E, generator=g)}


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sizes", [(2, 8, 6, 4), (1, 3, 5, 2), (3, 20, 40, 20), (2, 64, 48, 32), (1, 128, 144, 128), (2, 18, 16, 6), (1, 256, 20, 0)],
                         ids=lambda s: "H%d-D%d-E%d-rot%d" % s)
@pytest.mark.parametrize("apart", [False, True], ids=["packed", "apart"])
def test_retention_alone(where, kernels, sizes, apart):
    """Three requests of unequal length side by side, cut into steps (in chunks, and token by token for steps of few tokens),
    against the recurrence written out token by token; then the slots are used again by new requests, which must start from
    zero. Decays of 0, of 1 and between; projections as columns of one tensor and as tensors of their own."""
    device, dtype = where
    H, D, E, rot = sizes
    dt, eps = _dt(dtype), 1e-5
    decay = [0.97, 1.0, 0.0][:H] if H != 1 else [0.9]
    g = torch.Generator().manual_seed(D)
    x = {r: {n: t.to(dt) for n, t in _retention_case(g, T, H, D, E).items()} for r, T in LENGTHS.items()}
    spec = {"dims": rot, "base": 50.0}
    want = {}
    for r, T in LENGTHS.items():
        q, k, v = (x[r][n].double().view(T, H, -1) for n in "qkv")
        o = plain.decayed_memory(plain.turn(q, spec), plain.turn(k, spec) * D ** -0.5, v, decay)
        want[r] = (plain.over_rms(o, eps).reshape(T, H * E) * plain.silu(x[r]["g"].double())).float()
    log2 = torch.tensor([math.log2(max(d, 2.0 ** -1000)) for d in decay], dtype=torch.float32).to(device)
    freqs = plain.pair_frequencies(rot, 50.0, None, torch.float64)[0].to(device) if rot else None
    state = torch.full((4, H, E, D), float("nan")).to(device)
    for slot_of in ({"a": 2, "b": 0, "c": 1}, {"a": 0, "b": 1, "c": 2}):
        def one(batch, slots, rows):
            parts = [torch.cat([x[r][n][a:b] for r, (a, b) in rows.items()]) for n in "qkvg"]
            if apart and E == D:
                q, k, v, gate = (t.contiguous().to(device) for t in parts)
            else:
                packed = torch.cat(parts, dim=1).to(device)
                q, k, v, gate = packed.split([H * D, H * D, H * E, H * E], dim=1)
            rule = ops.Retention(log2, freqs, batch.positions, D ** -0.5)
            return ops.linear_recurrence(rule, q, k, v, gate, state, eps, batch, slots, dt).float().cpu()
        got = _run_in_steps(device, slot_of, PLAN, LENGTHS, one)
        for r in LENGTHS:
            # (where a read-out nearly vanishes, its division by its own size lets float rounding through)
            bound = _tol(dtype, want[r], 3e-4, 5e-3) + (2.0 ** -8 * want[r].abs() if dtype == "bfloat16" else 0.0)
            assert bool(((got[r] - want[r]).abs() <= bound).all()), (r, first_difference(got[r], want[r], 1e-3))


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sizes", [(2, 8, 4), (1, 3, 1), (3, 20, 9), (2, 64, 40), (1, 128, 64), (2, 18, 33), (1, 256, 16)],
                         ids=lambda s: "H%d-D%d-rank%d" % s)
@pytest.mark.parametrize("w0", [-2.0, 2.0], ids=["slow decays", "strong decays"])
def test_wkv_alone(where, kernels, sizes, w0):
    """The same for the recurrence with decays per channel and token. With w0 around 2 a channel decays by e^-7 and much more
    in one token: products over sixteen tokens leave every float's range, and what is kept must be zeros, not
    infinities."""
    device, dtype = where
    H, D, R = sizes
    dt, eps = _dt(dtype), 1e-5
    g = torch.Generator().manual_seed(R)
    n = H * D
    w2 = (torch.randn(n, R, generator=g) * 1.5 / R ** 0.5).to(dt)
    w0_t = w0 + 1.5 * torch.randn(n, generator=g)
    u, norm = 0.5 + torch.randn(H, D, generator=g), 1.0 + 0.2 * torch.randn(n, generator=g)
    x = {r: dict({name: torch.randn(T, n, generator=g).to(dt) for name in "rkvg"}, z=2.0 * torch.randn(T, R, generator=g))
         for r, T in LENGTHS.items()}
    want = {}
    for rid, T in LENGTHS.items():
        r, k, v = (x[rid][name].double().view(T, H, D) for name in "rkv")
        lin = torch.tanh(x[rid]["z"].double()) @ w2.double().T + w0_t.double()
        o = plain.bonus_memory(r, k, v, torch.exp(-torch.exp(lin)).view(T, H, D), u.double())
        want[rid] = (plain.over_rms(o, eps).reshape(T, n) * norm.double() * plain.silu(x[rid]["g"].double())).float()
    state = torch.full((4, H, D, D), float("nan")).to(device)
    for slot_of in ({"a": 2, "b": 0, "c": 1}, {"a": 0, "b": 1, "c": 2}):
        def one(batch, slots, rows):
            r, k, v, gate, z = (torch.cat([x[q][name][a:b] for q, (a, b) in rows.items()]).to(device) for name in ("r", "k", "v", "g", "z"))
            rule = ops.WKV(z, w2.to(device), w0_t.to(device), u.to(device))
            return ops.linear_recurrence(rule, r, k, v, gate, state, eps, batch, slots, dt, norm_weight=norm.to(device)).float().cpu()
        got = _run_in_steps(device, slot_of, PLAN, LENGTHS, one)
        for r in LENGTHS:
            bound = _tol(dtype, want[r], 3e-4, 5e-3) + (2.0 ** -8 * want[r].abs() if dtype == "bfloat16" else 0.0)
            assert bool(((got[r] - want[r]).abs() <= bound).all()), (r, first_difference(got[r], want[r], 1e-3))
    # one product's float columns as they come (rows further apart than their entries)
    T = LENGTHS["c"]
    packed = torch.cat([x["c"][name].float() for name in ("r", "k", "v", "g", "z")], dim=1).to(device)
    r, k, v, gate, z = packed.split([n, n, n, n, R], dim=1)
    outs, at = [], 0
    for count in (2, 5, 1, 1):
        rows = slice(at, at + count)
        rule = ops.WKV(z[rows], w2.to(device), w0_t.to(device), u.to(device))
        outs.append(ops.linear_recurrence(rule, r[rows], k[rows], v[rows], gate[rows], state, eps, _batch(device, [count], [at]),
                                          torch.tensor([3], dtype=torch.int32).to(device), dt, norm_weight=norm.to(device)).float().cpu())
        at += count
    got = torch.cat(outs)
    bound = _tol(dtype, want["c"], 3e-4, 5e-3) + (2.0 ** -8 * want["c"].abs() if dtype == "bfloat16" else 0.0)
    assert at == T and bool(((got - want["c"]).abs() <= bound).all())


@pytest.mark.parametrize("where", WHERE)
def test_a_value_written_far_back_is_read_from_the_state(where, kernels):
    """One token writes a value under a key that no other token uses, with decays of (nearly) 1. Every later query that asks
    for that key reads that value back from the state, hundreds of tokens later, whatever the portions were (the slot held
    no numbers before); a query before the marked token reads nothing of it. For both recurrences; the one with a bonus reads
    its own token's value through the bonus alone (u = 0 for the marked key: not at all)."""
    device, dtype = where
    dt = _dt(dtype)
    H, D, T, marked = 2, 16, 400, 37
    g = torch.Generator().manual_seed(4)
    q, k = torch.zeros(T, H, D), 0.5 * torch.randn(T, H, D, generator=g)
    q[:, :, 0] = 1.0
    k[:, :, 0] = 0.0
    k[marked] = 0.0
    k[marked, :, 0] = 2.0
    v = 0.3 * torch.randn(T, H, D, generator=g)
    v[marked] = torch.tensor([3.0, -3.0] * (D // 2))
    v = v.to(dt).float()
    gate = torch.full((T, H * D), 2.0)
    shown = v[marked] / v[marked].pow(2).mean(-1, keepdim=True).sqrt() * float(plain.silu(torch.tensor(2.0)))
    rows = [t.reshape(T, -1).to(dt).to(device) for t in (q, k, v, gate)]
    z, w2 = torch.zeros(T, 4).to(device), torch.zeros(H * D, 4, dtype=dt).to(device)
    for kind in ("retention", "wkv"):
        for portions in ([T], [marked] + [1] * 20 + [T - marked - 20], [2, 33, 5, 1, 1, 200, 1, 1, 156]):
            state, at, outs = torch.full((3, H, D, D), float("nan")).to(device), 0, []
            for n in portions:
                batch, part = _batch(device, [n], [at]), slice(at, at + n)
                rule = ops.Retention(torch.zeros(H).to(device), None, batch.positions) if kind == "retention" else \
                    ops.WKV(z[part], w2, torch.full((H * D,), -20.0).to(device), torch.zeros(H, D).to(device))
                outs.append(ops.linear_recurrence(rule, *(t[part] for t in rows), state, 1e-6, batch,
                                                  torch.tensor([1], dtype=torch.int32).to(device), dt).float().cpu().view(n, H, D))
                at += n
            got = torch.cat(outs)
            first = marked if kind == "retention" else marked + 1
            close = ((got[first:] - shown).abs() < 0.03).all(-1).all(-1)
            assert bool(close.all()), (kind, portions, first + int((~close).nonzero()[0]))
            assert float(got[:first].abs().max()) < 1e-2, (kind, portions)


@pytest.mark.parametrize("where", WHERE)
def test_choice_among_groups_of_experts(where, kernels):
    """Scores over all experts, the correction in the choice alone, groups by their best choice score (negative ones among
    them: a closed group's experts never win), numbers that stand for identity experts."""
    device, _ = where
    g = torch.Generator().manual_seed(8)
    for E, top, count, keep in ((18, 4, 2, 1), (8, 3, 4, 2), (6, 6, 1, 1), (1, 1, 1, 1), (12, 2, 12, 3), (96, 5, 8, 3), (1200, 7, 6, 2)):
        z = 2.0 * torch.randn(50, E, generator=g)
        for correction in (None, 0.3 * torch.randn(E, generator=g), -1.0 - torch.rand(E, generator=g)):
            ids, scores = ops.route_groups(z.to(device), top, None if correction is None else correction.to(device), count, keep)
            for t in range(50):
                chosen, s = plain.choose(z[t], torch.zeros(E) if correction is None else correction, top, count, keep)
                assert ids[t].tolist() == chosen, (E, t)
                assert max_abs_diff(scores[t].cpu(), s[chosen]) <= 1e-6
    with pytest.raises(ops.KernelError):
        ops.route_groups(z.to(device), 401, None, 6, 2)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("T", [1, 5, 16, 17, 70, 300])
@pytest.mark.parametrize("sizes", [(40, 24, 5, 2), (36, 10, 3, 4), (64, 48, 4, 1)], ids=lambda s: "W%d-F%d-E%d-same%d" % s)
def test_experts_without_a_gate_and_identity_experts(where, kernels, T, sizes):
    """Experts D relu(U x)^2 and experts that hand their input on, weighed by their scores: few rows, and rows sorted by
    expert in tiles of 16, 64 and 128."""
    device, dtype = where
    W, F, E, same = sizes
    dt = _dt(dtype)
    if device == "cpu" and T > 70:
        pytest.skip("the stand-in has one way for any number of rows")
    g = torch.Generator().manual_seed(T + W)
    h = torch.randn(T, W, generator=g).to(dt)
    up, down = (torch.randn(E, F, W, generator=g) * 1.5 / W ** 0.5).to(dt), (torch.randn(E, W, F, generator=g) / F ** 0.5).to(dt)
    top = min(3, E + same)
    ids = torch.stack([torch.randperm(E + same, generator=g)[:top] for _ in range(T)]).to(torch.int32)
    if T > 16:
        ids[:8, 0] = E                                      # (tokens whose experts are all identities, where there are enough)
        ids[:8, 1:] = torch.arange(1, top)[None] % same + E
    scores = torch.rand(T, top, generator=g)
    want = torch.zeros(T, W)
    for t in range(T):
        for j in range(top):
            e = int(ids[t, j])
            x = h[t].float()
            y = x if e >= E else down[e].float() @ (torch.relu(up[e].float() @ x) ** 2)
            want[t] += scores[t, j] * y
    got = ops.routed_experts(h.to(device), ids.to(device), scores.to(device), up.to(device), down.to(device), "relu2",
                             scores_on="output", gated=False, identity=True)
    # (in bfloat16 an expert's inner row is rounded before its second product)
    bound = _tol(dtype, want, 2e-5, 3e-2) + (2.0 ** -7 * want.abs() if dtype == "bfloat16" else 0.0)
    assert bool(((got.float().cpu() - want).abs() <= bound).all()), first_difference(got.float().cpu(), want, 1e-2)


# ------------------------------------------------------------------ configuration and weights
def test_configuration_and_names():
    from nanohybrid_vlm_amd.parts.base import PagedKVNeed, StateNeed
    from nanohybrid_vlm_amd.parts.model import DecoderModel
    arch = resolve_architecture(zc.CONFIG_A)
    assert arch.name == "Zigelorn"
    for config in (zc.CONFIG_A, zc.CONFIG_B, zc.CONFIG_C, zc.CONFIG_W):
        tensors = zc.random_tensors(config, 0)
        cfg = arch.parse_config(config, {k: tuple(t.shape) for k, t in tensors.items()})
        model = DecoderModel(arch.build_spec(cfg))
        # every stored tensor has its place, and every parameter is filled by stored tensors
        names = arch.checkpoint_names(cfg)
        assert set(names) == set(tensors)
        assert {s.param for s in names.values()} == set(model.all_param_specs())
    tensors = zc.random_tensors(zc.CONFIG_A, 0)
    shapes = {k: tuple(t.shape) for k, t in tensors.items()}
    cfg = arch.parse_config(zc.CONFIG_A, shapes)
    assert cfg.owners() == [0, 1, 2, 4] and cfg.layers[5].weights_of == 0 and cfg.layers[0].mixer.decay_rank == 3
    spec = arch.build_spec(cfg)
    assert [e.layer for e in spec.order()] == [0, 1, 2, 1, 3, 0] and all(e.cache is None for e in spec.order())
    # every run of a layer has pages or a state of its own, also where two runs share their weights
    needs = DecoderModel(spec).cache_needs()
    assert isinstance(needs[1], PagedKVNeed) and needs[1] == needs[3] and needs[1].window == 6
    assert isinstance(needs[0], StateNeed) and set(needs[0].tensors) == {"S", "row"} and needs[5] == needs[0]
    # a checkpoint may store the norms of a feed-forward that a layer does not have
    spare = dict(shapes, **{"l2.norm2": (40,), "l2.norm2b": (40,)})
    cfg = arch.parse_config(zc.CONFIG_A, spare)
    assert set(arch.checkpoint_names(cfg)) == set(spare)
    assert {s.param for s in arch.checkpoint_names(cfg).values()} == set(DecoderModel(arch.build_spec(cfg)).all_param_specs())
    chain = json.loads(json.dumps(zc.CONFIG_A))
    chain["layers"].append(dict(chain["layers"][3], weights_of=3))                # (layer 3 itself runs layer 1's weights)
    assert arch.parse_config(chain, shapes).layers[6].weights_of == 1
    for change, match in ((lambda c: c["layers"][5].update(weights_of=5), "weights_of"),
                          (lambda c: c["layers"][5].update(weights_of=1), "must equal"),
                          (lambda c: c["layers"][1].update(type="other"), "not known"),
                          (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3), "rot.dims"),
                          (lambda c: c["layers"][1]["mixer"].update(vdim=4), "vdim"),
                          (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "mask.size"),
                          (lambda c: c["layers"][2]["mixer"].update(decay=[0.5]), "decay"),
                          (lambda c: c["layers"][2]["mixer"].update(decay=[0.5, 1.5]), "decay"),
                          (lambda c: c["layers"][2]["mixer"]["rot"].update(scaling={"factor": 2.0}), "scaling"),
                          (lambda c: c["layers"][4]["mlp"]["router"].update(identity=1), "router"),
                          (lambda c: c["layers"][4]["mlp"]["router"].update(top=7), "router")):
        bad = json.loads(json.dumps(zc.CONFIG_A))
        change(bad)
        with pytest.raises(ConfigError, match=match):
            arch.parse_config(bad, shapes)
    with pytest.raises(ConfigError, match="decay_rank"):
        arch.parse_config(zc.CONFIG_A)


# ------------------------------------------------------------------ whole models through the step function
def _requests(name, lengths):
    vocab = zc.CASES[name][0]["vocab"]
    return {f"r{i}": zc.tokens(vocab, n, 100 * i + n) for i, n in enumerate(lengths)}


def _plain_logits(folder, requests, dtype=torch.float64):
    """(in float64: what the comparison then shows is the engine's own rounding, not the oracle's)"""
    cfg, w = plain.read_model_folder(folder)
    return {rid: plain.logits(cfg, w, toks, dtype).float() for rid, toks in requests.items()}


def _replay(folder, where, steps, page_size, max_live, **options):
    device, dtype = where
    for i, s in enumerate(steps):
        s["step"] = i
    pages = max(1, zc.peak_tokens(steps, page_size) // page_size)
    runner = ModelRunner(folder, dtype=dtype, device=device, page_size=page_size, num_pages=pages, num_state_slots=max_live,
                         max_model_len=pages * page_size, poison_freed_pages=True, **options)
    got = replay(runner, steps)
    assert not runner.cache.requests and all(runner.cache.num_free_pages(g) == pages for g in range(len(runner.cache.groups)))
    return got


def _compare(got, want, dtype, what):
    """float32: every logit within 3e-4 of the logits' spread (a read-out that nearly vanishes is divided by its own size, which
    lets float rounding through). bfloat16: for the same reason single positions of these small models are far off by rounding
    alone, and a router's close call may fall the other way, so the bound is on the positions' errors taken together. What
    it cannot see (one key more or less in a window, a state or a page of another request) shows in the float32 run of the
    same steps and in the tests of the mechanisms alone, which hold the bfloat16 kernels to a close bound."""
    spread = float(torch.cat([t.reshape(-1) for t in want.values()]).float().std())
    if dtype == "float32":
        for rid in want:
            assert max_abs_diff(got[rid], want[rid]) <= 3e-4 * spread, (what, rid, first_difference(got[rid], want[rid], 3e-4 * spread))
        return
    errors = torch.cat([(got[rid].float() - want[rid].float()).abs().max(dim=-1).values for rid in want]) / spread
    assert bool(torch.isfinite(errors).all()), what
    assert float(errors.median()) <= 0.12 and float((errors > 0.3).float().mean()) <= 0.2, \
        (what, float(errors.median()), float((errors > 0.3).float().mean()), float(errors.max()))


@pytest.mark.parametrize("where", WHERE)
def test_layers_one_by_one(where, kernels, tmp_path):
    """Models cut off after 1, 2, ... layer runs."""
    device, dtype = where
    for name in ("A", "B"):
        cfg, seed = zc.CASES[name]
        w = zc.random_tensors(cfg, seed)
        toks = zc.tokens(cfg["vocab"], 21, 9)
        for runs in range(1, len(cfg["layers"]) + 1):
            cut = dict(cfg, layers=cfg["layers"][:runs])
            keep = {f"l{i}." for i, layer in enumerate(cut["layers"]) if "weights_of" not in layer}
            tensors = {k: v for k, v in w.items() if not k.startswith("l") or k[:k.index(".") + 1] in keep}
            folder = zc.write_model(str(tmp_path / f"{name}{runs}"), cut, 0, tensors)
            want = _plain_logits(folder, {"a": toks})
            got = _replay(folder, where, zc.in_portions({"a": toks}, [8, 1, 5, 7]), page_size=4, max_live=1)
            _compare(got, want, dtype, f"{name}: {runs} layer runs")


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", ["A", "B", "C", "R"])
def test_ways_of_cutting_agree_with_the_plain_model(folders, where, kernels, name):
    """Whole prompts, a prompt followed by its last tokens one by one, portions of several sizes down to two tokens
    (and single tokens between them), and unequal requests side by side on pages and slots that are used again: all
    give the plain model's logits at every position."""
    device, dtype = where
    lengths = [1, 2, 26, 19, 37, 5, 30] if device == "cpu" else [1, 2, 26, 19, 61, 5, 150, 43]
    requests = _requests(name, lengths)
    want = _plain_logits(folders[name], requests)
    ways = {
        "whole": (zc.whole(requests), 3),
        "tail": ([s for rid, toks in requests.items()
                  for s in zc.in_portions({rid: toks}, [max(1, len(toks) - 12)] + [1] * 12)], 3),
        "portions": (zc.in_portions(requests, [2, 3, 5, 2, 1, 7, 4, 2, 11]), 3),
        "side by side": (zc.interleaved(requests, [3, 1, 2, 6, 1, 1, 4], 3), 3),
    }
    for what, (steps, live) in ways.items():
        got = _replay(folders[name], where, steps, page_size=4, max_live=live)
        _compare(got, want, dtype, what)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(where, kernels, seed, tmp_path):
    """Models of sizes drawn at random (see ``zigelorn_cases.random_config``) in portions, side by side and with a decoded
    tail, on pages of 16 tokens that are used again, against the plain model."""
    device, dtype = where
    cfg = zc.random_config(seed)
    folder = zc.write_model(str(tmp_path / "m"), cfg, 500 + seed)
    lengths = [1, 21, 40, 7] if device == "cpu" else [1, 70, 210, 33, 131]
    requests = {f"r{i}": zc.tokens(cfg["vocab"], n, 7 * i + n) for i, n in enumerate(lengths)}
    want = _plain_logits(folder, requests)
    ways = {"portions": zc.in_portions(requests, [17, 2, 3, 64, 1, 33]),
            "side by side": zc.interleaved(requests, [5, 1, 2, 31, 1, 1, 16], 3),
            "tail": [s for rid, toks in requests.items() for s in zc.in_portions({rid: toks}, [max(1, len(toks) - 20)] + [1] * 20)]}
    for what, steps in ways.items():
        got = _replay(folder, where, steps, page_size=16, max_live=3)
        _compare(got, want, dtype, (seed, what))


@pytest.mark.parametrize("where", ON_GPU)
def test_pages_of_64_and_windows_longer_than_a_page(folders, where, kernels):
    """Pages of 64 tokens (whole tiles of the prompt kernel lie in one page) under windows of 80 and 150 positions,
    requests of up to 400 tokens in portions that end anywhere, beside decoded tokens, on few pages."""
    device, dtype = where
    requests = _requests("S", [400, 130, 70, 257])
    want = _plain_logits(folders["S"], requests)
    for what, steps in (("portions", zc.in_portions(requests, [37, 2, 64, 5, 1, 129, 1, 1, 96])),
                        ("side by side", zc.interleaved(requests, [33, 1, 1, 64, 1, 7, 1, 100], 3))):
        got = _replay(folders["S"], where, steps, page_size=64, max_live=3)
        _compare(got, want, dtype, what)


@pytest.mark.parametrize("where", ON_GPU)
def test_sizes_of_a_real_models_layers(where, kernels, tmp_path):
    """Heads and states of 128, 256 and 64 entries, a width of 1,024: the kernels' makes that real sizes take, in portions and
    side by side on pages of 64, with decoded tokens between."""
    device, dtype = where
    folder = zc.write_model(str(tmp_path / "w"), zc.CONFIG_W, 26)
    requests = {f"r{i}": zc.tokens(zc.CONFIG_W["vocab"], n, 11 * i + n) for i, n in enumerate([300, 40, 129])}
    want = _plain_logits(folder, requests, torch.float32)
    for what, steps in (("portions", zc.in_portions(requests, [150, 1, 1, 16, 3, 64, 1, 1, 1])),
                        ("side by side", zc.interleaved(requests, [40, 1, 1, 1, 17, 1, 64, 1], 3))):
        got = _replay(folder, where, steps, page_size=64, max_live=3)
        _compare(got, want, dtype, what)


@pytest.mark.parametrize("where", WHERE)
def test_long_decoding(folders, where, kernels):
    """Two tokens of prompt, then many tokens one by one: the windows of every layer pass many times, pages go back
    to the pool on the way, and the recurrent states are carried through every step."""
    device, dtype = where
    n = 60 if device == "cpu" else 142
    requests = _requests("A", [n])
    want = _plain_logits(folders["A"], requests)
    got = _replay(folders["A"], where, zc.in_portions(requests, [2] + [1] * n), page_size=4, max_live=1)
    _compare(got, want, dtype, "decoding")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_recorded_steps_equal_eager_steps(folders, dtype):
    """Steps replayed from HIP graphs (single tokens, and short mixed steps) give what eager steps give."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU here")
    old = ops._backend
    ops.set_backend(None)
    try:
        requests = _requests("R", [40, 3, 17, 9])
        steps = zc.interleaved(requests, [3, 1, 1, 1, 2, 1, 1], 3)
        for s in steps:                                      # a recorded short step gives one place a request
            for e in s["entries"]:
                e["want"] = e["want"][-1:]
        where = ("cuda:0", dtype)
        eager = _replay(folders["R"], where, steps, page_size=8, max_live=3, use_graphs=False)
        recorded = _replay(folders["R"], where, steps, page_size=8, max_live=3, use_graphs=True)
        for rid in eager:
            # (a recorded step of two or three tokens a request goes through the chunks' kernels, an eager one does not)
            assert max_abs_diff(eager[rid], recorded[rid]) <= (3e-4 if dtype == "float32" else 0.1) * float(eager[rid].std()), rid
    finally:
        ops.set_backend(old)


# ------------------------------------------------------------------ generation through the entry point
@pytest.mark.parametrize("where", [pytest.param(CPU, id="cpu-stand-in"), ON_GPU[0]])
@pytest.mark.parametrize("options", [dict(kvcache_block_size=4, num_kvcache_blocks=64),
                                     dict(kvcache_block_size=8, num_kvcache_blocks=40, max_num_batched_tokens=7, max_num_seqs=2)],
                         ids=["whole prompts", "portions of 7, two at a time"])
def test_greedy_generation_through_the_entry_point(folders, where, kernels, options):
    from nanohybrid_vlm_amd import LLM, SamplingParams
    device, dtype = where
    cfg, w = plain.read_model_folder(folders["A"])
    prompts = [zc.tokens(cfg["vocab"], n, 300 + n) for n in (1, 13, 22)]
    llm = LLM(folders["A"], device=device, dtype=dtype, **options)
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=9, ignore_eos=True), use_tqdm=False)
    for prompt, out in zip(prompts, outs):
        assert out["token_ids"] == plain.greedy_generate(cfg, w, prompt, 9)
    stats = llm.get_memory_stats()
    assert stats["live_requests"] == 0 and all(g["free_pages"] == g["pages"] for g in stats["groups"])
    assert stats["state_pool_bytes"] > 0


# ------------------------------------------------------------------ the command line
def _command(*args):
    import os
    import subprocess
    import sys
    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, "-m", "nanohybrid_vlm_amd", *args], cwd=repo, capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-3000:]
    return proc.stdout


def test_random_model_of_a_named_shape(tmp_path, emulated_kernels):
    """``random-model --shape zigelorn-tiny`` writes a folder that the plain implementation and the engine both read."""
    out = str(tmp_path / "m")
    _command("random-model", "--out", out, "--shape", "zigelorn-tiny", "--seed", "5")
    cfg, w = plain.read_model_folder(out)
    assert cfg["architecture"] == "Zigelorn" and "l6.norm1" not in w and cfg["layers"][6]["weights_of"] == 2
    requests = {"a": zc.tokens(cfg["vocab"], 31, 1)}
    want = {"a": plain.logits(cfg, w, requests["a"])}
    got = _replay(out, CPU, zc.in_portions(requests, [4, 1, 9]), page_size=8, max_live=1)
    _compare(got, want, "float32", "portions")


@pytest.mark.gpu
def test_generate_command_with_random_weights():
    if not torch.cuda.is_available():
        pytest.skip("no GPU here")
    out = json.loads(_command("generate", "--random-weights", "4", "--shape", "zigelorn-tiny", "--prompt-ids", "5 17 3",
                              "--prompt-ids", "9 8 7 6 5 4 3 2 1", "--output-tokens", "6", "--temperature", "0", "--ignore-eos",
                              "--block-size", "8", "--num-blocks", "32", "--max-model-len", "64", "--quiet"))
    assert [len(o["token_ids"]) for o in out] == [6, 6]


# ------------------------------------------------------------------ the replay program
@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_replay_program_on_a_model_of_this_design(folders, dtype, tmp_path):
    """``bin/trace_run`` as a user starts it: steps on standard input, ``<step>.f32`` files, pages of 64 and four
    state slots that several traces in one run use again, steps of single tokens and short mixed steps from graphs."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU here")
    from test_replay import _logits_from_files, _renamed, _trace_run
    requests = _requests("S", [150, 9, 71, 2, 40])
    want = _plain_logits(folders["S"], requests)
    ways = {"portions": zc.in_portions(requests, [37, 2, 64, 5, 1, 1]),
            "side by side": zc.interleaved(requests, [33, 1, 1, 16, 1, 7, 1], 4)}
    steps, first = [], 0
    for k, (what, t) in enumerate(ways.items()):
        steps += _renamed(t, f"#{k}", first)
        first += len(t)
    out_dir = str(tmp_path / "out")
    _trace_run(folders["S"], dtype, steps, out_dir, max(zc.peak_tokens(t, 64) for t in ways.values()))
    got = _logits_from_files(out_dir, steps, zc.CONFIG_S["vocab"])
    for k, what in enumerate(ways):
        _compare({rid: got[f"{rid}#{k}"] for rid in want}, want, dtype, what)
