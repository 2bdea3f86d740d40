"""The Gabelorn design in the engine against its plain whole-sequence implementation (``plain_gabelorn.py``): every
mechanism alone through the kernels' entry points, then whole models through the step function (whole prompts, decoding
token by token, portions down to two tokens, unequal requests side by side on few pages and slots that are used again),
and greedy generation through the entry point and its scheduler. Every test runs on the CPU stand-in for the kernels (the
engine's logic) and, marked ``gpu``, on the HIP kernels in both element types.
"""
import json
import os

import pytest
import torch

import gabelorn_cases as gc
import plain_gabelorn as plain
from helpers import first_difference, max_abs_diff, tolerance_for
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
    old = ops._backend
    if device == "cpu":
        from emulated_kernels import EmulatedBackend
        ops.set_backend(EmulatedBackend())
    else:
        if not torch.cuda.is_available():
            pytest.skip("no GPU here")
        ops.set_backend(None)
    yield
    ops.set_backend(old)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: gc.write_model(str(tmp_path_factory.mktemp(f"gabelorn_{name}")), cfg, seed)
            for name, (cfg, seed) in gc.CASES.items()}


def _dt(name):
    return {"float32": torch.float32, "bfloat16": torch.bfloat16}[name]


def _tol(dtype, plain_values, fine=2e-5, coarse=4e-2):
    """Largest allowed difference, as a share of the spread of the plain values."""
    return (fine if dtype == "float32" else coarse) * float(plain_values.float().std())


def _near(got, want, dtype, what):
    """Within the tolerance; in bfloat16, where queries, values, weights and the result are each rounded to eight bits, an
    entry may also be off by a part in 2^7 of itself."""
    bound = _tol(dtype, want) + (2.0 ** -7 * want.abs() if dtype == "bfloat16" else 0.0)
    bad = ((got - want).abs() > bound).nonzero()
    assert bad.numel() == 0, (what, f"{bad.shape[0]} of {want.numel()} entries, first at {bad[0].tolist()}, largest difference "
                              f"{max_abs_diff(got, want):.3e} with a spread of {float(want.std()):.3e}")


def _rounded(t, dtype):
    return t.bfloat16().float() if dtype == "bfloat16" else t


# ------------------------------------------------------------------ mechanisms alone
def _single_request_batch(T, start, device, page_size, pages):
    pos = torch.arange(start, start + T, dtype=torch.int32)
    slots = torch.tensor([pages[p // page_size] * page_size + p % page_size for p in pos.tolist()], dtype=torch.int32)
    batch = AttentionBatch(num_tokens=T, num_requests=1, token_req=torch.zeros(T, dtype=torch.int32).to(device),
                           positions=pos.to(device), cu_seqlens_q=torch.tensor([0, T], dtype=torch.int32).to(device),
                           context_lens=torch.tensor([start + T], dtype=torch.int32).to(device), max_q_len=T,
                           max_context_len=start + T)
    return batch, slots.to(device), torch.tensor([pages], dtype=torch.int32).to(device)


def _pages(T, page_size):
    """(pages of a request of T tokens in a scrambled order, number of pages there are)"""
    n = -(-T // page_size)
    return torch.randperm(n + 2, generator=torch.Generator().manual_seed(T)).tolist()[:n], n + 2


def _biased_through_kernels(where, m, rows, sinks, portions, page_size, first=None, lam=None):
    """``rows`` [T, columns]: the packed projection of one request as the layer's product leaves it (q | k | v). Scaled,
    mixed, stored and read back by the kernels in the given portions, on pages with stale contents (NaN). ``first`` =
    (rows of another layer, column of its values)."""
    device, dtype = where
    T, H, G, D, E = rows.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pages, total = _pages(T, page_size)
    k_cache = torch.full((total, page_size, G, D), float("nan"), dtype=_dt(dtype)).to(device)
    v_cache = torch.full((total, page_size, G, E), float("nan"), dtype=_dt(dtype)).to(device)
    packed = rows.to(_dt(dtype)).to(device)
    other = None if first is None else first[0].to(_dt(dtype)).to(device)
    temperature = (m["q_temp"]["coef"], m["q_temp"]["every"]) if m.get("q_temp") else None
    slopes = plain.slopes(H).float().to(device)
    outs, at = [], 0
    for n in portions:
        batch, slots, table = _single_request_batch(n, at, device, page_size, pages)
        mix = None if first is None else ((other[at:at + n].contiguous(), first[1]), torch.tensor(lam).to(device))
        q = ops.rotary_split_write(packed[at:at + n].contiguous(), None, None, None, batch.positions, slots, k_cache, v_cache,
                                   H, G, D, E, temperature=temperature, mix=mix)
        outs.append(ops.paged_attention(q, k_cache, v_cache, batch, table, m["scale"], sink=sinks.to(device), slopes=slopes).float().cpu())
        at += n
    assert at == T
    return torch.cat(outs)


def _biased_plain(m, rows, sinks, first=None, lam=None):
    T, H, G, D, E = rows.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    x = rows.double()
    q = x[:, :H * D].view(T, H, D)
    if m.get("q_temp"):
        q = q * plain.query_temperature(torch.arange(T), m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    v = x[:, (H + G) * D:].reshape(T, G, E)
    if first is not None:
        v = plain.mixed_values(v, first[0].double()[:, first[1]:first[1] + G * E].reshape(T, G, E), lam)
    return plain.read_heads(q, x[:, H * D:(H + G) * D].view(T, G, D), v, m["scale"], sinks.double(), plain.window_mask(T, None),
                            plain.distance_bias(T, H)).float()


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sizes", [(12, 20, 2, 3), (32, 32, 2, 2), (16, 16, 1, 17), (64, 64, 1, 8), (1, 1, 1, 1), (128, 128, 1, 5), (48, 16, 3, 1)],
                         ids=lambda s: "D%d-E%d-kv%d-group%d" % s)
def test_attention_with_a_bias_by_distance(where, kernels, sizes):
    """Random queries, keys and values under slopes of any number of heads, a sink per head, queries scaled by their
    position and values mixed with another layer's: head sizes that the matrix-core kernels take and sizes that they do
    not, more than 16 query heads on a key/value head; portions that end inside pages."""
    device, dtype = where
    D, E, G, group = sizes
    H = G * group
    g = torch.Generator().manual_seed(5)
    T = 60 if device == "cpu" else 150
    m = gc.biased(H, G, D, E, 1.2 * D ** -0.5, 0.4, 9, True)["mixer"]
    rows = _rounded(torch.randn(T, (H + G) * D + G * E, generator=g), dtype)
    first = _rounded(torch.randn(T, G * E + 5, generator=g), dtype)
    sinks = 1.0 + torch.randn(H, generator=g)
    for other, lam in (((first, 3), 0.35), (None, None)):
        want = _biased_plain(m, rows, sinks, other, lam)
        for portions in ([T], [1] * T, [2, 5, 3, 11, 1, 2, 21, T - 45]):
            got = _biased_through_kernels(where, m, rows, sinks, portions, 8, other, lam)
            _near(got, want, dtype, portions[:3])


@pytest.mark.parametrize("where", WHERE)
def test_single_terms_of_the_biased_softmax(where, kernels):
    """Inputs made so that one term of the softmax shows: a far key whose score beats bias and sinks, the sink of one head
    alone (the others' at minus a hundred), queries that only their temperature lifts over the sink, slopes of numbers of
    heads that are no power of two. Queries and keys are known vectors, so each weight is known too."""
    device, dtype = where
    T, D, page = 300, 16, 16

    def rows_of(H, q, k, v):
        x = torch.zeros(T, (H + 1) * D + D)
        x[:, :H * D].view(T, H, D)[..., 0] = q
        x[:, H * D] = k
        x[:, (H + 1) * D:] = v
        return x
    ways = ([T], [T - 40] + [1] * 40)
    # a far key: its score is 40, every other 0; slopes of 3 heads; whoever sees it returns its value but for the bias
    for marked in (0, 15, 16, 63, 64, 100, 255):
        k, v = torch.zeros(T), torch.zeros(T, D)
        k[marked], v[marked] = 10.0, 1.0
        m = gc.biased(3, 1, D, D, 1.0, 0.0, 1, False)["mixer"]
        rows = rows_of(3, 4.0, k, v)
        sinks = torch.tensor([1.0, 30.0, -3.0])
        want = _biased_plain(m, rows, sinks)
        far = 8.0 if marked < 200 else 1.0
        assert float(want[:marked].abs().max()) == 0 if marked else True
        assert float(want[marked + 1, 2, 0]) > 0.9 and float(want[-1, 2, 0]) > 1e-3 / far
        for portions in ways:
            got = _biased_through_kernels(where, m, rows, sinks, portions, page)
            assert max_abs_diff(got, want) <= (1e-5 if dtype == "float32" else 1e-2), (marked, len(portions))
    # sinks alone: scores 0, values 1, no distance (every query at its own key): one head's sink takes 1 / (1 + e) there
    m = gc.biased(5, 1, D, D, 1.0, 0.0, 1, False)["mixer"]
    for h in range(5):
        sinks = torch.full((5,), -100.0)
        sinks[h] = 1.0
        got = _biased_through_kernels(where, m, rows_of(5, 0.0, torch.zeros(T), torch.ones(T, D)), sinks, [T], page)
        share = 1.0 / (1.0 + 2.718281828)
        assert abs(float(got[0, h, 0]) - share) < 4e-3 and all(abs(float(got[0, o, 0]) - 1.0) < 4e-3 for o in range(5) if o != h)
    # the temperature: score 2 (1 + 5 ln n) against a sink of 12, n steps up every 7 positions (p + 1 counts)
    m = gc.biased(1, 1, D, D, 1.0, 5.0, 7, False)["mixer"]
    k = torch.full((T,), -50.0)
    k[0] = 2.0
    v = torch.zeros(T, D)
    v[0] = 1.0
    rows = rows_of(1, 1.0, k, v)
    want = _biased_plain(m, rows, torch.tensor([12.0]))
    assert float(want[5, 0, 0]) < 1e-3 and float(want[6, 0, 0]) < 0.1 < float(want[20, 0, 0])
    for portions in ways:
        got = _biased_through_kernels(where, m, rows, torch.tensor([12.0]), portions, page)
        assert max_abs_diff(got, want) <= (2e-5 if dtype == "float32" else 2e-2), len(portions)


def _latent_through_kernels(where, m, eps, rows, w, portions, page_size):
    """``rows``: the packed projection q | latent and rotated key part | gates of one request. The layer's steps as the
    part takes them, in the given portions; the result is what goes into the output projection."""
    device, dtype = where
    dt = _dt(dtype)
    T, H, D, R, E, C = rows.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    row = -(-(C + R) // 16) * 16
    pages, total = _pages(T, page_size)
    cache = torch.full((total, page_size, 1, row), float("nan"), dtype=dt).to(device)
    packed = rows.to(dt).to(device)
    freqs = (m["rot"]["base"] ** (-2.0 * torch.arange(R // 2, dtype=torch.float64) / R)).to(device) if R else None
    uk_t = w["uk"].view(H, D, C).transpose(1, 2).contiguous().view(H * C, D).to(dt).to(device)
    uv, wc, sinks = w["uv"].to(dt).to(device), w["dkv.norm"].float().to(device), w["sink"].float().to(device)
    outs, at = [], 0
    for n in portions:
        batch, slots, table = _single_request_batch(n, at, device, page_size, pages)
        a = packed[at:at + n].contiguous()
        nq = H * (D + R)
        assert ops.latent_prepare(a, 0, 0, nq, C, R, None, wc, eps, freqs, 1.0, batch.positions, slots, cache, dt, halves=True) is None
        q_row = torch.zeros((n, H, row), dtype=dt, device=device)
        ops.head_gemm(a[:, :nq].unflatten(1, (H, D + R)), uk_t, False, C, D, out=q_row,
                      turn=(R, D, C, freqs, 1.0, batch.positions, True) if R else None)
        mixed = ops.paged_attention(q_row, cache, cache, batch, table, m["scale"], m["mask"]["size"], sink=sinks)
        o = ops.head_gemm(mixed, uv, False, E, C, gate=(a, nq + C + R, "per entry"))
        outs.append(o.reshape(n, H * E).float().cpu())
        at += n
    assert at == T
    return torch.cat(outs)


def _latent_plain(m, eps, rows, w):
    """The plain mixer with rows of the identity as its projections of the packed rows."""
    H, D, R, E, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    eye, nq = torch.eye(rows.shape[1], dtype=torch.float64), H * (D + R)
    full = {k: v.double() for k, v in w.items()}
    full.update(q=eye[:nq], dkv=eye[nq:nq + C + R], g=eye[nq + C + R:], o=torch.eye(H * E, dtype=torch.float64))
    return plain.latent_attention(rows.double(), full, m, eps).float()


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sizes", [(3, 8, 4, 6, 10), (20, 16, 16, 16, 48), (1, 1, 2, 1, 1), (4, 32, 16, 24, 100), (2, 64, 32, 64, 160), (2, 5, 6, 7, 9), (2, 8, 16, 8, 300)],
                         ids=lambda s: "H%d-D%d-R%d-E%d-C%d" % s)
@pytest.mark.parametrize("window", [1, 7, 40, 1000])
def test_latent_attention_alone(where, kernels, sizes, window):
    """Random packed rows: the latent's norm, the halves-paired rotation of queries and of the shared key part, the window,
    sinks and a gate per entry; more than 16 heads on a row, rows that are filled up to a multiple of 16 and rows that are
    one; portions that end inside pages and windows."""
    device, dtype = where
    H, D, R, E, C = sizes
    m = gc.latent(H, D, R, E, C, window, 50.0, 1.2 * (D + R) ** -0.5)["mixer"]
    g = torch.Generator().manual_seed(window)
    T, eps = (50 if device == "cpu" else 130), 1e-2
    rows = _rounded(torch.randn(T, H * (D + R) + C + R + H * E, generator=g), dtype)
    rows[:, H * (D + R):H * (D + R) + C] *= _rounded(0.05 + torch.rand(T, 1, generator=g), dtype)      # (small: the eps matters)
    rows = _rounded(rows, dtype)
    w = {"uk": (torch.randn(H * D, C, generator=g) * C ** -0.5).bfloat16(), "uv": (torch.randn(H * E, C, generator=g) * C ** -0.5).bfloat16(),
         "dkv.norm": (1 + 0.2 * torch.randn(C, generator=g)).bfloat16(), "sink": torch.randn(H, generator=g).bfloat16()}
    want = _latent_plain(m, eps, rows, w)
    for portions in ([T], [1] * T, [2, 5, 3, 11, 1, 2, 21, T - 45]):
        got = _latent_through_kernels(where, m, eps, rows, w, portions, 8)
        _near(got, want, dtype, portions[:3])


@pytest.mark.parametrize("where", WHERE)
def test_one_latent_that_stands_out_at_a_windows_edge(where, kernels):
    """Among 200 latents one carries nearly all the weight of every query that sees it, and a value no other has: a query
    returns that value exactly when the marked position is among its last ``window`` ones, itself included. Marked at a
    page's and a tile's borders, in a prompt and decoded one by one."""
    device, dtype = where
    T, C, D, window, page = 200, 16, 8, 48, 16
    m = gc.latent(2, D, 2, C, C, window, 10.0, 1.0)["mixer"]
    w = {"uk": torch.zeros(2 * D, C), "uv": torch.eye(C).repeat(2, 1), "dkv.norm": torch.ones(C), "sink": torch.tensor([3.0, -2.0])}
    w["uk"][0, 1] = w["uk"][D, 1] = 10.0                             # unrotated key entry 0 is ten times latent entry 1
    for marked in (0, 1, 15, 16, 47, 48, 63, 64, 100, 151):
        rows = torch.zeros(T, 2 * (D + 2) + C + 2 + 2 * C)
        rows[:, 0] = rows[:, D + 2] = 1.0                            # queries ask for entry 0
        rows[:, 2 * (D + 2)] = 1.0                                   # every latent lies along entry 0 ...
        rows[marked, 2 * (D + 2)], rows[marked, 2 * (D + 2) + 1] = 0.0, 1.0      # ... but the marked one, along entry 1
        rows[:, 2 * (D + 2) + C + 2:] = 20.0                         # the gates are open
        sees = torch.tensor([marked <= i < marked + window for i in range(T)])
        for portions in ([T], [marked + 1] + [1] * (T - marked - 1) if marked < 120 else [T - 60] + [1] * 60, [30, 2, 50, 1, 1, 116]):
            got = _latent_through_kernels(where, m, 1e-6, rows, w, portions, page).view(T, 2, C)
            for h in range(2):
                assert torch.equal(got[:, h, 1] > 3.9, sees), (marked, h, len(portions))
                assert torch.equal(got[:, h, 1] < 0.1, ~sees), (marked, h, len(portions))


@pytest.mark.parametrize("where", WHERE)
def test_rotation_far_from_the_start(where, kernels):
    """Rotated rows and queries at positions up to a million, both ways of pairing, against angles in float64."""
    device, dtype = where
    dt = _dt(dtype)
    positions = torch.tensor([0, 1, 255, 4096, 99_999, 1_000_003], dtype=torch.int32)
    g = torch.Generator().manual_seed(3)
    R, H, T = 12, 3, len(positions)
    x = torch.randn(T, H, R + 4, generator=g).to(dt)
    freqs = 10000.0 ** (-2.0 * torch.arange(R // 2, dtype=torch.float64) / R)
    for halves in (True, False):
        t = x.double()[..., 4:]
        want = plain.turn_halves(t if halves else torch.cat((t[..., 0::2], t[..., 1::2]), dim=-1), R, 10000.0, positions.double())
        if not halves:
            want = torch.stack((want[..., :R // 2], want[..., R // 2:]), dim=-1).flatten(-2)
        out = torch.zeros(T, H, R + 2, dtype=dt).to(device)
        got = ops.rotate_heads(x.to(device), 4, out, 1, R, freqs.to(device), 1.0, positions.to(device), halves=halves)[:, :, 1:R + 1]
        assert max_abs_diff(got.cpu(), want) <= (2e-6 if dtype == "float32" else 2e-2), halves
        assert float(out[:, :, 0].abs().max()) == 0 and float(out[:, :, R + 1:].abs().max()) == 0


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sizes", [(3, 10, 7), (2, 16, 8), (20, 48, 16), (1, 33, 40), (5, 128, 192), (2, 130, 24)], ids=lambda s: "H%d-N%d-K%d" % s)
def test_a_matrix_per_head(where, kernels, sizes):
    """Products with one matrix per head, of few rows and of many, stored either way, from dense rows and from a view of
    packed ones, into a part of wider rows, with no gate, a gate per head or per entry, and with a rotated part beside."""
    device, dtype = where
    dt = _dt(dtype)
    H, N, K = sizes
    R, pad = 4, 3
    g = torch.Generator().manual_seed(N)
    w = torch.randn(H, N, K, generator=g).to(dt) * K ** -0.5
    freqs = (30.0 ** (-2.0 * torch.arange(R // 2, dtype=torch.float64) / R)).to(device)
    for rows in (1, 5, 16, 17, 70) + ((150, 333) if device != "cpu" else ()):
        packed = torch.randn(rows, 8 + H * (K + R) + 8, generator=g).to(dt).to(device)
        view = packed[:, 8:8 + H * (K + R)].unflatten(1, (H, K + R))
        x = view.cpu().double()
        pure = torch.einsum("thk,hnk->thn", x[..., :K], w.double())
        pos = (torch.arange(rows, dtype=torch.int32) * 3).to(device)
        per_head = torch.randn(rows, H + 2, generator=g).to(device)
        per_entry = torch.randn(rows, H * N + 5, generator=g).to(dt).to(device)
        for form, stored in ((False, w.reshape(H * N, K)), (True, w.transpose(1, 2).reshape(H * K, N))):
            stored = stored.contiguous().to(device)
            for x_in in (view, view.contiguous()):
                out = torch.full((rows, H, N + R + pad), 7.0, dtype=dt).to(device)
                ops.head_gemm(x_in, stored, form, N, K, out=out, out_off=1, turn=(R, K, N + 2, freqs, 1.0, pos, True))
                turned = plain.turn_halves(x[..., K:], R, 30.0, pos.cpu().double())
                assert max_abs_diff(out[:, :, 1:N + 1].cpu(), pure) <= _tol(dtype, pure, fine=1e-5, coarse=2e-2), (rows, form)
                assert max_abs_diff(out[:, :, N + 2:N + 2 + R].cpu(), turned) <= _tol(dtype, turned, fine=1e-5, coarse=3e-2), (rows, form)
                assert bool((out[:, :, 0] == 7.0).all()) and bool((out[:, :, N + 1] == 7.0).all()) and bool((out[:, :, N + R + 2:] == 7.0).all())
            got = ops.head_gemm(view, stored, form, N, K, gate=(per_head, 1))
            want = pure * torch.sigmoid(per_head.cpu().double()[:, 1:H + 1])[:, :, None]
            assert max_abs_diff(got.cpu(), want) <= _tol(dtype, pure, fine=1e-5, coarse=2e-2), (rows, form, "gate per head")
            got = ops.head_gemm(view, stored, form, N, K, gate=(per_entry, 5, "per entry"))
            want = pure * torch.sigmoid(per_entry.cpu().double()[:, 5:]).view(rows, H, N)
            assert max_abs_diff(got.cpu(), want) <= _tol(dtype, pure, fine=1e-5, coarse=2e-2), (rows, form, "gate per entry")
            alone = ops.head_gemm(view[-1:], stored, form, N, K, gate=(per_entry[-1:].contiguous(), 5, "per entry"))
            assert max_abs_diff(alone.cpu(), got[-1:].cpu()) <= _tol(dtype, pure, fine=4e-6, coarse=1e-2)
    with pytest.raises(ops.KernelError):
        ops.head_gemm(view, stored, True, N, K, gate=(per_entry, 6, "per entry"))


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("sizes", [(24, 40), (7, 10), (16, 64), (130, 256)], ids=lambda s: "ff%d-width%d" % s)
def test_clamped_feed_forward(where, kernels, sizes):
    """The gated feed-forward with clamps and biases as a part, few rows and many, with inputs wide enough that each clamp
    binds (the gate from above only): against the plain equations."""
    from nanohybrid_vlm_amd.parts.base import FEED_FORWARDS
    device, dtype = where
    dt = _dt(dtype)
    F, W = sizes
    g = torch.Generator().manual_seed(F)
    w = {"gate": torch.randn(F, W, generator=g) * 3 * W ** -0.5, "up": torch.randn(F, W, generator=g) * 3 * W ** -0.5,
         "down": torch.randn(W, F, generator=g) * F ** -0.5, "gate.b": torch.randn(F, generator=g), "up.b": torch.randn(F, generator=g),
         "down.b": torch.randn(W, generator=g)}
    w = {k: v.bfloat16() for k, v in w.items()}
    part = FEED_FORWARDS.build({"kind": "swiglu", "hidden_size": W, "intermediate_size": F, "activation": "clamped_swish", "bias": True,
                                "limit": 1.25, "alpha": 1.702, "offset": 1.0})
    params = {"gate_up.weight": torch.cat((w["gate"], w["up"])), "gate_up.bias": torch.cat((w["gate.b"], w["up.b"])),
              "down.weight": w["down"], "down.bias": w["down.b"]}
    assert set(params) == set(part.all_param_specs())
    part.bind_all({k: v.to(dt).to(device) for k, v in params.items()})
    for n in (1, 3, 16, 17, 64, 65, 300):
        h = torch.randn(n, W, generator=g).to(dt)
        full = {k: v.double() for k, v in w.items()}
        want = plain.feed_forward(h.double(), full, 1.25).float()
        assert max_abs_diff(part.forward(h.to(device), None).cpu(), want) <= _tol(dtype, want, coarse=3e-2), n
    # the gate alone: values on both sides of every bound, at the bounds, far beyond them
    z = torch.tensor([-300.0, -9.0, -1.25, -1.0, 0.0, 1.0, 1.25, 1.5, 9.0, 300.0])
    gu = torch.cat((z.repeat_interleave(10), z.repeat(10)))[None].to(dt)
    got = ops.act_mul(gu.to(device), ops.Gate(2, 1.25, 1.702, 1.0)).cpu()
    want = plain.clamped_gate(gu[:, :100].double(), gu[:, 100:].double(), 1.25)
    assert max_abs_diff(got, want) <= (1e-6 if dtype == "float32" else 1e-2)
    with pytest.raises(ValueError):
        FEED_FORWARDS.build({"kind": "swiglu", "hidden_size": 8, "intermediate_size": 8, "activation": "clamped_swish"})


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("width", [40, 52, 1024])
def test_norms_and_products_that_take_them_over(where, kernels, width):
    """A norm that is rounded once, and the fused steps of few rows: a product that adds itself (with its bias) to the
    float32 stream, and a gated product with biases that scales its rows itself, against the plain sequence of steps."""
    device, dtype = where
    dt = _dt(dtype)
    g = torch.Generator().manual_seed(width)
    eps, F = 1e-3, 24
    norm_w = (1 + 0.2 * torch.randn(width, generator=g)).to(dt)
    w_o, b_o = (torch.randn(width, F, generator=g) * F ** -0.5).to(dt), torch.randn(width, generator=g).to(dt)
    w_gu, b_gu = (torch.randn(2 * F, width, generator=g) * 2 * width ** -0.5).to(dt), torch.randn(2 * F, generator=g).to(dt)
    gate = ops.Gate(2, 1.5, 1.702, 1.0)
    for rows in (1, 7, 16, 33):
        a, stream = torch.randn(rows, F, generator=g).to(dt), torch.randn(rows, width, generator=g) * 2
        residual = stream.clone().to(device)
        add = ops.AddTo(residual, norm_w.to(device), eps, (w_gu.to(device), True))
        y = ops.linear(a.to(device), w_o.to(device), b_o.to(device), add_to=add)
        if isinstance(y, ops.Summed):
            x = ops.Normed(y)
        else:
            x = ops.rmsnorm(y, norm_w.to(device), eps, residual=residual, rounds_between=False)
        total = stream.double() + a.double() @ w_o.double().T + b_o.double()
        # (where the product does not make the addition itself, its result is rounded to the rows' type before it)
        assert max_abs_diff(residual.cpu(), total) <= (1e-5 if dtype == "float32" or isinstance(y, ops.Summed) else 3e-2)
        h = plain.rms_norm(total, norm_w.double(), eps)
        got = ops.gated_linear(x, w_gu.to(device), gate, b_gu.to(device))
        z = h @ w_gu.double().T + b_gu.double()
        want = plain.clamped_gate(z[:, :F], z[:, F:], 1.5)
        assert max_abs_diff(got.cpu(), want) <= _tol(dtype, want), rows
    x = torch.randn(9, width, generator=g).to(dt)
    once = ops.rmsnorm(x.to(device), norm_w.to(device), eps, rounds_between=False).cpu()
    exact = plain.rms_norm(x.double(), norm_w.double(), eps)
    assert max_abs_diff(once, exact) <= (1e-6 if dtype == "float32" else 0.5 * 2.0 ** -7 * float(exact.abs().max()))
    if dtype == "bfloat16":                                         # once: the nearest bfloat16 number but for float's own rounding
        assert float((once != exact.to(torch.bfloat16)).float().mean()) < 0.01


# ------------------------------------------------------------------ configuration and weights
def test_configuration_and_checkpoint_names():
    from nanohybrid_vlm_amd.parts.base import PagedKVNeed
    from nanohybrid_vlm_amd.parts.model import DecoderModel
    arch = resolve_architecture(gc.CONFIG_A)
    assert arch.name == "Gabelorn"
    cfg = arch.parse_config(gc.CONFIG_A)
    assert cfg.first_mixing() == 1 and cfg.layers[2].mlp is None and cfg.layers[0].mlp.limit == 1.0
    model = DecoderModel(arch.build_spec(cfg), options={"residual_float32": False})
    assert all(layer.mixer_norm.residual_float32 for layer in model.layers)      # (this design's stream is float32 whatever is asked)
    names = arch.checkpoint_names(cfg)
    assert set(names) == set(gc.random_tensors(gc.CONFIG_A, 0))
    assert {s.param for s in names.values()} == set(model.all_param_specs())
    needs = model.cache_needs()
    assert all(isinstance(n, PagedKVNeed) for n in needs)
    assert needs[0].values_in_keys and (needs[0].head_dim, needs[0].window) == (16, 6) and needs[2].window == 9
    assert (needs[1].num_kv_heads, needs[1].head_dim, needs[1].value_size, needs[1].window) == (2, 6, 10, None)
    # a second norm that a checkpoint stores beside a layer without feed-forward is read and not used
    spare = arch.parse_config(gc.CONFIG_A, {"l2.norm2": (40,)})
    assert "l2.norm2" in arch.checkpoint_names(spare) and "layers.2.feed_forward_norm.weight" in DecoderModel(arch.build_spec(spare)).all_param_specs()
    for change, match in ((lambda c: c["layers"][1].update(type="other"), "not known"),
                          (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=2), "rot.dims"),
                          (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
                          (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "multiple"),
                          (lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0), "every"),
                          (lambda c: c["layers"][4]["mixer"].update(vdim=6), "values it mixes in"),
                          (lambda c: c["layers"][0]["mlp"].update(limit=0), "limit"),
                          (lambda c: c["layers"][0]["mlp"].pop("limit"), "limit"),
                          (lambda c: c["layers"][0]["mlp"].update(kind="other"), "dense"),
                          (lambda c: c.update(logit_softcap=-1.0), "logit_softcap")):
        bad = json.loads(json.dumps(gc.CONFIG_A))
        change(bad)
        with pytest.raises(ConfigError, match=match):
            arch.parse_config(bad)


# ------------------------------------------------------------------ whole models through the step function
def _requests(name, lengths):
    vocab = gc.CASES[name][0]["vocab"]
    return {f"r{i}": gc.tokens(vocab, n, 100 * i + n) for i, n in enumerate(lengths)}


def _plain_logits(folder, requests, dtype=torch.float64):
    cfg, w = plain.read_folder(folder)
    return {rid: plain.forward(cfg, w, toks, dtype).float() for rid, toks in requests.items()}


def _replay(folder, where, steps, page_size, max_live, **options):
    device, dtype = where
    pages = max(1, gc.peak_tokens(steps, page_size) // page_size)
    runner = ModelRunner(folder, dtype=dtype, device=device, page_size=page_size, num_pages=pages, num_state_slots=max_live,
                         max_model_len=pages * page_size, poison_freed_pages=True, **options)
    got = replay(runner, steps)
    assert not runner.cache.requests and all(runner.cache.num_free_pages(g) == pages for g in range(len(runner.cache.groups)))
    return got


def _numbered(steps):
    for i, s in enumerate(steps):
        s["step"] = i
    return steps


def _compare(got, want, dtype, what):
    """Every logit within the tolerance of ``helpers`` in float32: 1e-4 of the logits' spread. In bfloat16 the root mean square
    over the vocabulary within a tenth of the spread (it is a hundredth as a rule; one position in fifty, where a softmax is
    close to a tie, may be up to half as much again)."""
    tol = tolerance_for(dtype, want)
    for rid in want:
        if dtype == "float32":
            assert max_abs_diff(got[rid], want[rid]) <= tol, (what, rid, first_difference(got[rid], want[rid], tol))
        else:
            errors = (got[rid].float() - want[rid].float()).pow(2).mean(dim=-1).sqrt()
            over = (errors > tol).nonzero().flatten().tolist()
            assert bool((errors <= 1.5 * tol).all()) and len(over) <= max(1, len(errors) // 50), (what, rid, over[:4], float(errors.max()) / tol)


@pytest.mark.parametrize("where", WHERE)
def test_layers_one_by_one(folders, where, kernels):
    """Models cut off after 1, 2, ... layers give the plain model's logits: the stream after every layer is right."""
    cfg, w = plain.read_folder(folders["A"])
    toks = gc.tokens(cfg["vocab"], 21, 9)
    for n in range(1, len(cfg["layers"]) + 1):
        cut = dict(cfg, layers=cfg["layers"][:n])
        keep = tuple(f"l{i}." for i in range(n))
        tensors = {k: v for k, v in w.items() if not k.startswith("l") or k.startswith(keep)}
        folder = gc.write_model(os.path.join(folders["A"], f"cut{n}"), cut, 0, tensors)
        want = _plain_logits(folder, {"a": toks})
        got = _replay(folder, where, gc.in_portions({"a": toks}, [8, 1, 5, 7]), page_size=4, max_live=1)
        _compare(got, want, where[1], f"{n} layers")


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", ["A", "B", "C", "R"])
def test_ways_of_cutting_agree_with_the_plain_model(folders, where, kernels, name):
    """Whole prompts, a prompt followed by its last tokens one by one, portions of several sizes down to two tokens
    (and single tokens between them), and unequal requests side by side on pages and slots that are used again: all
    give the plain model's logits at every position. In float32 on the GPU the ways agree bit for bit."""
    device, dtype = where
    lengths = [1, 2, 26, 19, 37, 5] if device == "cpu" else [1, 2, 26, 19, 61, 5, 150, 43]
    requests = _requests(name, lengths)
    want = _plain_logits(folders[name], requests)
    ways = {
        "whole": (gc.whole(requests), 3),
        "tail": ([s for rid, toks in requests.items()
                  for s in gc.in_portions({rid: toks}, [max(1, len(toks) - 12)] + [1] * 12)], 3),
        "portions": (gc.in_portions(requests, [2, 3, 5, 2, 1, 7, 4, 2, 11]), 3),
        "side by side": (gc.interleaved(requests, [3, 1, 2, 6, 1, 1, 4], 3), 3),
    }
    results = {}
    for what, (steps, live) in ways.items():
        results[what] = _replay(folders[name], where, _numbered(steps), page_size=4, max_live=live)
        _compare(results[what], want, dtype, what)
    if device != "cpu" and dtype == "float32":
        for what in ("tail", "portions", "side by side"):
            for rid in want:
                assert torch.equal(results[what][rid], results["whole"][rid]), (what, rid)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(where, kernels, seed, tmp_path):
    """Models of sizes drawn at random (see ``gabelorn_cases.random_config``) in portions, side by side and with a decoded
    tail, on pages of 16 tokens that are used again, against the plain model; float32 bit-equal across the ways on the GPU."""
    device, dtype = where
    if device == "cpu" and seed >= 5:
        pytest.skip("the stand-in takes the first five")
    cfg = gc.random_config(seed)
    folder = gc.write_model(str(tmp_path / "m"), cfg, 500 + seed)
    lengths = [1, 21, 33, 7] if device == "cpu" else [1, 70, 210, 33, 131]
    requests = {f"r{i}": gc.tokens(cfg["vocab"], n, 7 * i + n) for i, n in enumerate(lengths)}
    want = _plain_logits(folder, requests)
    ways = {"portions": gc.in_portions(requests, [17, 2, 3, 64, 1, 33]),
            "side by side": gc.interleaved(requests, [5, 1, 2, 31, 1, 1, 16], 3),
            "tail": [s for rid, toks in requests.items() for s in gc.in_portions({rid: toks}, [max(1, len(toks) - 20)] + [1] * 20)]}
    results = {}
    for what, steps in ways.items():
        results[what] = _replay(folder, where, _numbered(steps), page_size=16, max_live=3)
        _compare(results[what], want, dtype, (seed, what))
    if device != "cpu" and dtype == "float32":
        for rid in want:
            assert torch.equal(results["portions"][rid], results["side by side"][rid]) and \
                torch.equal(results["portions"][rid], results["tail"][rid]), (seed, rid)


@pytest.mark.parametrize("where", ON_GPU)
def test_pages_of_64_and_windows_longer_than_a_page(folders, where, kernels):
    """Pages of 64 tokens (whole tiles of the prompt kernel lie in one page) under windows of 65, 128 and 150 positions,
    requests of up to 400 tokens in portions that end anywhere, beside decoded tokens, on few pages."""
    device, dtype = where
    requests = _requests("S", [400, 130, 70, 257])
    want = _plain_logits(folders["S"], requests)
    for what, steps in (("portions", gc.in_portions(requests, [37, 2, 64, 5, 1, 129, 1, 1, 96])),
                        ("side by side", gc.interleaved(requests, [33, 1, 1, 64, 1, 7, 1, 100], 3))):
        got = _replay(folders["S"], where, steps, page_size=64, max_live=3)
        _compare(got, want, dtype, what)


@pytest.mark.parametrize("where", ON_GPU)
def test_sizes_of_a_real_models_layers(where, kernels, tmp_path):
    """Heads of 128 and 64 entries, rows of 256 under 20 heads, a width of 1,024: the kernels' makes that real sizes take, in
    portions (also of several hundred tokens) and side by side on pages of 64, with decoded tokens between."""
    device, dtype = where
    folder = gc.write_model(str(tmp_path / "w"), gc.CONFIG_W, 26)
    requests = {f"r{i}": gc.tokens(gc.CONFIG_W["vocab"], n, 11 * i + n) for i, n in enumerate([700, 40, 129])}
    want = _plain_logits(folder, requests, torch.float32)
    for what, steps in (("portions", gc.in_portions(requests, [530, 1, 1, 16, 3, 64, 1, 1, 1])),
                        ("side by side", gc.interleaved(requests, [40, 1, 1, 1, 17, 1, 300, 1], 3))):
        got = _replay(folder, where, steps, page_size=64, max_live=3)
        _compare(got, want, dtype, what)


@pytest.mark.parametrize("where", WHERE)
def test_long_decoding(folders, where, kernels):
    """Two tokens of prompt, then many tokens one by one: the windows pass many times, the queries' temperature steps up
    and pages go back to the pool on the way."""
    device, dtype = where
    n = 60 if device == "cpu" else 300
    for name in ("A", "C"):
        requests = _requests(name, [n])
        want = _plain_logits(folders[name], requests)
        got = _replay(folders[name], where, gc.in_portions(requests, [2] + [1] * n), page_size=4, max_live=1)
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
        steps = gc.interleaved(requests, [3, 1, 1, 1, 2, 1, 1], 3)
        for s in steps:                                      # a recorded short step gives one place a request
            for e in s["entries"]:
                e["want"] = e["want"][-1:]
        where = ("cuda:0", dtype)
        eager = _replay(folders["R"], where, steps, page_size=8, max_live=3, use_graphs=False)
        recorded = _replay(folders["R"], where, steps, page_size=8, max_live=3, use_graphs=True)
        for rid in eager:
            if dtype == "float32":
                assert torch.equal(eager[rid], recorded[rid]), rid
            else:
                assert max_abs_diff(eager[rid], recorded[rid]) <= 0.05 * float(eager[rid].std()), rid
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
    cfg, w = plain.read_folder(folders["A"])
    prompts = [gc.tokens(cfg["vocab"], n, 300 + n) for n in (1, 13, 22)]
    llm = LLM(folders["A"], device=device, dtype=dtype, **options)
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=9, ignore_eos=True), use_tqdm=False)
    for prompt, out in zip(prompts, outs):
        assert out["token_ids"] == plain.greedy_generate(cfg, w, prompt, 9)
    stats = llm.get_memory_stats()
    assert stats["live_requests"] == 0 and all(g["free_pages"] == g["pages"] for g in stats["groups"])


# ------------------------------------------------------------------ the command line
def _command(*args):
    import subprocess
    import sys
    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, "-m", "nanohybrid_vlm_amd", *args], cwd=repo, capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-3000:]
    return proc.stdout


def test_random_model_of_a_named_shape(tmp_path, emulated_kernels):
    """``random-model --shape gabelorn-tiny`` writes a folder that the plain implementation and the engine both read."""
    out = str(tmp_path / "m")
    _command("random-model", "--out", out, "--shape", "gabelorn-tiny", "--seed", "5")
    cfg, w = plain.read_folder(out)
    assert cfg["architecture"] == "Gabelorn" and w["l0.mix.sink"].shape == (cfg["layers"][0]["mixer"]["heads"],)
    requests = {"a": gc.tokens(cfg["vocab"], 31, 1)}
    want = _plain_logits(out, requests)
    got = _replay(out, CPU, gc.in_portions(requests, [4, 1, 9]), page_size=8, max_live=1)
    _compare(got, want, "float32", "portions")


@pytest.mark.gpu
def test_generate_command_with_random_weights():
    if not torch.cuda.is_available():
        pytest.skip("no GPU here")
    out = json.loads(_command("generate", "--random-weights", "4", "--shape", "gabelorn-tiny", "--prompt-ids", "5 17 3",
                              "--prompt-ids", "9 8 7 6 5 4 3 2 1", "--output-tokens", "6", "--temperature", "0", "--ignore-eos",
                              "--block-size", "8", "--num-blocks", "32", "--max-model-len", "64", "--quiet"))
    assert [len(o["token_ids"]) for o in out] == [6, 6]


# ------------------------------------------------------------------ the replay program
@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_replay_program_on_a_model_of_this_design(folders, dtype, tmp_path):
    """``bin/trace_run`` as a user starts it: steps on standard input, ``<step>.f32`` files, pages of 64 and four
    slots that several traces in one run use again, steps of single tokens and short mixed steps from graphs."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU here")
    from test_replay import _logits_from_files, _renamed, _trace_run
    requests = _requests("S", [150, 9, 71, 2, 40])
    want = _plain_logits(folders["S"], requests)
    ways = {"portions": gc.in_portions(requests, [37, 2, 64, 5, 1, 1]),
            "side by side": gc.interleaved(requests, [33, 1, 1, 16, 1, 7, 1], 4)}
    steps, first = [], 0
    for k, (what, t) in enumerate(ways.items()):
        steps += _renamed(t, f"#{k}", first)
        first += len(t)
    out_dir = str(tmp_path / "out")
    _trace_run(folders["S"], dtype, steps, out_dir, max(gc.peak_tokens(t, 64) for t in ways.values()))
    got = _logits_from_files(out_dir, steps, gc.CONFIG_S["vocab"])
    for k, what in enumerate(ways):
        _compare({rid: got[f"{rid}#{k}"] for rid in want}, want, dtype, what)
