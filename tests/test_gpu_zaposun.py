"""The Zaposun decoder on the GPU against the plain implementation in ``plain_zaposun.py``: each mechanism alone,
whole prompts, decoding, portions, mixed batches, pages and slots used again, peaked attention at the edges of chunks,
the first tokens of a sequence, sizes that are 1, equal or odd, and greedy generation through ``LLM``."""

import copy
from types import SimpleNamespace

import pytest
import torch

import plain_zaposun as plain
import zaposun_util as zu
from replay_util import mixed_trace, portion_trace, random_tokens, round64, run_steps, tail_trace, whole_trace

pytestmark = pytest.mark.gpu

F64 = torch.float64
LENGTHS = {"a": 83, "b": 40, "c": 7, "d": 1, "e": 150, "f": 29, "g": 2}
CONFIGS = {"mixed": (zu.MIXED, 41, zu.RANKS), "sharp": (zu.SHARP, 42, zu.RANKS), "ones": (zu.ONES, 43, {1: 1}),
           "odd": (zu.ODD, 44, {1: 5}), "no_pages": (zu.NO_PAGES, 45, None)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: zu.write_model(str(tmp_path_factory.mktemp(name)), cfg, seed, ranks=ranks)
            for name, (cfg, seed, ranks) in CONFIGS.items()}


def _oracle(folder, tokens, store=None, cfg_edit=None, tensors_edit=None):
    cfg, tensors = plain.zaposun_read(folder, F64)
    if cfg_edit is not None:
        cfg_edit(cfg)
    if tensors_edit is not None:
        tensors_edit(tensors)
    return plain.zaposun_forward(cfg, tensors, tokens, store or plain._keep).to(torch.float32)


def _rel_rows(got, want):
    """Per row: RMS of the difference (mean taken off) over the RMS of the wanted row."""
    d = (got - want).double()
    d = d - d.mean(dim=1, keepdim=True)
    return d.pow(2).mean(dim=1).sqrt() / want.double().pow(2).mean(dim=1).sqrt()


def _rel(got, want):
    return _rel_rows(got, want).max().item()


def _like_rounding(errors, rounding, slack=1e-3):
    """``errors``: per-row distances of the engine's logits from exact arithmetic; ``rounding``: the same for the
    plain model with its stored activations rounded."""
    return (errors.median() < 2 * rounding.median() + slack
            and errors.quantile(0.9) < 3 * rounding.quantile(0.9) + slack)


def _replayer(folder, dtype, max_tokens, max_live=4):
    from qwen25vl_lite_amd.engine.replay import Replayer
    return Replayer(folder, dtype, max_tokens, 16, max_live)


def _rows(got, rid, n):
    return torch.stack([got[(rid, p)] for p in range(n)])


def _requests(vocab, seed=0):
    return {rid: random_tokens(n, vocab, seed + i) for i, (rid, n) in enumerate(LENGTHS.items())}


def _i32(values):
    return torch.tensor(list(values), dtype=torch.int32).cuda()


def _run_arrays(runs):
    """``(cu_q, req_slots, token_req)`` on the device for runs of ``(slot, tokens)``."""
    cu = [0]
    for _, n in runs:
        cu.append(cu[-1] + n)
    return _i32(cu), _i32(s for s, _ in runs), _i32(i for i, (_, n) in enumerate(runs) for _ in range(n))


# portions of three sequences over two slots; "r" takes q's slot once q has ended
PORTIONS = [[("p", 1), ("q", 4)], [("q", 1), ("p", 2)], [("p", 1)], [("p", 5), ("q", 1)], [("q", 5), ("p", 1)], [("p", 1)],
            [("p", 9)], [("r", 9), ("p", 3)], [("p", 17)]]
SLOT = {"p": 0, "q": 1, "r": 1}
TOTAL = {"p": 40, "q": 11, "r": 9}


def _over_portions(states, call, rows):
    """Run ``call(rows of the step, cu_q, req_slots, token_req)`` over PORTIONS and join its outputs per sequence."""
    at, got = {k: 0 for k in TOTAL}, {k: [] for k in TOTAL}
    for step in PORTIONS:
        for rid, _ in step:
            if at[rid] == 0:
                for s in states:
                    s[SLOT[rid]].zero_()      # the runner clears a slot when a new request takes it
        out = call(torch.cat([rows[rid][at[rid]:at[rid] + n] for rid, n in step]), *_run_arrays([(SLOT[r], n) for r, n in step]))
        k = 0
        for rid, n in step:
            got[rid].append(out[..., k:k + n, :].cpu())
            at[rid] += n
            k += n
    return {rid: torch.cat(parts, dim=-2) for rid, parts in got.items()}


# ---------------------------------------------------------------------------------------------
# each mechanism alone
# ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("width", [6, 64, 300])
@pytest.mark.parametrize("buckets, muls", [(1, (1, 1)), (37, (5, 3)), (2000003, (999983, 77))])
def test_rows_picked_by_pairs_of_tokens(width, buckets, muls):
    from qwen25vl_lite_amd.ops.previous_token import bigram_gather
    torch.manual_seed(width)
    rows = min(buckets, 500)
    table, pairs = torch.randn(90000, width), torch.randn(buckets + 1, width) if buckets < 1000 else None
    if pairs is None:       # products beyond 32 bits: a table that only says which row it is
        pairs = torch.arange(buckets + 1).float()[:, None].repeat(1, width)
        table = torch.zeros(90000, width)
    ids = {k: torch.tensor(random_tokens(n, 90000, n)) for k, n in TOTAL.items()}
    state = torch.zeros(2, 1, dtype=torch.int32, device="cuda")
    tab, par = table.cuda(), pairs.cuda()
    got = _over_portions([state], lambda x, cu, slots, req: bigram_gather(x[:, 0].int().cuda(), tab, par, state, cu, slots, req,
                                                                         *muls), {k: v[:, None] for k, v in ids.items()})
    for k, v in ids.items():
        row = plain.bigram_rows(v.tolist(), {"buckets": buckets, "mul_prev": muls[0], "mul_cur": muls[1]})
        assert torch.equal(got[k], table[v] + pairs[row]), k
    assert state[:, 0].tolist() == [int(ids["p"][-1]) + 1, int(ids["r"][-1]) + 1] and rows


@pytest.mark.parametrize("width", [7, 72, 1100])
@pytest.mark.parametrize("shift, mixes", [(True, 0), (False, 3), (True, 5)])
def test_mixes_with_the_previous_token_over_portions(width, shift, mixes):
    from qwen25vl_lite_amd.ops.previous_token import token_mix
    torch.manual_seed(width)
    w = torch.rand(width) if shift else None
    mu = torch.rand(mixes, width) if mixes else None
    xs = {k: torch.randn(n, width) for k, n in TOTAL.items()}
    prev = torch.zeros(2, width, device="cuda") if shift else None
    prev_mixed = torch.zeros(2, width, device="cuda") if mixes else None
    states = [s for s in (prev, prev_mixed) if s is not None]
    on = lambda t: None if t is None else t.cuda()
    got = _over_portions(states, lambda x, cu, slots, req: token_mix(
        x.cuda(), cu, slots, req, torch.float32, shift=on(w), prev=prev, mu=on(mu), prev_mixed=prev_mixed), xs)
    for k, x in xs.items():
        g = plain.towards_previous(x.double(), w.double()) if shift else x.double()
        want = torch.stack([plain.towards_previous(g, m.double()) for m in mu]) if mixes else g
        assert torch.allclose(got[k].double(), want, atol=1e-5), k


def _copies_case(n, s, width, groups, pending, seed, equal):
    torch.manual_seed(seed)
    t = {"a.mix": torch.eye(s) + 0.3 * torch.randn(s, s), "a.out": torch.randn(s), "a.in": torch.randn(s)}
    h = torch.randn(n, width)
    copies = None if equal else torch.randn(n, s, width) * 2
    w = 1 + 0.3 * torch.randn(width)
    y = y64 = None
    if pending == "slabs":
        y = torch.randn(3, n, width)
        y64 = y.double().sum(0)
    elif pending == "mean":
        from qwen25vl_lite_amd.parts import NormedMean
        a, b = torch.randn(2, n, width), torch.randn(n, width) * 5
        g = 1 + 0.3 * torch.randn(2, width)
        y = NormedMean(a.cuda(), b.cuda(), g[0].contiguous().cuda(), g[1].contiguous().cuda(), 1e-4, 0.5)
        y64 = 0.5 * (plain.unit_rms(a.double().sum(0), 1e-4) * g[0].double() + plain.unit_rms(b.double(), 1e-4) * g[1].double())
    elif pending is not None:
        y = torch.randn(n, width).to(getattr(torch, pending))
        y64 = y.double()
    old = (h[None].repeat(s, 1, 1) if equal else copies.permute(1, 0, 2)).double()
    t64 = {k: v.double() for k, v in t.items()}
    new = old if pending is None else plain.join(old, y64, t64, "a.")
    return t, h, copies, w, (y if y is None or pending == "mean" else y.cuda()), new, t64


@pytest.mark.parametrize("s, width, groups", [(1, 40, 1), (2, 50, 5), (3, 72, 3), (4, 96, 4), (5, 1048, 2), (4, 4400, 4),
                                              (2, 2050, 2)])
@pytest.mark.parametrize("pending", [None, "float32", "bfloat16", "slabs", "mean"])
@pytest.mark.parametrize("equal", [False, True])
def test_copies_joined_read_and_normed_in_one_pass(s, width, groups, pending, equal):
    """Every copy from the copies as they were; the norm in parts of the row; chosen rows of the copies' sum."""
    from qwen25vl_lite_amd.ops.hyper import join_norm
    t, h, copies, w, y, new, t64 = _copies_case(9, s, width, groups, pending, s + width, equal)
    join = None if pending is None else (t["a.mix"].cuda(), t["a.out"].cuda())
    want = plain.grouped_norm(plain.read(new, t64, "a."), w.double(), groups, 1e-5)
    scale = new.abs().max().item()
    for out_dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2e-2)):
        c = None if copies is None else copies.cuda()
        got, after = join_norm(h.cuda(), c, join, y, t["a.in"].cuda(), w.cuda(), groups, 1e-5, out_dtype, num_copies=s)
        assert torch.allclose(got.double().cpu(), want, atol=tol, rtol=tol)
        if pending is None:
            assert after is c
        else:
            assert torch.allclose(after.double().cpu().permute(1, 0, 2), new, atol=1e-6 * scale + 1e-5)
            assert c is None or after.data_ptr() == c.data_ptr()
    rows = [7, 0, 3]
    c = None if copies is None else copies.cuda()
    got, _ = join_norm(h.cuda(), c, join, y, None, w.cuda(), groups, 1e-5, torch.float32, num_copies=s, rows=_i32(rows))
    want = plain.grouped_norm(new.sum(0)[rows], w.double(), groups, 1e-5)
    assert torch.allclose(got.double().cpu(), want, atol=2e-5, rtol=2e-5)
    assert c is None or torch.equal(c.cpu(), copies)          # choosing rows writes nothing


@pytest.mark.parametrize("s, width, groups", [(3, 72, 3), (1, 50, 1), (4, 1048, 2), (2, 4400, 4)])
@pytest.mark.parametrize("shift, mixes", [(True, 0), (False, 2), (True, 5)])
def test_single_tokens_are_mixed_behind_the_norm_as_runs_are(s, width, groups, shift, mixes):
    """One token of five requests with state rows anywhere: the norm's kernel against norm, then mixes; two steps."""
    from qwen25vl_lite_amd.ops.hyper import SingleTokens, join_norm
    torch.manual_seed(width)
    n, slots = 5, [6, 0, 3, 2, 5]
    sh = torch.rand(width) if shift else None
    mu = torch.rand(mixes, width) if mixes else None
    on = lambda v: None if v is None else v.cuda()
    prev, prev_mixed = torch.randn(8, width), torch.randn(8, width)
    dev_prev, dev_mixed = prev.cuda() if shift else None, prev_mixed.cuda() if mixes else None
    for seed in (1, 2):
        t, h, copies, w, y, new, t64 = _copies_case(n, s, width, groups, "float32", seed, False)
        got, _ = join_norm(h.cuda(), copies.cuda(), (t["a.mix"].cuda(), t["a.out"].cuda()), y, t["a.in"].cuda(), w.cuda(), groups,
                           1e-5, torch.float32, num_copies=s,
                           single=SingleTokens(_i32(slots), on(sh), dev_prev, on(mu), dev_mixed))
        g = plain.grouped_norm(plain.read(new, t64, "a."), w.double(), groups, 1e-5)
        if shift:
            before = prev.double()[slots]
            prev[slots] = g.float()
            g = g + (before - g) * sh.double()
        want = g
        if mixes:
            before = prev_mixed.double()[slots]
            want = torch.stack([g + (before - g) * m.double() for m in mu])
            prev_mixed[slots] = g.float()
        assert torch.allclose(got.double().cpu(), want, atol=3e-5, rtol=3e-5)
        assert not shift or torch.allclose(dev_prev.cpu(), prev, atol=3e-5, rtol=3e-5)
        assert not mixes or torch.allclose(dev_mixed.cpu(), prev_mixed, atol=3e-5, rtol=3e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("c, stride", [(70, 70), (72, 96), (1100, 2200)])
@pytest.mark.parametrize("taps", [1, 2, 4, 7])
def test_convolution_with_bias_and_silu(taps, c, stride, dtype):
    """Runs in portions shorter and longer than the taps; a slot used again; columns of a wider tensor."""
    from qwen25vl_lite_amd.ops.short_conv import short_conv
    torch.manual_seed(taps + c)
    w, b = torch.randn(c, taps), torch.randn(c)
    xs = {k: torch.randn(n, c).to(dtype) for k, n in TOTAL.items()}
    state = torch.zeros(2, taps - 1, c, device="cuda") if taps > 1 else None

    def call(x, cu, slots, req):
        wide = torch.full((x.shape[0], stride), 5.0, dtype=dtype, device="cuda")
        wide[:, :c] = x.cuda()
        return short_conv(wide[:, :c], w.t().contiguous().cuda(), state, cu, slots, req, dtype, bias=b.cuda(), silu=True)
    got = _over_portions([] if state is None else [state], call, xs)
    for k, x in xs.items():
        want = plain.silu(plain.causal_conv(x.double(), w.double(), b.double()))
        tol = 2e-5 if dtype == torch.float32 else 2e-2
        assert torch.allclose(got[k].double(), want, atol=tol, rtol=tol), k


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("c, states", [(88, 8), (300, 16), (27, 35), (64, 1), (70, 3), (130, 40)])
def test_selective_scan_alone(c, states, dtype):
    """Runs of unequal length from states that are not zero, scanned whole and in chunks side by side (the last
    chunk short, a run of one token beside a long one), against the loop over tokens."""
    from qwen25vl_lite_amd.ops.linear_attention import plan_chunks
    from qwen25vl_lite_amd.ops.selective_scan import LOG2_E, selective_scan
    torch.manual_seed(c + states)
    lens = [150, 1, 70, 2]
    n = sum(lens)
    x, z = torch.randn(n, c).to(dtype), torch.randn(n, 2 * c).to(dtype)
    dt, bias = torch.randn(n, c), torch.randn(c) - 1.0
    a = -torch.exp(torch.log(torch.arange(1, states + 1).float())[None, :] + 0.3 * torch.randn(c, states))
    bc, d = torch.randn(n, 5 + 2 * states), torch.randn(c)
    start = torch.randn(6, states, c)
    slots = [4, 0, 5, 2]
    cu, sl, _ = _run_arrays(list(zip(slots, lens)))
    a2 = (a.t() * LOG2_E).contiguous().cuda()
    tol = 3e-5 if dtype == torch.float32 else 2e-2
    for plan in (None, plan_chunks([0, 150, 151, 221, 223], "cuda"), plan_chunks([0, 150, 151, 221, 223], "cuda", 16)):
        state = start.cuda()
        got = selective_scan(x.cuda(), dt.cuda(), bias.cuda(), a2, bc.cuda(), 5, 5 + states, d.cuda(), z.cuda()[:, c:], state,
                             cu, sl, plan).double().cpu()
        at = 0
        for slot, m in zip(slots, lens):
            rows = slice(at, at + m)
            S, out = start[slot].double().t(), torch.zeros(m, c, dtype=F64)
            steps = plain.softplus(dt[rows].double() + bias.double())
            for i in range(m):
                S = torch.exp(steps[i][:, None] * a.double()) * S + (steps[i] * x[at + i].double())[:, None] * bc[at + i, 5:5 + states].double()
                out[i] = S @ bc[at + i, 5 + states:].double() + d.double() * x[at + i].double()
            want = out * plain.silu(z[rows, c:].double())
            scale = want.abs().max().item()
            assert torch.allclose(got[rows], want, atol=tol * scale), (slot, (got[rows] - want).abs().max())
            assert torch.allclose(state[slot].double().cpu(), S.t(), atol=3e-5 * S.abs().max().item()), slot
            at += m
        untouched = [1, 3]
        assert torch.equal(state[untouched].cpu(), start[untouched])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, dim, vdim", [(2, 16, 16), (3, 5, 5), (1, 64, 64), (2, 32, 80), (5, 8, 8)])
def test_recurrence_with_bonus_and_double_exponential_decay(heads, dim, vdim, dtype):
    """Scanned whole, with the key channels in groups, and in chunks side by side, from states that are not zero;
    q, k and v as parts of one tensor.  Without a bonus the token itself counts after the state has moved on."""
    from qwen25vl_lite_amd.ops.linear_attention import chunked_scan, decayed_scan, plan_chunks
    torch.manual_seed(heads + dim)
    lens, slots = [140, 1, 66, 3], [3, 0, 4, 1]
    n, hk, hv = sum(lens), heads * dim, heads * vdim
    wide = max(hk, hv)
    proj = torch.randn(3, n, wide).to(dtype)
    z, zb, u = torch.randn(n, hk) - 2.0, 0.5 * torch.randn(hk), torch.randn(hk)
    start = torch.randn(5, heads, dim, vdim)
    cu, sl, _ = _run_arrays(list(zip(slots, lens)))
    plan = plan_chunks([0, 140, 141, 207, 210], "cuda")
    w = torch.exp(-torch.exp(z.double() + zb.double())).view(n, heads, dim)
    for bonus in (True, False):
        want, last, at = torch.zeros(n, heads, vdim, dtype=F64), {}, 0
        for slot, m in zip(slots, lens):
            S = start[slot].double()
            for i in range(at, at + m):
                q, k = proj[0, i, :hk].double().view(heads, dim), proj[1, i, :hk].double().view(heads, dim)
                kv = k[:, :, None] * proj[2, i, :hv].double().view(heads, 1, vdim)
                new = w[i][:, :, None] * S + kv
                seen = S + u.double().view(heads, dim)[:, :, None] * kv if bonus else new
                want[i] = (seen * q[:, :, None]).sum(1)
                S = new
            last[slot] = S
            at += m
        how = dict(z=z.cuda(), z_bias=zb.cuda(), exp_decay=True, bonus=u.cuda() if bonus else None)
        tol = 3e-5 * want.abs().max().item()
        groups = [g for g in (1, 2, 4) if g == 1 or dim % (4 * g) == 0]
        for kind in groups + ["chunks"]:
            state = start.cuda()
            p = proj.cuda()
            if kind == "chunks":
                out = chunked_scan(p, 0, wide, 2 * wide, heads, dim, vdim, state, plan, sl, **how)
            else:
                out = decayed_scan(p, 0, wide, 2 * wide, heads, dim, vdim, state, cu, sl, groups=kind, **how)
            got = out.sum(0).double().cpu().view(n, heads, vdim)
            assert torch.allclose(got, want, atol=tol), (kind, bonus, (got - want).abs().max())
            for slot, S in last.items():
                assert torch.allclose(state[slot].double().cpu(), S, atol=3e-5 * S.abs().max().item()), (kind, slot)
            assert torch.equal(state[2].cpu(), start[2])


@pytest.mark.parametrize("dtype, rows, width, ff", [(torch.float32, 70, 56, 27), (torch.float32, 3, 56, 88), (torch.bfloat16, 5, 64, 88),
                                                   (torch.bfloat16, 20, 64, 40), (torch.bfloat16, 70, 64, 88), (torch.bfloat16, 70, 56, 27)])
def test_feed_forward_with_gelu(dtype, rows, width, ff):
    """Inside the product's kernel (few rows) and behind it, gate and up in groups of eight or not; large gates too."""
    from qwen25vl_lite_amd.parts.base import PartSpec, build_part
    torch.manual_seed(rows + ff)
    t = {k: (torch.randn(*shape) / shape[1] ** 0.5 * (4.0 if k == "gate" else 1.0)).to(torch.bfloat16)
         for k, shape in (("gate", (ff, width)), ("up", (ff, width)), ("down", (width, ff)))}
    part = build_part("ffn", PartSpec("swiglu", {"hidden_size": width, "intermediate_size": ff, "activation": "gelu_tanh",
                                                 "names": {k: k for k in t}}), dtype, torch.device("cuda:0"))
    part.load({f"{k}.weight": v.to(dtype).cuda() for k, v in t.items()})
    x = torch.randn(rows, width, dtype=F64)
    store = plain._keep if dtype == torch.float32 else plain.to_bfloat16_and_back
    t64 = {k: v.double() for k, v in t.items()}
    want = plain.gated_ff(store(x), t64, "", store)
    got = part.forward(x.to(dtype).cuda(), SimpleNamespace(residual=None))
    got = (got.sum(0) if got.dim() == 3 else got).double().cpu()
    assert torch.allclose(got, want, atol=(2e-5 if dtype == torch.float32 else 3e-2) * want.abs().max().item())
    silu = store(plain.silu(store(store(x) @ t64["gate"].T)) * store(store(x) @ t64["up"].T)) @ t64["down"].T
    assert not torch.allclose(silu, want, atol=3e-2 * want.abs().max().item())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("s, rows, n, k", [(4, 1, 48, 56), (4, 8, 3584, 3584), (2, 20, 70, 64), (3, 32, 1000, 2048), (4, 9, 15, 50),
                                           (4, 100, 48, 72), (5, 17, 200, 4096)])
def test_a_stack_of_products(s, rows, n, k, dtype):
    from qwen25vl_lite_amd.ops.linear import linear_stack
    torch.manual_seed(n)
    x, w = torch.randn(s, rows, k).to(dtype), (torch.randn(s, n, k) / k ** 0.5).to(dtype)
    got = linear_stack(x.cuda(), w.cuda()).double().cpu()
    want = torch.stack([a.double() @ b.double().T for a, b in zip(x, w)])
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    assert torch.allclose(got, want, atol=tol, rtol=tol)


# ---------------------------------------------------------------------------------------------
# a mixer in its layer
# ---------------------------------------------------------------------------------------------
def _one_layer(tmp_path, lay, dtype=torch.float32, seed=0, width=56, tensors_edit=None, name="one", streams=2, max_live=3):
    from qwen25vl_lite_amd.config import EngineConfig, load_config
    from qwen25vl_lite_amd.engine import ModelRunner
    from qwen25vl_lite_amd.models import build_model
    from qwen25vl_lite_amd.weights import load_weights
    cfg = zu.config(width, 50, lay if isinstance(lay, list) else [lay], streams=streams, groups=2, eps=1e-4)
    tensors = zu.random_tensors(cfg, seed)
    if tensors_edit is not None:
        tensors_edit(tensors)
    d = zu.write_model(str(tmp_path / name), cfg, seed, tensors)
    model = build_model(load_config(d), dtype, "cuda:0")
    load_weights(d, model)
    ecfg = EngineConfig(num_blocks=48, block_size=16, max_num_seqs=max_live, max_num_batched_tokens=512, max_model_len=512,
                        enable_prefix_cache=False, dtype=dtype)
    cfg, t64 = plain.zaposun_read(d, F64)
    return ModelRunner(model, ecfg), model, cfg, t64


def _run_mixer(runner, call, runs, x):
    """``call(x, step, entry slot)`` for ``runs``: (request id, tokens, start); a request is admitted at start 0."""
    from qwen25vl_lite_amd.engine import StepEntry
    from qwen25vl_lite_amd.engine.batch import build_step
    entries = []
    for rid, n, start in runs:
        if start == 0:
            runner.admit(rid)
        entries.append(StepEntry(rid, [0] * n, start))
        runner.cache.reserve(rid, start + n)
    runner._clear_state(entries)
    step = build_step(entries, runner.cache, 1, runner.dtype, runner.device)
    out = call(x.cuda(), step, runner.slots[0])
    for rid, n, start in runs:
        runner.cache.commit(rid, start + n)
    return (out.sum(0) if out.dim() == 3 else out).double().cpu()


LEFT = {"attention": zu.left(6, 2, 24, 16, 37, base=80.0, dims=16, scale=0.7),
        "attention_full_rotation": zu.left(2, 2, 16, 16, 20, base=30.0, scale=0.5),
        "attention_values_by_registers": zu.left(4, 2, 64, 32, 50, base=200.0, dims=32, scale=0.4),
        "attention_wide_values": zu.left(4, 1, 16, 24, 90, base=500.0, dims=8, scale=0.9),
        "attention_long_chunk": zu.left(3, 3, 16, 16, 1000, base=50.0, dims=4, scale=0.6),
        "attention_one_token": zu.left(2, 1, 8, 8, 1, base=20.0, scale=0.6),
        "attention_no_rotation": zu.left(3, 1, 10, 14, 5, base=77.0, dims=0, scale=0.5)}
RIGHT = {"state_space": zu.right(88, 8, 5, 3), "state_space_one": zu.right(1, 1, 1, 1), "state_space_wide": zu.right(300, 16, 24, 4),
         "state_space_odd": zu.right(27, 35, 3, 5)}
WKV = {"wkv": zu.wkv(3, 16), "wkv_one": zu.wkv(1, 8), "wkv_odd": zu.wkv(3, 5), "wkv_wide": zu.wkv(2, 64)}


def _mixer_case(case, tmp_path, dtype):
    """``(runner, call, plain function of x)`` of a mixer by itself."""
    some_left, some_right = LEFT["attention"], RIGHT["state_space"]
    if case in WKV:
        runner, model, cfg, t = _one_layer(tmp_path, zu.layer(WKV[case]), dtype)
        m = WKV[case]["mixer"]
        return (runner, lambda x, step, slot: model.blocks[0].mixer.forward(x.float(), step, slot.of("mix")),
                lambda x, store: plain.wkv(x, None, t, "l0.mix.", m, 1e-4, store))
    if case in LEFT:
        runner, model, cfg, t = _one_layer(tmp_path, zu.layer(zu.parallel(LEFT[case], some_right)), dtype)
        return (runner, lambda x, step, slot: model.blocks[0].mixer.left.forward(x.to(dtype), step, slot.of("mix").of("left")),
                lambda x, store: plain.chunked_attention(store(x), torch.arange(x.shape[0]), t, "l0.mix.left.", LEFT[case], 1e-4, store))
    runner, model, cfg, t = _one_layer(tmp_path, zu.layer(zu.parallel(some_left, RIGHT[case])), dtype)
    return (runner, lambda x, step, slot: model.blocks[0].mixer.right.forward(x.to(dtype), step, slot.of("mix").of("right")),
            lambda x, store: plain.mamba(store(x), t, "l0.mix.right.", RIGHT[case], store))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case", sorted({**LEFT, **RIGHT, **WKV}))
def test_a_mixer_alone_whole_in_two_steps_and_token_by_token(case, dtype, tmp_path):
    """The mixer's own forward against the plain function: one run of 150 tokens (scanned in chunks), the same cut
    inside a page, and (in float32) the last tokens one by one beside another request's prompt."""
    runner, call, fn = _mixer_case(case, tmp_path, dtype)
    torch.manual_seed(5)
    n = 150
    x, other = torch.randn(n, 56), torch.randn(21, 56)
    store = plain._keep if dtype == torch.float32 else plain.to_bfloat16_and_back
    want, want_other = fn(x.double(), store), fn(other.double(), store)
    tol = (2e-5 if dtype == torch.float32 else 4e-2) * want.abs().max().item()
    got = _run_mixer(runner, call, [("a", n, 0)], x)
    assert torch.allclose(got, want, atol=tol), (got - want).abs().max()
    first = _run_mixer(runner, call, [("b", 23, 0)], x[:23])
    second = _run_mixer(runner, call, [("b", n - 23, 23)], x[23:])
    assert torch.allclose(torch.cat([first, second]), want, atol=tol)
    if dtype == torch.float32:
        runner.release("a")
        runner.release("b")
        rows = [_run_mixer(runner, call, [("d", 2, 0)], x[:2])]
        for p in range(2, 90):
            if p == 30:      # another request's whole prompt beside the decoded token
                out = _run_mixer(runner, call, [("o", 21, 0), ("d", 1, p)], torch.cat([other, x[p:p + 1]]))
                assert torch.allclose(out[:21], want_other, atol=tol)
                rows.append(out[21:])
            else:
                rows.append(_run_mixer(runner, call, [("d", 1, p)], x[p:p + 1]))
        assert torch.allclose(torch.cat(rows), want[:90], atol=tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("hd, vd", [(64, 32), (16, 24), (24, 16)])
@pytest.mark.parametrize("share", [False, True])
def test_attention_kernels_at_chunk_edges(hd, vd, share, dtype):
    """One key's score stands out by far: the tokens of its chunk from it on see it, the next chunk's first does not.
    Both kinds of the matrix-core kernel and the generic one; values lie in the pages turned and come back unturned."""
    from qwen25vl_lite_amd.ops import attention_window, kernels
    torch.manual_seed(hd)
    n, ps, chunk, nq, nkv = 90, 16, 21, 4, 2
    pages = (n + ps - 1) // ps
    q, k, v = torch.randn(n, nq, hd), 0.05 * torch.randn(n, nkv, hd), torch.randn(n, nkv, vd)
    q[..., 0] = 3.0
    for loud in (20, 21, 33, 62, 63):                       # a chunk's last and first positions among them
        k[loud, :, 0] = 4.0
    pos = torch.arange(n)
    f = plain.frequencies(50.0, vd)
    angle = pos.double()[:, None] * f[None, :]
    turn = torch.stack([angle.cos(), angle.sin()], dim=-1).float().cuda()
    qr, kr = q.to(dtype), k.to(dtype)
    vr = plain.rotate(v.double(), pos, f).to(dtype)
    want = plain.rotate(plain.attend_in_chunks(qr.double(), kr.double(), vr.double(), 1.0, chunk), -pos, f)
    table = torch.randperm(pages)
    kc, vc = torch.zeros(pages, nkv, ps, hd, dtype=dtype), torch.zeros(pages, nkv, vd, ps, dtype=dtype)
    for p in range(n):
        kc[table[p // ps], :, p % ps], vc[table[p // ps], :, :, p % ps] = kr[p], vr[p]
    for first in (0, 60, 89):                                # the whole prompt, a portion of it, one decoded token
        m = n - first
        cu = _i32([0, m])
        step = SimpleNamespace(num_reqs=1, cu_q=cu, cu_q_host=[0, m], ctx_len=_i32([n]), ctx_len_host=[n], max_q_len=m, derived={})
        args = (qr[first:].reshape(m, -1).contiguous().cuda(), kc.cuda(), vc.cuda(), table.int().view(1, -1).cuda())
        if dtype == torch.bfloat16:
            got = attention_window.try_attention(*args, step, nq, None, 0, 1.0, share=share, chunk=chunk,
                                                 turn=turn[first:].contiguous())
        else:
            got = kernels.paged_attention_generic(*args, _i32([0] * m), _i32(range(first, n)), nq, None, 1.0, chunk=chunk,
                                                  turn=turn[first:].contiguous())
        tol = 2e-5 if dtype == torch.float32 else 3e-2
        assert torch.allclose(got.double().cpu().view(m, nq, vd), want[first:], atol=tol), first
    # one position less or more in a chunk moves the result: the inputs above would show it
    for other in (20, 22):
        off = plain.rotate(plain.attend_in_chunks(qr.double(), kr.double(), vr.double(), 1.0, other), -pos, f)
        assert (off - want).abs().amax(dim=(1, 2))[[21, 63]].max() > 0.3


def test_values_that_are_turned_in_neighbouring_pairs():
    """The other layout of pairs: written turned and read back turned back, in both kernels."""
    from qwen25vl_lite_amd.ops import attention_window, gated, kernels
    torch.manual_seed(3)
    n, ps, nq, nkv, hd, vd, rot = 33, 16, 2, 1, 16, 24, 8
    x = torch.randn(n, (nq + nkv) * hd + nkv * vd)
    fk, fv = plain.frequencies(30.0, rot), plain.frequencies(30.0, vd)
    table = lambda f: torch.stack([(torch.arange(n).double()[:, None] * f).cos(), (torch.arange(n).double()[:, None] * f).sin()], -1).float()

    def near(x, f, sign=1.0):
        angle = sign * torch.arange(n, dtype=F64)[:, None] * f
        c, s = angle.cos()[:, None], angle.sin()[:, None]
        out = x.clone()
        m = 2 * f.shape[0]
        out[..., 0:m:2], out[..., 1:m:2] = x[..., 0:m:2] * c - x[..., 1:m:2] * s, x[..., 1:m:2] * c + x[..., 0:m:2] * s
        return out
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 4e-2)):
        kc, vc = torch.zeros(3, nkv, ps, hd, dtype=dtype, device="cuda"), torch.zeros(3, nkv, vd, ps, dtype=dtype, device="cuda")
        q = gated.qk_norm_rope_write(x.cuda(), None, None, 0.0, table(fk).cuda(), _i32(range(n)), kc, vc, nq, nkv, hd, ps, dtype,
                                     interleaved=True, values_are_keys=False, norm=None, value_dim=vd, value_cs=table(fv).cuda())
        xd = x.double()
        qw, kw = near(xd[:, :nq * hd].view(n, nq, hd), fk), near(xd[:, nq * hd:(nq + nkv) * hd].view(n, nkv, hd), fk)
        vw = near(xd[:, (nq + nkv) * hd:].view(n, nkv, vd), fv)
        got_v = vc.permute(0, 3, 1, 2).reshape(3 * ps, nkv, vd)[:n]
        assert torch.allclose(got_v.double().cpu(), vw, atol=tol, rtol=tol)
        want = near(plain.attend_in_chunks(qw, kw, vw, 0.3, None), fv, -1.0)
        step = SimpleNamespace(num_reqs=1, cu_q=_i32([0, n]), cu_q_host=[0, n], ctx_len=_i32([n]), ctx_len_host=[n], max_q_len=n, derived={})
        if dtype == torch.float32:
            got = kernels.paged_attention_generic(q, kc, vc, _i32([0, 1, 2]).view(1, 3), _i32([0] * n), _i32(range(n)), nq, None, 0.3,
                                                  turn=table(fv).cuda(), turn_pairs=True)
        else:
            got = attention_window.try_attention(q, kc, vc, _i32([0, 1, 2]).view(1, 3), step, nq, None, 0, 0.3, turn=table(fv).cuda(),
                                                 turn_pairs=True)
        assert torch.allclose(got.double().cpu().view(n, nq, vd), want, atol=tol * want.abs().max().item())


def test_a_layers_copies_against_the_plain_models(tmp_path):
    """After a whole step of three layers the copies equal the plain model's streams, each of them."""
    from qwen25vl_lite_amd.engine import StepEntry
    layers = [zu.layer(zu.wkv(2, 8), 24), zu.layer(zu.parallel(LEFT["attention"], RIGHT["state_space"]), 40), zu.layer(zu.wkv(1, 16))]
    runner, model, cfg, t = _one_layer(tmp_path, layers, streams=3)
    toks = random_tokens(19, 50, 2)
    kept = {}
    inner = model.final_norm.forward

    def spy(stream, rows=None, **kw):
        kept["copies"] = (stream.copies.double().cpu(), stream.pending.double().cpu(), stream.pending_join)
        return inner(stream, rows=rows, **kw)
    model.final_norm.forward = spy
    runner.admit("a")
    runner.execute([StepEntry("a", toks, 0, want=[len(toks) - 1])])
    streams = torch.stack([plain.embed(cfg, t, toks)] * 3)
    for i in range(3):
        streams = plain.layer(cfg, t, i, streams, torch.arange(len(toks)))
    copies, pending, (mix, out) = kept["copies"]
    pending = pending.sum(0) if pending.dim() == 3 else pending
    got = plain.join(copies.permute(1, 0, 2), pending, {"mix": mix.double().cpu(), "out": out.double().cpu()}, "")
    assert torch.allclose(got, streams, atol=2e-5 * streams.abs().max().item())
    assert (streams[0] - streams[1]).abs().max() > 0.1 * streams.abs().max()        # they are not copies of one another


# ---------------------------------------------------------------------------------------------
# whole models, every schedule
# ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name", ["mixed", "ones", "odd", "no_pages"])
def test_float32_every_schedule_against_the_plain_model(name, folders):
    """Whole prompts, decoding, portions down to two tokens, mixed batches with more requests than slots: all the
    same logits, and the plain model's."""
    folder = folders[name]
    cfg, _ = plain.zaposun_read(folder, F64)
    reqs = _requests(cfg["vocab"], seed=20)
    want = {rid: _oracle(folder, toks) for rid, toks in reqs.items()}
    mixed, peak = mixed_trace(reqs, seed=4, max_live=4)
    holders = {}
    for steps, size in ((whole_trace(reqs), 192), (tail_trace(reqs, 50), 192), (portion_trace(reqs), 192), (mixed, peak)):
        got = run_steps(_replayer(folder, "float32", size), steps, holders if steps is mixed else None)
        for rid, toks in reqs.items():
            assert _rel(_rows(got, rid, len(toks)), want[rid]) < 2e-5, (name, rid)
    if name != "no_pages":
        assert any(len(who) > 1 for who in holders.values()), "no page was used by two requests"


@pytest.mark.parametrize("name", ["mixed", "ones", "odd", "no_pages"])
def test_bfloat16_within_rounding_of_the_plain_model(name, folders):
    """bfloat16 kernels: no further from exact arithmetic than rounding the stored activations to bfloat16 takes the
    plain model, whatever the schedule."""
    folder = folders[name]
    cfg, _ = plain.zaposun_read(folder, F64)
    reqs = _requests(cfg["vocab"], seed=30)
    exact = {rid: _oracle(folder, toks) for rid, toks in reqs.items()}
    rounding = torch.cat([_rel_rows(_oracle(folder, toks, plain.to_bfloat16_and_back), exact[rid])
                          for rid, toks in reqs.items()])
    mixed, peak = mixed_trace(reqs, seed=5, max_live=4)
    for steps, size in ((whole_trace(reqs), 192), (tail_trace(reqs, 50), 192), (portion_trace(reqs), 192), (mixed, peak)):
        got = run_steps(_replayer(folder, "bfloat16", size), steps)
        errors = torch.cat([_rel_rows(_rows(got, rid, len(toks)), exact[rid]) for rid, toks in reqs.items()])
        assert _like_rounding(errors, rounding), (name, errors.median(), rounding.median(), errors.quantile(0.9),
                                                  rounding.quantile(0.9))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_peaked_attention_at_chunk_edges_and_far_keys(dtype, folders):
    """Score scales so large that the softmax picks single keys, across page borders and at the chunks' edges.  The
    last 70 tokens are decoded, so every layer's chunks begin among decoded tokens; then the same in portions."""
    folder = folders["sharp"]
    toks = random_tokens(330, zu.SHARP["vocab"], 40)
    want = _oracle(folder, toks)
    if dtype == "float32":
        # scores this large make float32 arithmetic itself visible: the measure is the plain model run in float32
        cfg, t32 = plain.zaposun_read(folder, torch.float32)
        rounding, slack = _rel_rows(plain.zaposun_forward(cfg, t32, toks), want), 1e-5
    else:
        rounding, slack = _rel_rows(_oracle(folder, toks, plain.to_bfloat16_and_back), want), 1e-3
    for steps in (tail_trace({"s": toks}, 70), portion_trace({"s": toks}, (64, 3, 41, 2, 17, 90))):
        got = _rows(run_steps(_replayer(folder, dtype, round64(len(toks))), steps), "s", len(toks))
        errors = _rel_rows(got, want)
        assert _like_rounding(errors, rounding, slack), (errors.median(), rounding.median(), errors.quantile(0.9),
                                                         rounding.quantile(0.9))
        assert errors.max() < 4 * rounding.max() + slack, (errors.max(), rounding.max())


def test_what_the_schedules_would_show(folders):
    """Each of these changes the plain model's last logits well beyond the tolerances above: chunks one position
    longer, a step towards the previous token left out, a bigram row of the pair the other way round, a bonus left
    out, values not turned, a mix of copies transposed, a norm in one part, the far past replaced."""
    toks = random_tokens(330, zu.SHARP["vocab"], 40)
    folder = folders["sharp"]
    whole = _oracle(folder, toks)

    def chunks(cfg):
        for lay in cfg["layers"]:
            if lay["type"] == "parallel":
                lay["mixer"]["left"]["mask"]["size"] += 1

    def swap(cfg):
        b = cfg["embedding"]["bigram"]
        b["mul_prev"], b["mul_cur"] = b["mul_cur"], b["mul_prev"]

    def zero(ending):
        def edit(t):
            for name in t:
                if name.endswith(ending):
                    t[name] = torch.zeros_like(t[name])
        return edit

    def transpose(t):
        for name in t:
            if name.endswith(".mix"):
                t[name] = t[name].T.contiguous()

    def one_part(cfg):
        cfg["norm"]["groups"] = 1

    for kw in ({"cfg_edit": chunks}, {"cfg_edit": swap}, {"cfg_edit": one_part}, {"tensors_edit": zero(".shift")},
               {"tensors_edit": zero(".mix.u")}, {"tensors_edit": zero(".mu.w")}, {"tensors_edit": transpose}):
        assert _rel(_oracle(folder, toks, **kw)[-30:], whole[-30:]) > 0.02, kw
    turned = plain.rotate
    try:
        plain.rotate = lambda x, pos, f: turned(x, pos, f) if x.shape[1] != 1 and pos[-1] >= 0 else x
        assert _rel(_oracle(folder, toks)[-30:], whole[-30:]) > 0.02
    finally:
        plain.rotate = turned
    other = random_tokens(290, zu.SHARP["vocab"], 41) + toks[290:]
    assert _rel(_oracle(folder, other)[-30:], whole[-30:]) > 0.02


def test_long_decoding(folders):
    """A short prompt and 200 tokens decoded one by one, through several pages and chunks."""
    folder = folders["mixed"]
    toks = random_tokens(205, zu.MIXED["vocab"], 50)
    want = _oracle(folder, toks)
    got = _rows(run_steps(_replayer(folder, "float32", 256), tail_trace({"l": toks}, 200)), "l", len(toks))
    assert _rel(got, want) < 2e-5


def test_chunked_groups_give_pages_back_while_decoding(folders):
    from qwen25vl_lite_amd.engine.replay import Replayer
    rp = Replayer(folders["mixed"], "float32", 256, 16, 2)
    toks = random_tokens(200, zu.MIXED["vocab"], 51)
    run_steps(rp, [{"step": 0, "entries": [{"id": "x", "tokens": toks, "want": []}], "end": []}])
    cache = rp.runner.cache
    held = {g.need.chunk: [i for i, p in enumerate(cache.table("x", k)) if p >= 0] for k, g in enumerate(cache.groups)}
    # the next token is 200: chunks of 37 began at 185 (page 11), of 9 at 198 (page 12), of 64 at 192 (page 12)
    assert held == {37: [11, 12], 9: [12], 64: [12]}
    rp.step({"entries": [], "end": ["x"]})
    cache.check()


def test_a_fork_continues_from_the_same_states(folders):
    """Pages, recurrent states, the last rows and the last token all go to the fork."""
    from qwen25vl_lite_amd.engine import StepEntry
    rp = _replayer(folders["mixed"], "float32", 256)
    toks = random_tokens(60, zu.MIXED["vocab"], 55)
    want = _oracle(folders["mixed"], toks)
    runner = rp.runner
    runner.admit("a")
    runner.execute([StepEntry("a", toks[:41], 0)])
    runner.fork("a", "b")
    runner.execute([StepEntry("a", [1, 2, 3], 41)])            # the original goes elsewhere
    got = runner.execute([StepEntry("b", toks[41:], 41, want=list(range(19)))]).cpu()
    assert _rel(got, want[41:]) < 2e-5


@pytest.mark.parametrize("name", ["mixed", "no_pages"])
@pytest.mark.parametrize("graph", [False, True])
def test_greedy_generation_through_the_entry_point(graph, name, folders):
    """``LLM.generate`` with the scheduler (three prompts, two slots, portions of 16 tokens, decode steps from HIP
    graphs or not) picks the plain model's tokens."""
    from qwen25vl_lite_amd import LLM, SamplingParams
    folder = folders[name]
    vocab = CONFIGS[name][0]["vocab"]
    prompts = [random_tokens(n, vocab, 70 + n) for n in (37, 5, 21)]
    steps = 12
    want = []
    for p in prompts:
        ids = list(p)
        for _ in range(steps):
            ids.append(int(torch.argmax(_oracle(folder, ids)[-1])))
        want.append(ids[len(p):])
    with LLM(folder, dtype="float32", num_blocks=32, block_size=16, max_num_seqs=2, max_num_batched_tokens=16,
             hip_graph=graph) as llm:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True))
    assert [o.output_token_ids for o in outs] == want


def test_preempted_requests_start_again_from_cleared_states(folders):
    """Pages for one and a half requests: one gives way, is computed again from its first token, and both still pick
    the plain model's tokens."""
    from qwen25vl_lite_amd import LLM, SamplingParams
    folder = folders["mixed"]
    prompts = [random_tokens(n, zu.MIXED["vocab"], 170 + n) for n in (30, 27)]
    steps = 24
    want = []
    for p in prompts:
        ids = list(p)
        for _ in range(steps):
            ids.append(int(torch.argmax(_oracle(folder, ids)[-1])))
        want.append(ids[len(p):])
    with LLM(folder, dtype="float32", num_blocks=5, block_size=16, max_num_seqs=2, max_num_batched_tokens=32) as llm:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True))
    assert [o.output_token_ids for o in outs] == want


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_replay_program_and_the_command_line(dtype, folders, tmp_path):
    """``bin/trace_run`` as a user calls it on a Zaposun folder (steps on standard input, ``done`` lines, files of
    float32 logits), and ``generate`` of the command line, whose tokens are the plain model's."""
    import ast
    import json
    import os
    import subprocess
    import sys

    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder = folders["mixed"]
    vocab = zu.MIXED["vocab"]
    toks = random_tokens(45, vocab, 4)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": toks[:19], "want": [0, 18]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": toks[19:44], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": toks[44:], "want": [0]},
                                {"id": "b", "tokens": toks[:3], "want": [2]}], "end": ["a", "b"]},
    ]
    out = tmp_path / "out"
    proc = subprocess.run(
        [sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
         "--max-tokens", "128"],
        input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [w for w in proc.stdout.split() if w == "done" or w.isdigit()][-6:] == ["done", "0", "done", "1", "done", "2"]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32"]
    want = _oracle(folder, toks)
    s0 = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(2, vocab))
    s2 = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(2, vocab))
    # a sequence's first token, whose recurrences hold little yet, is moved further by rounding than the others
    rounding = _rel_rows(_oracle(folder, toks, plain.to_bfloat16_and_back), want)[[0, 18, 44, 2]]
    limit = torch.full((4,), 2e-5) if dtype == "float32" else 2 * rounding + 2e-3
    assert (_rel_rows(torch.cat([s0, s2]), want[[0, 18, 44, 2]]) < limit).all()
    if dtype == "float32":
        prompt = toks[:12]
        cli = [sys.executable, os.path.join(root, "bin", "qwen25vl-lite"), "generate", "--model", folder, "--dtype", "float32",
               "--num-blocks", "32", "--max-num-seqs", "2", "--max-model-len", "256", "--max-tokens", "6", "--ignore-eos",
               "--prompt-token-ids", ",".join(map(str, prompt))]
        proc = subprocess.run(cli, capture_output=True, text=True, timeout=110)
        assert proc.returncode == 0, proc.stderr[-2000:]
        ids = list(prompt)
        for _ in range(6):
            ids.append(int(torch.argmax(_oracle(folder, ids)[-1])))
        assert ast.literal_eval(proc.stdout.strip().splitlines()[-1]) == ids[len(prompt):]


def test_bfloat16_generation_from_graphs_matches_eager_steps(folders):
    from qwen25vl_lite_amd import LLM, SamplingParams
    prompts = [random_tokens(n, zu.MIXED["vocab"], 90 + n) for n in (18, 3, 40, 9)]
    outs = []
    for graph in (False, True):
        with LLM(folders["mixed"], dtype="bfloat16", num_blocks=48, block_size=16, max_num_seqs=4,
                 max_num_batched_tokens=64, hip_graph=graph) as llm:
            outs.append([o.output_token_ids for o in
                         llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True))])
    assert outs[0] == outs[1]
