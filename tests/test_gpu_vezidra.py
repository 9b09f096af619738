"""The Vezidra decoder on the GPU against the plain implementation in ``plain_vezidra.py``: each mechanism alone,
whole prompts, decoding, portions, mixed batches, pages and slots used again, peaked attention at window edges and far
back, sinks, the first tokens of a sequence, sizes that are 1, equal or odd, and greedy generation through ``LLM``."""

from types import SimpleNamespace

import pytest
import torch

import plain_vezidra as plain
import vezidra_util as vu
from replay_util import mixed_trace, portion_trace, random_tokens, round64, run_steps, tail_trace, whole_trace

pytestmark = pytest.mark.gpu

F64 = torch.float64
LENGTHS = {"a": 83, "b": 40, "c": 7, "d": 1, "e": 150, "f": 29, "g": 2}
CONFIGS = {"mixed": (vu.MIXED, 41), "sharp": (vu.SHARP, 42), "ones": (vu.ONES, 43), "odd": (vu.ODD, 44), "wide": (vu.WIDE, 45)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: vu.write_model(str(tmp_path_factory.mktemp(name)), cfg, seed) for name, (cfg, seed) in CONFIGS.items()}


def _oracle(folder, tokens, store=None, cfg_edit=None, tensors_edit=None):
    cfg, tensors = plain.vezidra_read(folder, F64)
    if cfg_edit is not None:
        cfg_edit(cfg)
    if tensors_edit is not None:
        tensors_edit(tensors)
    return plain.vezidra_forward(cfg, tensors, tokens, store or plain._keep).to(torch.float32)


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


# ---------------------------------------------------------------------------------------------
# each mechanism alone
# ---------------------------------------------------------------------------------------------
def _scan_case(h, g, d, v, rule, dtype, seed, lens, strong):
    """Inputs of a recurrence and what the plain loop makes of them, run by run from states that are not zero."""
    torch.manual_seed(seed)
    n, slots = sum(lens), [4, 0, 5, 2][:len(lens)]
    x = torch.randn(n, 2 * g * d + h * v + 4).to(dtype)
    raw = torch.randn(n, 2 * h + 3)
    bias, a_log = torch.randn(h) - 1.0, -0.5 + torch.randn(h)
    if strong:      # tokens that forget almost everything beside tokens that forget nothing
        raw[::7] += 30.0
        raw[1::7] -= 12.0
    skip = torch.randn(h)
    start = torch.randn(6, h, d, v)
    q = x[:, :g * d].double().view(n, g, d)
    k = x[:, g * d:2 * g * d].double().view(n, g, d)
    val = x[:, 2 * g * d + 4:2 * g * d + 4 + h * v].double().view(n, h, v)
    step = plain.softplus(raw[:, :h].double() + bias.double())
    decay = torch.exp(-torch.exp(a_log.double()) * step)
    if rule == "delta":
        q, k = plain.unit_vector(q) * d ** -0.5, plain.unit_vector(k)
    q, k = plain.spread(q, h), plain.spread(k, h)
    out, last, at = torch.zeros(n, h, v, dtype=F64), {}, 0
    for slot, m in zip(slots, lens):
        r = slice(at, at + m)
        if rule == "delta":
            beta = torch.sigmoid(raw[r, h + 1:2 * h + 1].double())
            out[r], last[slot] = plain.delta_rule(q[r], k[r], val[r], decay[r], beta, start[slot].double())
        else:
            out[r], last[slot] = plain.decayed_products(q[r], k[r], val[r], decay[r], step[r], start[slot].double())
            out[r] += skip.double()[None, :, None] * val[r]
        at += m
    how = (dict(beta_off=h + 1, unit_eps=plain.UNIT_FLOOR, q_scale=d ** -0.5) if rule == "delta" else dict(skip=skip.cuda()))
    return x, raw, bias, -torch.exp(a_log), start, slots, out, last, how


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rule", ["delta", "plain"])
@pytest.mark.parametrize("h, g, d, v", [(2, 1, 16, 16), (4, 2, 12, 20), (3, 3, 37, 5), (6, 3, 64, 80), (2, 1, 128, 48),
                                        (1, 1, 1, 1), (2, 2, 256, 24), (2, 1, 272, 16), (4, 1, 24, 33)])
def test_recurrences_with_one_decay_per_head(h, g, d, v, rule, dtype):
    """Runs of unequal length from states that are not zero, token after token and in chunks side by side (a last chunk
    that is short, a run of one token beside a long one, a run of exactly a chunk), with decays near zero and near one."""
    from qwen25vl_lite_amd.ops.head_scan import MAX_CHUNKED_KEY_SIZE, head_scan
    from qwen25vl_lite_amd.ops.linear_attention import plan_chunks
    lens = [150, 1, 64, 3]
    cu = [0, 150, 151, 215, 218]
    for strong in (False, True):
        x, raw, bias, a_neg, start, slots, want, last, how = _scan_case(h, g, d, v, rule, dtype, h + d, lens, strong)
        tol = 3e-5 * want.abs().max().item()
        for plan in (None, plan_chunks(cu, "cuda")):
            if plan is not None and d > MAX_CHUNKED_KEY_SIZE:
                continue
            state = start.cuda()
            got = head_scan(x.cuda(), 0, g * d, 2 * g * d + 4, h, g, d, v, raw.cuda(), 0, bias.cuda(), a_neg.cuda(), state,
                            _i32(cu), _i32(slots), plan=plan, **how).double().cpu().view(want.shape)
            assert torch.allclose(got, want, atol=tol), (plan is None, strong, (got - want).abs().max(), tol)
            for slot, S in last.items():
                assert torch.allclose(state[slot].double().cpu(), S, atol=3e-5 * S.abs().max().item()), (plan is None, slot)
            assert torch.equal(state[[1, 3]].cpu(), start[[1, 3]])


def test_a_slow_head_remembers_across_chunks():
    """One write at the first token, a decay so near one that it is read hundreds of tokens on; and the same key written
    again replaces it under the delta rule."""
    from qwen25vl_lite_amd.ops.head_scan import head_scan
    from qwen25vl_lite_amd.ops.linear_attention import plan_chunks
    n, d, v = 300, 8, 16
    x = torch.zeros(n, 2 * d + v)
    x[:, :d] = 0.01 * torch.randn(n, d)
    x[:, 2 * d + 1:] = 0.01
    x[0, d:2 * d] = x[200, d:2 * d] = x[299, :d] = x[199, :d] = torch.eye(d)[3] * 5
    x[0, 2 * d], x[200, 2 * d] = 7.0, -4.0
    raw = torch.full((n, 2), -12.0)           # beta and step of almost nothing
    raw[0, 1] = raw[200, 1] = 40.0            # but here beta is one
    state = torch.zeros(1, 1, d, v, device="cuda")
    cu = [0, n]
    for plan in (None, plan_chunks(cu, "cuda")):
        state.zero_()
        out = head_scan(x.cuda(), 0, d, 2 * d, 1, 1, d, v, raw.cuda(), 0, torch.zeros(1).cuda(), torch.full((1,), -1.0).cuda(), state,
                        _i32(cu), _i32([0]), beta_off=1, unit_eps=1e-6, q_scale=1.0, plan=plan).cpu()
        assert out[199, 0].item() == pytest.approx(7.0, rel=5e-3) and out[299, 0].item() == pytest.approx(-4.0, rel=5e-3)


@pytest.mark.parametrize("width", [7, 72, 1100, 3584, 4400])
@pytest.mark.parametrize("kinds", [("float32",), ("bfloat16",), ("slabs",), ("float32", "float32"), ("bfloat16", "slabs"),
                                   ("slabs", "bfloat16"), ("bfloat16", "bfloat16")])
@pytest.mark.parametrize("gains", [False, True])
@pytest.mark.parametrize("norm", [False, True])
def test_sum_and_norm_in_one_pass(width, kinds, gains, norm):
    from qwen25vl_lite_amd.ops.sum_norm import sum_norm_
    from qwen25vl_lite_amd.parts import SumTerm
    torch.manual_seed(width + len(kinds))
    n, eps, alpha = 5, 1e-4, 1.7
    h, w, b = 3 * torch.randn(n, width) + 1.0, 1 + 0.3 * torch.randn(width), torch.randn(width)
    want, terms = alpha * h.double(), []
    for i, kind in enumerate(kinds):
        y = torch.randn(3, n, width) if kind == "slabs" else (torch.randn(n, width) * (1 + 4 * i)).to(getattr(torch, kind))
        y64 = y.double().sum(0) if kind == "slabs" else y.double()
        gain = 1 + 0.3 * torch.randn(width) if gains else None
        factor = (0.6, -1.4)[i]
        want = want + factor * (plain.unit_rms(y64, eps) * gain.double() if gains else y64)
        terms.append(SumTerm(y.cuda(), factor, gain.cuda() if gains else None, eps))
    if norm:
        want = plain.layer_norm(want, w.double(), b.double(), eps)
    tol = 2e-5 * want.abs().max().item()
    for copy in (None, torch.bfloat16, torch.float32):
        hd = h.cuda()
        got = sum_norm_(hd, alpha, terms, w.cuda() if norm else None, b.cuda() if norm else None, eps, copy)
        assert torch.allclose(hd.double().cpu(), want, atol=tol)
        assert got is None if copy is None else torch.equal(got, hd.to(copy))


@pytest.mark.parametrize("width", [6, 300, 3584, 9001, 20000])
def test_sum_and_norm_of_many_rows(width):
    """Narrow blocks from some hundred rows on: the same rows as among few."""
    from qwen25vl_lite_amd.ops.sum_norm import sum_norm_
    from qwen25vl_lite_amd.parts import SumTerm
    torch.manual_seed(width)
    n = 600
    h, y, z = torch.randn(n, width), torch.randn(n, width).to(torch.bfloat16), torch.randn(n, width)
    w, b, gain = 1 + 0.3 * torch.randn(width), torch.randn(width), 1 + 0.3 * torch.randn(width)
    want = plain.layer_norm(0.9 * h.double() + 0.5 * plain.unit_rms(y.double(), 1e-5) * gain.double() - 2.0 * z.double(),
                            w.double(), b.double(), 1e-5)
    for rows in (slice(0, n), slice(0, 4)):
        hd = h[rows].contiguous().cuda()
        terms = [SumTerm(y[rows].contiguous().cuda(), 0.5, gain.cuda(), 1e-5), SumTerm(z[rows].contiguous().cuda(), -2.0)]
        copy = sum_norm_(hd, 0.9, terms, w.cuda(), b.cuda(), 1e-5, torch.bfloat16)
        assert torch.allclose(hd.double().cpu(), want[rows], atol=3e-5) and torch.equal(copy, hd.to(torch.bfloat16))


@pytest.mark.parametrize("width", [7, 72, 1100, 4400])
def test_layer_norm_with_a_bias_on_chosen_rows(width):
    from qwen25vl_lite_amd.ops.rownorm import layer_norm
    torch.manual_seed(width)
    x, w, b = torch.randn(9, width) + 2.0, 1 + 0.3 * torch.randn(width), torch.randn(width)
    want = plain.layer_norm(x.double(), w.double(), b.double(), 1e-5)
    rows = [7, 0, 3]
    got = layer_norm(x.cuda(), w.cuda(), 1e-5, torch.float32, rows=_i32(rows), bias=b.cuda())
    assert torch.allclose(got.double().cpu(), want[rows], atol=2e-5)
    assert torch.allclose(layer_norm(x.cuda(), w.cuda(), 1e-5, torch.float32, bias=b.cuda()).double().cpu(), want, atol=2e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("c, parts, stride", [(40, 4, 40), (96, 1, 200), (27, 3, 31), (2048, 2, 2048), (6000, 1, 6001)])
def test_a_gate_before_the_norm(c, parts, stride, dtype):
    from qwen25vl_lite_amd.ops.gated import group_norm_gate
    torch.manual_seed(c)
    x, w = torch.randn(7, c), 1 + 0.3 * torch.randn(c)
    gate = torch.randn(7, stride).to(dtype)
    z = gate[:, :c].double()
    want = plain.norm_in_parts(x.double() * plain.silu(z), parts, 1e-5) * w.double()
    got = group_norm_gate(x.cuda(), w.cuda(), c // parts, 1e-5, dtype, gate=gate.cuda()[:, :c], gate_act="silu", gate_first=True)
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    assert torch.allclose(got.double().cpu(), want, atol=tol, rtol=tol)
    behind = plain.norm_in_parts(x.double(), parts, 1e-5) * w.double() * plain.silu(z)
    assert not torch.allclose(behind, want, atol=0.1)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows, c, first", [(1, 1, 0), (5, 6, 12), (70, 16, 48), (3, 256, 0)])
def test_rows_of_the_second_table_gated(rows, c, first, dtype):
    from qwen25vl_lite_amd.ops.sum_norm import gelu_rows
    torch.manual_seed(rows + c)
    table, z = torch.randn(31, first + c + 5).to(dtype), 3 * torch.randn(rows, c)
    ids = torch.tensor(random_tokens(rows, 31, c))
    want = plain.gelu_tanh(z.double()) * table[ids, first:first + c].double()
    tol = 2e-5 if dtype == torch.float32 else 3e-2
    got = gelu_rows(z.cuda(), table.cuda(), first, ids.int().cuda())
    assert got.dtype == dtype and torch.allclose(got.double().cpu(), want, atol=tol, rtol=tol)


@pytest.mark.parametrize("dtype, rows, width, ff", [(torch.float32, 70, 56, 27), (torch.float32, 3, 56, 88), (torch.bfloat16, 1, 64, 88),
                                                   (torch.bfloat16, 9, 3584, 200), (torch.bfloat16, 20, 64, 43), (torch.bfloat16, 5, 50, 24),
                                                   (torch.bfloat16, 70, 64, 88), (torch.bfloat16, 33, 56, 27)])
def test_squared_relu_in_and_behind_the_product(dtype, rows, width, ff):
    from qwen25vl_lite_amd.ops.linear import linear_relu2
    torch.manual_seed(rows + ff)
    x, w = torch.randn(rows, width).to(dtype), (torch.randn(ff, width) / width ** 0.5).to(dtype)
    want = torch.clamp(x.double() @ w.double().T, min=0.0) ** 2
    got = linear_relu2(x.cuda(), w.cuda()).double().cpu()
    tol = 2e-5 if dtype == torch.float32 else 3e-2
    assert torch.allclose(got, want, atol=tol, rtol=tol) and (got == 0).any()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh, hd", [(3, 16), (5, 7), (28, 128)])
def test_a_gate_per_head(nh, hd, dtype):
    from qwen25vl_lite_amd.ops.gated import head_gate_
    torch.manual_seed(nh)
    o, gate = torch.randn(9, nh * hd).to(dtype), torch.randn(9, nh + 4)
    want = (o.double().view(9, nh, hd) * torch.sigmoid(gate[:, 1:1 + nh].double())[:, :, None]).view(9, -1)
    got = head_gate_(o.cuda(), gate.cuda()[:, 1:1 + nh], nh)
    tol = 1e-6 if dtype == torch.float32 else 2e-2
    assert torch.allclose(got.double().cpu(), want, atol=tol, rtol=tol)


@pytest.mark.parametrize("window", [None, 37, 90])
@pytest.mark.parametrize("nq, nkv, hd", [(4, 2, 128), (6, 2, 48), (3, 3, 64), (5, 1, 16)])
def test_sinks_and_gates_in_every_kind_of_matrix_core_attention(nq, nkv, hd, window, monkeypatch):
    """Prompt portions with one and two groups of waves and with three column tiles a wave; decoded tokens with the keys
    whole, split among blocks and merged in the launch, and merged by a second one.  Two sinks stand out: one that takes
    most of the weight and one that takes none."""
    from qwen25vl_lite_amd.ops import attention_mfma
    torch.manual_seed(hd + nq)
    n, ps, scale = 210, 16, 0.5 * hd ** -0.5
    pages = (n + ps - 1) // ps
    q, k, v = torch.randn(n, nq, hd), torch.randn(n, nkv, hd), torch.randn(n, nkv, hd)
    k[11] *= 4.0                                  # a far key that some queries pick
    sinks = torch.randn(nq)
    sinks[0], sinks[-1] = 6.0, -30.0
    gate = 2 * torch.randn(n, nq + 3)             # a gate per head, columns of a wider tensor
    q, k, v = (t.to(torch.bfloat16) for t in (q, k, v))
    want = plain.attend(q.double(), k.double(), v.double(), scale, window, sinks.double())
    none = plain.attend(q.double(), k.double(), v.double(), scale, window, None)
    assert (want - none).abs().amax(dim=(1, 2)).min() > 0.02
    table = torch.randperm(pages)
    kc, vc = torch.zeros(pages, nkv, ps, hd, dtype=torch.bfloat16), torch.zeros(pages, nkv, hd, ps, dtype=torch.bfloat16)
    for p in range(n):
        kc[table[p // ps], :, p % ps], vc[table[p // ps], :, :, p % ps] = k[p], v[p]
    kc, vc, table = kc.cuda(), vc.cuda(), table.int().view(1, -1).cuda()

    def run(first, plan, **kw):
        m = n - first
        monkeypatch.setattr(attention_mfma, "plan_splits", lambda *a: plan)
        step = SimpleNamespace(num_reqs=1, cu_q=_i32([0, m]), cu_q_host=[0, m], ctx_len=_i32([n]), ctx_len_host=[n], max_q_len=m,
                               max_ctx_len=n, derived={})
        args = (q[first:].reshape(m, -1).contiguous().cuda(), kc, vc, table, step, nq, window, scale)
        for s, g in ((sinks.cuda(), None), (sinks.cuda(), gate[first:, 1:1 + nq].cuda()), (None, gate[first:, 1:1 + nq].cuda())):
            w = want if s is not None else none
            w = w if g is None else w * torch.sigmoid(gate[:, 1:1 + nq].double())[:, :, None]
            got = attention_mfma.try_attention(*args, sinks=s, gate=g, **kw)
            assert torch.allclose(got.double().cpu().view(m, nq, hd), w[first:], atol=2e-2, rtol=2e-2), (first, plan, kw)

    for first in (0, 130):
        for kw in (dict(force_groups=1, force_wide=False), dict(force_groups=2, force_wide=False), dict(force_groups=1, force_wide=True)):
            run(first, ("tile", 1, 0), **kw)
    for first in (205, 209):
        run(first, ("coop", 1, 0))
        run(first, ("coop", 4, 64))
    monkeypatch.setattr(attention_mfma, "MERGE_COUNTERS", 0)
    run(209, ("coop", 4, 64))


# ---------------------------------------------------------------------------------------------
# a mixer in its layer
# ---------------------------------------------------------------------------------------------
def _one_layer(tmp_path, layers, dtype=torch.float32, seed=0, width=56, tensors_edit=None, name="one", max_live=3, side=4):
    from qwen25vl_lite_amd.config import EngineConfig, load_config
    from qwen25vl_lite_amd.engine import ModelRunner
    from qwen25vl_lite_amd.models import build_model
    from qwen25vl_lite_amd.weights import load_weights
    cfg = vu.config(width, 50, layers if isinstance(layers, list) else [layers], side=side, eps=1e-4)
    tensors = vu.random_tensors(cfg, seed)
    if tensors_edit is not None:
        tensors_edit(tensors)
    d = vu.write_model(str(tmp_path / name), cfg, seed, tensors)
    model = build_model(load_config(d), dtype, "cuda:0")
    load_weights(d, model)
    ecfg = EngineConfig(num_blocks=48, block_size=16, max_num_seqs=max_live, max_num_batched_tokens=512, max_model_len=512,
                        enable_prefix_cache=False, dtype=dtype)
    cfg, t64 = plain.vezidra_read(d, F64)
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
    out = call(x.to(runner.dtype).cuda(), step, runner.slots[0])
    for rid, n, start in runs:
        runner.cache.commit(rid, start + n)
    return (out.sum(0) if out.dim() == 3 else out).double().cpu()


ALONE = {"attention": vu.heads(6, 2, 24, 16, 80.0, 16, 0.7, window=37), "attention_one_token": vu.heads(2, 1, 8, 8, 20.0, scale=0.6, window=1),
         "attention_matrix_cores": vu.heads(4, 2, 32, 32, 200.0, 20, 0.4, window=50), "attention_all_keys": vu.heads(3, 1, 16, 24, 50.0, 0, 0.6)}
LEFT = {"left": vu.heads(6, 2, 24, 16, 80.0, 16, 0.5, vu.waves()), "left_matrix_cores": vu.heads(4, 1, 32, 32, 80.0, 32, 0.3, vu.waves()),
        "left_odd": vu.heads(3, 1, 7, 5, 80.0, 4, 0.5)}
LEFT_2 = {"left_2": vu.heads(6, 2, 24, 16, 80.0, 16, 0.5, vu.ramp()), "left_2_matrix_cores": vu.heads(4, 4, 48, 48, 80.0, 48, 0.2, vu.ramp()),
          "left_2_odd": vu.heads(3, 3, 9, 5, 80.0, 6, 0.5, vu.ramp())}
DELTA = {"delta": vu.delta(4, 2, 12, 20, 3), "delta_one": vu.delta(1, 1, 1, 1, 1), "delta_wide": vu.delta(2, 1, 64, 80, 4),
         "delta_odd": vu.delta(3, 3, 37, 5, 5)}
DUAL = {"dual": vu.dual(6, 8, 24, 3, 4, 4), "dual_one": vu.dual(1, 1, 1, 1, 1, 1), "dual_wide": vu.dual(4, 40, 64, 1, 2, 3),
        "dual_odd": vu.dual(3, 9, 37, 1, 3, 5)}


def _mixer_case(case, tmp_path, dtype):
    """``(runner, call, plain function of x)`` of a mixer by itself."""
    def build(mixer, pick, fn):
        runner, model, cfg, t = _one_layer(tmp_path, vu.layer(mixer), dtype)
        def call(x, step, slot):
            part, s = model.blocks[0].mixer, slot.of("mix")
            return part.forward(x, step, s) if pick is None else getattr(part, pick).forward(x, step, s.of(pick))
        return runner, call, lambda x, store: fn(store(x), torch.arange(x.shape[0]), t, store)
    if case in ALONE:
        return build(vu.attention(ALONE[case]), None,
                     lambda x, pos, t, store: plain.attention(x, pos, t, "l0.mix.", ALONE[case], 1e-4, store))
    if case in LEFT:
        return build(vu.parallel(LEFT[case], DELTA["delta"]), "left",
                     lambda x, pos, t, store: plain.left_with_sink(x, pos, t, "l0.mix.left.", LEFT[case], 1e-4, store))
    if case in LEFT_2:
        return build(vu.parallel_2(LEFT_2[case], DUAL["dual"]), "left",
                     lambda x, pos, t, store: plain.left_plus_one(x, pos, t, "l0.mix.left.", LEFT_2[case], 1e-4, store))
    if case in DELTA:
        return build(vu.parallel(LEFT["left"], DELTA[case]), "right",
                     lambda x, pos, t, store: plain.gated_delta(x, t, "l0.mix.right.", DELTA[case], 1e-4, store))
    return build(vu.parallel_2(LEFT_2["left_2"], DUAL[case]), "right",
                 lambda x, pos, t, store: plain.state_space_dual(x, t, "l0.mix.right.", DUAL[case], 1e-4, store))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case", sorted({**ALONE, **LEFT, **LEFT_2, **DELTA, **DUAL}))
def test_a_mixer_alone_whole_in_two_steps_and_token_by_token(case, dtype, tmp_path):
    """The mixer's own forward against the plain function: one run of 150 tokens (recurrences in chunks), the same cut
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
    first = _run_mixer(runner, call, [("b", 21, 0)], x[:21])
    second = _run_mixer(runner, call, [("b", n - 21, 21)], x[21:])
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
@pytest.mark.parametrize("shape", [(24, 16), (32, 32)])
def test_one_key_just_inside_and_just_outside_a_window(shape, dtype, tmp_path):
    """One token's key stands out by far: the ``window`` tokens from it on read its value, the next does not.  The last
    of them are decoded one by one."""
    d, dv = shape
    window, loud = 21, 13
    m = vu.heads(2, 1, d, dv, 50.0, 0, 1.0, window=window)

    def edit(t):
        # every query is one direction; a key has it where the input's second channel says so
        t["l0.mix.sink"] = torch.full((2,), -40.0).to(torch.bfloat16)
        t["l0.mix.q"].zero_()
        t["l0.mix.q"][::d, 0] = 1.0
        t["l0.mix.k"][:, :2] = 0.0
        t["l0.mix.k"][::d, 1] = 20.0
    runner, model, cfg, t = _one_layer(tmp_path, vu.layer(vu.attention(m)), dtype, tensors_edit=edit)
    torch.manual_seed(3)
    n = 60
    x = torch.randn(n, 56)
    x[:, 0], x[:, 1] = 1.0, 0.0
    x[loud, 1] = 1.0
    mixer = model.blocks[0].mixer
    store = plain._keep if dtype == torch.float32 else plain.to_bfloat16_and_back
    call = lambda x, step, slot: mixer.forward(x, step, slot.of("mix"))
    want = plain.attention(store(x.double()), torch.arange(n), t, "l0.mix.", m, 1e-4, store)
    got = torch.cat([_run_mixer(runner, call, [("a", 20, 0)], x[:20])]
                    + [_run_mixer(runner, call, [("a", 1, p)], x[p:p + 1]) for p in range(20, n)])
    tol = (2e-5 if dtype == torch.float32 else 4e-2) * want.abs().max().item()
    assert torch.allclose(got, want, atol=tol)
    # a window one token shorter or longer moves the row at its edge
    for other in (window - 1, window + 1):
        off = plain.attention(store(x.double()), torch.arange(n), t, "l0.mix.", {**m, "mask": {"size": other}}, 1e-4, store)
        edge = loud + min(window, other)
        assert (off - want).abs().amax(dim=1)[edge] > 8 * tol, other


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_layer_that_reads_another_layers_cache_with_a_longer_window(dtype, tmp_path):
    """The reader sees 40 keys of a cache whose own layer sees 9: its pages stay for the reader."""
    from qwen25vl_lite_amd.engine import StepEntry
    layers = [vu.layer(vu.attention(vu.heads(4, 2, 32, 32, 50.0, 16, 0.5, window=9)), 24),
              vu.layer(vu.attention(vu.heads(4, 2, 32, 32, 50.0, 16, 0.6, window=40, kv_from=0)))]
    runner, model, cfg, t = _one_layer(tmp_path, layers, dtype)
    assert [g.need.window for g in runner.cache.groups] == [40] and "l1.mix.k" not in t
    toks = random_tokens(120, 50, 2)
    want = plain.vezidra_forward(cfg, t, toks).float()
    rounding = _rel_rows(plain.vezidra_forward(cfg, t, toks, plain.to_bfloat16_and_back).float(), want)
    runner.admit("a")
    rows = [runner.execute([StepEntry("a", toks[:70], 0, want=list(range(70)))]).cpu()]
    for p in range(70, 120):
        rows.append(runner.execute([StepEntry("a", [toks[p]], p, want=[0])]).cpu())
    errors = _rel_rows(torch.cat(rows), want)
    assert errors.max() < 2e-5 if dtype == torch.float32 else _like_rounding(errors, rounding)
    held = [i for i, p in enumerate(runner.cache.table("a", 0)) if p >= 0]
    assert held == [5, 6, 7]                        # token 120 sees keys from 81 on


def test_the_residual_after_every_layer(tmp_path):
    """What the stream holds behind each layer of a whole step equals the plain model's, side input included; leaving the
    side input out would show."""
    from qwen25vl_lite_amd.engine import StepEntry
    layers = [vu.layer(vu.parallel(LEFT["left"], DELTA["delta"]), 40), vu.layer(vu.attention(ALONE["attention"])),
              vu.layer(vu.parallel_2(LEFT_2["left_2"], DUAL["dual"]), 24)]
    runner, model, cfg, t = _one_layer(tmp_path, layers)
    toks, seen = random_tokens(47, 50, 2), []
    for block in model.blocks:
        def spy(stream, step, slot, inner=block.forward):
            out = inner(stream, step, slot)
            seen.append(out.h.double().cpu())
            return out
        block.forward = spy
    runner.admit("a")
    runner.execute([StepEntry("a", toks, 0, want=[46])])
    trace = []
    plain.vezidra_forward(cfg, t, toks, trace=trace)
    for got, want in zip(seen, trace):
        assert torch.allclose(got, want, atol=2e-5 * want.abs().max().item())
    without = []
    plain.vezidra_forward({**cfg, "token_side": None}, t, toks, trace=without)
    assert (without[0] - trace[0]).abs().max() > 0.1 * trace[0].abs().max()


# ---------------------------------------------------------------------------------------------
# whole models, every schedule
# ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name", ["mixed", "ones", "odd", "wide"])
def test_float32_every_schedule_against_the_plain_model(name, folders):
    """Whole prompts, decoding, portions down to two tokens, mixed batches with more requests than slots: all the
    same logits, and the plain model's."""
    folder = folders[name]
    cfg, _ = plain.vezidra_read(folder, F64)
    reqs = _requests(cfg["vocab"], seed=20)
    want = {rid: _oracle(folder, toks) for rid, toks in reqs.items()}
    mixed, peak = mixed_trace(reqs, seed=4, max_live=4)
    # a root mean square over one value is a sign: with heads of one channel float32 arithmetic itself is visible, and the
    # measure is the plain model run in float32
    rounding = None
    if name == "ones":
        cfg, t32 = plain.vezidra_read(folder, torch.float32)
        rounding = torch.cat([_rel_rows(plain.vezidra_forward(cfg, t32, toks), want[rid]) for rid, toks in reqs.items()])
    holders = {}
    for steps, size in ((whole_trace(reqs), 192), (tail_trace(reqs, 50), 192), (portion_trace(reqs), 192), (mixed, peak)):
        got = run_steps(_replayer(folder, "float32", size), steps, holders if steps is mixed else None)
        errors = torch.cat([_rel_rows(_rows(got, rid, len(toks)), want[rid]) for rid, toks in reqs.items()])
        if rounding is None:
            assert errors.max() < 2e-5, (name, errors.max())
        else:
            assert _like_rounding(errors, rounding, 1e-6), (errors.median(), rounding.median(), errors.quantile(0.9), rounding.quantile(0.9))
            assert errors.max() < 4 * rounding.max() + 1e-5, (errors.max(), rounding.max())
    assert any(len(who) > 1 for who in holders.values()), "no page was used by two requests"


@pytest.mark.parametrize("name", ["mixed", "ones", "odd", "wide"])
def test_bfloat16_within_rounding_of_the_plain_model(name, folders):
    """bfloat16 kernels: no further from exact arithmetic than rounding the stored activations to bfloat16 takes the
    plain model, whatever the schedule."""
    folder = folders[name]
    cfg, _ = plain.vezidra_read(folder, F64)
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
def test_peaked_attention_at_window_edges_and_far_keys(dtype, folders):
    """Score scales so large that the softmax picks single keys, across page borders, hundreds of tokens back and at the
    windows' edges.  The last 70 tokens are decoded, so every window passes over decoded tokens; then the same in
    portions."""
    folder = folders["sharp"]
    toks = random_tokens(330, vu.SHARP["vocab"], 40)
    want = _oracle(folder, toks)
    if dtype == "float32":
        # scores this large make float32 arithmetic itself visible: the measure is the plain model run in float32
        cfg, t32 = plain.vezidra_read(folder, torch.float32)
        rounding, slack = _rel_rows(plain.vezidra_forward(cfg, t32, toks), want), 1e-5
    else:
        rounding, slack = _rel_rows(_oracle(folder, toks, plain.to_bfloat16_and_back), want), 1e-3
    for steps in (tail_trace({"s": toks}, 70), portion_trace({"s": toks}, (64, 3, 41, 2, 17, 90))):
        got = _rows(run_steps(_replayer(folder, dtype, round64(len(toks))), steps), "s", len(toks))
        errors = _rel_rows(got, want)
        assert _like_rounding(errors, rounding, slack), (errors.median(), rounding.median(), errors.quantile(0.9),
                                                         rounding.quantile(0.9))
        assert errors.max() < 4 * rounding.max() + slack, (errors.max(), rounding.max())


def test_what_the_schedules_would_show(folders):
    """Each of these changes the plain model's last logits well beyond the tolerances above: windows one token longer,
    a reader given its own window only, sinks left out, gates left out, betas of one, decays of one, a scale of the sum,
    rotation in the other layout, unstretched frequencies, the far past replaced."""
    toks = random_tokens(330, vu.SHARP["vocab"], 40)
    folder = folders["sharp"]
    whole = _oracle(folder, toks)

    def windows(cfg):
        for lay in cfg["layers"]:
            if lay["mixer"].get("mask"):
                lay["mixer"]["mask"]["size"] += 1

    def reader(cfg):
        cfg["layers"][3]["mixer"]["mask"]["size"] = 21

    def scaling(cfg):
        for lay in cfg["layers"]:
            m = lay["mixer"].get("left", lay["mixer"])
            m["rot"].pop("scaling", None)

    def swap(cfg):
        for lay in cfg["layers"]:
            if lay["type"] == "parallel":
                m = lay["mixer"]
                m["left_scale"], m["right_scale"] = m["right_scale"], m["left_scale"]

    def to(ending, value):
        def edit(t):
            for name in t:
                if name.endswith(ending):
                    t[name] = torch.full_like(t[name], value)
        return edit

    for kw in ({"cfg_edit": windows}, {"cfg_edit": reader}, {"cfg_edit": scaling}, {"cfg_edit": swap},
               {"cfg_edit": lambda c: c.__setitem__("postln_alpha", 2.2)}, {"tensors_edit": to(".sink", -40.0)},
               {"tensors_edit": to("mix.g", 0.0)}, {"tensors_edit": to("right.A_log", -20.0)}, {"tensors_edit": to(".dt_bias", 0.0)},
               {"tensors_edit": to("right.b", 0.0)}, {"tensors_edit": to("right.D", 0.0)}, {"tensors_edit": to("norm1.b", 0.0)}):
        assert _rel(_oracle(folder, toks, **kw)[-30:], whole[-30:]) > 0.02, kw
    turned, attend = plain.rotate, plain.attend
    try:
        plain.rotate = lambda x, pos, f, near, amp=1.0: turned(x, pos, f, not near, amp)
        assert _rel(_oracle(folder, toks)[-30:], whole[-30:]) > 0.02
        plain.rotate = turned
        plain.attend = lambda q, k, v, s, w, sink: attend(q, k, v, s, w, None if (sink == 0).all() else sink)
        assert _rel(_oracle(folder, toks), whole) > 0.02               # the one in the denominator
    finally:
        plain.rotate, plain.attend = turned, attend
    other = random_tokens(290, vu.SHARP["vocab"], 41) + toks[290:]
    assert _rel(_oracle(folder, other)[-30:], whole[-30:]) > 0.02


def test_long_decoding(folders):
    """A short prompt and 200 tokens decoded one by one, through several pages and windows."""
    folder = folders["mixed"]
    toks = random_tokens(205, vu.MIXED["vocab"], 50)
    want = _oracle(folder, toks)
    got = _rows(run_steps(_replayer(folder, "float32", 256), tail_trace({"l": toks}, 200)), "l", len(toks))
    assert _rel(got, want) < 2e-5


def test_a_fork_continues_from_the_same_states(folders):
    """Pages, recurrent states and the convolutions' last rows all go to the fork."""
    from qwen25vl_lite_amd.engine import StepEntry
    rp = _replayer(folders["mixed"], "float32", 256)
    toks = random_tokens(60, vu.MIXED["vocab"], 55)
    want = _oracle(folders["mixed"], toks)
    runner = rp.runner
    runner.admit("a")
    runner.execute([StepEntry("a", toks[:41], 0)])
    runner.fork("a", "b")
    runner.execute([StepEntry("a", [1, 2, 3], 41)])            # the original goes elsewhere
    got = runner.execute([StepEntry("b", toks[41:], 41, want=list(range(19)))]).cpu()
    assert _rel(got, want[41:]) < 2e-5


def _greedy(folder, prompts, steps):
    want = []
    for p in prompts:
        ids = list(p)
        for _ in range(steps):
            ids.append(int(torch.argmax(_oracle(folder, ids)[-1])))
        want.append(ids[len(p):])
    return want


@pytest.mark.parametrize("name", ["mixed", "odd"])
@pytest.mark.parametrize("graph", [False, True])
def test_greedy_generation_through_the_entry_point(graph, name, folders):
    """``LLM.generate`` with the scheduler (three prompts, two slots, portions of 16 tokens, decode steps from HIP
    graphs or not) picks the plain model's tokens."""
    from qwen25vl_lite_amd import LLM, SamplingParams
    folder, vocab, steps = folders[name], CONFIGS[name][0]["vocab"], 12
    prompts = [random_tokens(n, vocab, 70 + n) for n in (37, 5, 21)]
    want = _greedy(folder, prompts, steps)
    with LLM(folder, dtype="float32", num_blocks=32, block_size=16, max_num_seqs=2, max_num_batched_tokens=16,
             hip_graph=graph) as llm:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True))
    assert [o.output_token_ids for o in outs] == want


def test_preempted_requests_start_again_from_cleared_states(folders):
    """Pages for one and a half requests: one gives way, is computed again from its first token, and both still pick
    the plain model's tokens."""
    from qwen25vl_lite_amd import LLM, SamplingParams
    folder, steps = folders["mixed"], 24
    prompts = [random_tokens(n, vu.MIXED["vocab"], 170 + n) for n in (30, 27)]
    want = _greedy(folder, prompts, steps)
    with LLM(folder, dtype="float32", num_blocks=5, block_size=16, max_num_seqs=2, max_num_batched_tokens=32) as llm:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True))
    assert [o.output_token_ids for o in outs] == want


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_replay_program_and_the_command_line(dtype, folders, tmp_path):
    """``bin/trace_run`` as a user calls it on a Vezidra folder (steps on standard input, ``done`` lines, files of
    float32 logits), and ``generate`` of the command line, whose tokens are the plain model's."""
    import ast
    import json
    import os
    import subprocess
    import sys

    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder, vocab = folders["mixed"], vu.MIXED["vocab"]
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
    rounding = _rel_rows(_oracle(folder, toks, plain.to_bfloat16_and_back), want)[[0, 18, 44, 2]]
    limit = torch.full((4,), 2e-5) if dtype == "float32" else 3 * rounding + 4e-3
    assert (_rel_rows(torch.cat([s0, s2]), want[[0, 18, 44, 2]]) < limit).all()
    if dtype == "float32":
        prompt = toks[:12]
        cli = [sys.executable, os.path.join(root, "bin", "qwen25vl-lite"), "generate", "--model", folder, "--dtype", "float32",
               "--num-blocks", "32", "--max-num-seqs", "2", "--max-model-len", "256", "--max-tokens", "6", "--ignore-eos",
               "--prompt-token-ids", ",".join(map(str, prompt))]
        proc = subprocess.run(cli, capture_output=True, text=True, timeout=110)
        assert proc.returncode == 0, proc.stderr[-2000:]
        assert ast.literal_eval(proc.stdout.strip().splitlines()[-1]) == _greedy(folder, [prompt], 6)[0]


def test_bfloat16_generation_from_graphs_matches_eager_steps(folders):
    from qwen25vl_lite_amd import LLM, SamplingParams
    prompts = [random_tokens(n, vu.MIXED["vocab"], 90 + n) for n in (18, 3, 40, 9)]
    outs = []
    for graph in (False, True):
        with LLM(folders["mixed"], dtype="bfloat16", num_blocks=48, block_size=16, max_num_seqs=4,
                 max_num_batched_tokens=64, hip_graph=graph) as llm:
            outs.append([o.output_token_ids for o in
                         llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True))])
    assert outs[0] == outs[1]
