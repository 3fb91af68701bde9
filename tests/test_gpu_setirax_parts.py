"""Each mechanism of Setirax alone, the engine's kernels against the plain functions: convolution, rotation, unit norm and
cache write (alone and beside the linear side's step); softmax attention with capped scores under a window; attention over a
latent under a window and with a sink, in each of its kernels; gated linear attention (chunks, single tokens, states carried,
slots used again, padding); the real-gated linear recurrent unit; the squared-ReLU feed-forward in every product kernel; the
post-norm block's kernels; two mixers summed in one product."""
import math

import numpy as np
import pytest
import torch

from plain import setirax_plain as plain

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


def ops_for(dtype):
    from minivllm_amd.kernels.ops import Ops
    return Ops(dtype)


def i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def step_ints(q_lens, slots, pad_rows=0, pad_seqs=0):
    seq = [s for s, n in enumerate(q_lens) for _ in range(n)] + [-1] * pad_rows
    cu = np.concatenate([[0], np.cumsum(q_lens)]).tolist()
    cu += [cu[-1]] * pad_seqs
    return i32(seq), i32(cu), i32(list(slots) + [0] * pad_seqs)


def close(got, want, tol, what=""):
    got, want = got.double().cpu(), want.double().cpu()
    assert torch.isfinite(got).all(), what
    err = float((got - want).abs().max() / want.abs().max().clamp_min(1e-30))
    assert err <= tol, f"{what}: relative error {err:.3e} exceeds {tol:.1e}"


def runtime(dtype, max_positions=4096):
    from minivllm_amd.parts.base import Runtime, Workspace
    return Runtime(device=torch.device(DEV), dtype=dtype, ops=ops_for(dtype), workspace=Workspace(torch.device(DEV)),
                   max_positions=max_positions)


def context(q_lens, slots, states, pad_rows=0, pad_seqs=0, starts=None, kv=None, page=16):
    """A step on its own: ``states`` by name; ``kv`` = (k pages, v pages, block table rows of the requests)."""
    from minivllm_amd.engine.step import AttentionPlan, KVView, StepContext
    from minivllm_amd.parts.base import Workspace
    ctx = StepContext()
    ctx.token_seq, ctx.cu_seqlens, ctx.state_slots = step_ints(q_lens, slots, pad_rows, pad_seqs)
    ctx.n_tokens, ctx.n_seqs = sum(q_lens) + pad_rows, len(q_lens) + pad_seqs
    starts = starts or [0] * len(q_lens)
    ctx.positions = i32([s + t for s, n in zip(starts, q_lens) for t in range(n)] + [0] * pad_rows)
    ctx._state = {0: states}
    if kv is not None:
        ctx._kv[0] = KVView(kv[0], kv[2], page)
    ctx.attention_plan = AttentionPlan(decode_only=all(n == 1 for n in q_lens) and not pad_rows, max_q_len=max(q_lens),
                                       max_context_len=max(s + n for s, n in zip(starts, q_lens)), n_seqs=ctx.n_seqs, q_lens=q_lens,
                                       cu_seqlens=ctx.cu_seqlens, workspace=Workspace(torch.device(DEV)))
    return ctx


# ---------------------------------------------------------------------------------------
# convolution, rotation, unit norm, cache write
# ---------------------------------------------------------------------------------------
CONV_SIZES = [(4, 2, 16, 24, 3, 8), (3, 1, 10, 6, 1, 6), (6, 3, 64, 64, 4, 64), (2, 1, 128, 128, 4, 32), (5, 5, 64, 64, 2, 0), (1, 1, 256, 256, 6, 256),
              (2, 2, 64, 40, 4, 16), (16, 8, 128, 128, 4, 128), (1, 1, 12, 300, 5, 2)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, G, D, Dv, taps, rot", CONV_SIZES)
@pytest.mark.parametrize("q_lens, beside", [([9, 1, 2, 3], False), ([70, 2, 33, 1], False), ([1, 1, 1, 1], False), ([1, 1, 1, 1], True)])
def test_convolution_rotation_and_store(dtype, H, G, D, Dv, taps, rot, q_lens, beside):
    """Requests in the middle of their sequences, on slots out of order, with kept inputs that are not zero; a padding row;
    scattered pages; portions shorter than the filter; single tokens alone and in the launch of the linear side's step."""
    from minivllm_amd.parts.rope import RotaryEmbedding, RotarySpec
    rt = runtime(dtype)
    ops, page, eps = rt.ops, 16, 1e-5
    g = torch.Generator().manual_seed(H * 100 + D + taps)
    q_dim, k_dim, v_dim = H * D, G * D, G * Dv
    C = q_dim + k_dim + v_dim
    n, S = sum(q_lens), len(q_lens)
    single = max(q_lens) == 1
    R, rd, rv, rank = 2, 8, 8, 3                                # the linear side, for `beside`
    base = 0
    right = C + (-C) % 8
    width = right + 2 * R * (rd + rv) + 32
    rows = torch.randn(n + 1, width, generator=g).to(dtype)
    taps_w = 0.7 * torch.randn(C, taps, generator=g)
    hist = torch.randn(S + 1, taps - 1, C, generator=g).to(dtype)
    slots, starts = [2, 4, 0, 3][:S], [13, 0, 30, 15][:S]
    scaling = (4.0, 1.0, 3.0, 40.0)
    table = None
    if rot:
        emb = RotaryEmbedding(RotarySpec(rotary_dim=rot, theta=300.0, by_wavelength=scaling), {}, rt)
        table = emb.table
    bt_width = (max(s + m for s, m in zip(starts, q_lens)) - 1) // page + 1
    perm = torch.randperm(S * bt_width + 3, generator=g)[:S * bt_width].view(S, bt_width)
    k_pages = torch.full((S * bt_width + 3, G, page, D), float("nan"), dtype=dtype, device=DEV)
    v_pages = torch.full((S * bt_width + 3, G, Dv, page), float("nan"), dtype=dtype, device=DEV)
    pad = 1
    tsq, cu, ss = step_ints(q_lens, slots, pad_rows=pad)
    pos = [s + t for s, m in zip(starts, q_lens) for t in range(m)]
    conv_state = hist.clone().to(DEV) if taps > 1 else None
    out = torch.full((n + pad, q_dim + v_dim), float("nan"), dtype=dtype, device=DEV)
    dev = rows.to(DEV)
    args = dict(rows=dev, base=base, num_heads=H, num_kv_heads=G, head_dim=D, value_dim=Dv, taps_t=taps_w.t().contiguous().to(DEV),
                conv_state=conv_state, positions=i32(pos + [0]), cu_seqlens=cu, state_slots=ss, n_seqs=S, rope_table=table, unit_norm=True,
                eps=eps, k_pages=k_pages, v_pages=v_pages, block_table=perm.to(torch.int32).contiguous().to(DEV), page_size=page, out=out)
    if beside:
        state = torch.zeros(S + 1, R, rv, rd, device=DEV)
        y = torch.empty(n + pad, R * rv, dtype=dtype, device=DEV)
        ran = ops.gated_linear_step(dev, right, right + 2 * R * (rd + rv), R, rd, rv, torch.randn(rank, R * rd, generator=g).to(DEV),
                                    torch.zeros(R * rd, device=DEV), 4.0, torch.ones(rv, device=DEV), eps, state, tsq, ss, y, beside=args)
        fits = D == Dv and D in (64, 128, 256) and rot % 16 == 0
        assert ran == (2 if fits else 1), ran
        if ran == 1:
            return                                  # (the store then runs in a launch of its own, as in the case above)
    else:
        ops.qkv_conv_store(tsq, single=single, **args)
    torch.cuda.synchronize()
    tol = 3e-6 if dtype == torch.float32 else 8e-3
    m = {"dims": rot, "base": 300.0, "scaling": dict(zip(("factor", "low", "high", "original"), scaling))}
    written, at = 0, 0
    for s, (count, slot, start) in enumerate(zip(q_lens, slots, starts)):
        x = rows[at:at + count, :C].double()
        y, kept = plain.short_conv(x, taps_w.double(), hist[slot].double())
        q, k, v = y[:, :q_dim].view(count, H, D), y[:, q_dim:q_dim + k_dim].view(count, G, D), y[:, q_dim + k_dim:].view(count, G, Dv)
        if rot:
            q, k = plain.rotate(q, start, m), plain.rotate(k, start, m)
        close(out[at:at + count, :q_dim].view(count, H, D), plain.unit_rms(q, eps), tol, f"queries of {s}")
        where = [(int(perm[s, p // page]), p % page) for p in range(start, start + count)]
        close(torch.stack([k_pages[a, :, b] for a, b in where]), plain.unit_rms(k, eps), tol, f"keys of {s}")
        close(torch.stack([v_pages[a, :, :, b] for a, b in where]), v, tol, f"values of {s}")
        if taps > 1:
            assert torch.equal(conv_state[slot].double().cpu(), kept), f"kept inputs of {s}"
        written, at = written + count, at + count
    assert int(torch.isfinite(k_pages.float()).sum()) == written * k_dim and int(torch.isfinite(v_pages.float()).sum()) == written * v_dim
    assert torch.equal(dev.cpu(), rows), "the rows were written"
    if taps > 1:
        untouched = sorted(set(range(S + 1)) - set(slots))
        assert torch.equal(conv_state[untouched].cpu(), hist[untouched]), "a slot of nobody was touched"


# ---------------------------------------------------------------------------------------
# softmax attention with capped scores under a window
# ---------------------------------------------------------------------------------------
class Capped:
    """One request's keys and values on scattered pages (pages that the window has let go of, and slots that nobody has
    written yet, hold NaN) and the plain answer. ``far``: (key, query) positions; queries from there on single the key out."""

    def __init__(self, H, G, D, Dv, n, page, dtype, seed, cap, size, far):
        self.H, self.G, self.D, self.Dv, self.n, self.page, self.dtype, self.cap, self.size = H, G, D, Dv, n, page, dtype, cap, size
        g = torch.Generator().manual_seed(seed)
        q, k, v = torch.randn(n, H, D, generator=g), torch.randn(n, G, D, generator=g), torch.randn(n, G, Dv, generator=g)
        mark = torch.randn(D, generator=g)
        mark = mark / mark.norm() * D ** 0.5
        for p in far:
            k[p] = 2.2 * mark
        q = 0.3 * q + 2.0 * mark
        self.q, self.k, self.v = q.to(dtype), k.to(dtype), v.to(dtype)
        self.scale = 1.2 / D ** 0.5
        self.table = torch.randperm(-(-n // page) + 4, generator=g)[:-(-n // page)].tolist()

    def want(self, first, count):
        out = torch.empty(count, self.H, self.Dv, dtype=torch.float64)
        for h in range(self.H):
            kv = h // (self.H // self.G)
            s = (self.q[first:first + count, h].double() @ self.k[:first + count, kv].double().T) * self.scale
            out[:, h] = plain.sink_softmax(plain.windowed(plain.capped(s, self.cap), first, self.size), None) @ self.v[:first + count, kv].double()
        return out.reshape(count, self.H * self.Dv)

    def run(self, ops, first, count, splits=None, variant=None, plan=True):
        from minivllm_amd.engine.step import AttentionPlan
        from minivllm_amd.parts.base import Workspace
        lowest = 0 if self.size is None else max(0, first - self.size + 1)
        k_pages = torch.full((len(self.table) + 4, self.G, self.page, self.D), float("nan"), dtype=self.dtype)
        v_pages = torch.full((len(self.table) + 4, self.G, self.Dv, self.page), float("nan"), dtype=self.dtype)
        for p in range(lowest // self.page * self.page, first + count):
            k_pages[self.table[p // self.page], :, p % self.page] = self.k[p]
            v_pages[self.table[p // self.page], :, :, p % self.page] = self.v[p]
        bt = [t if b >= lowest // self.page else -1 for b, t in enumerate(self.table)]
        p = AttentionPlan(decode_only=(count == 1), max_q_len=count, max_context_len=first + count, n_seqs=1, q_lens=[count],
                          cu_seqlens=i32([0, count]), workspace=Workspace(torch.device(DEV)), decode_splits=splits, prefill_variant=variant,
                          kv_tokens=first + count)
        out = torch.empty(count, self.H * self.Dv, dtype=self.dtype, device=DEV)
        ops.ledger = []
        ops.attention(self.q[first:first + count].reshape(count, -1).contiguous().to(DEV), out, k_pages.to(DEV), v_pages.to(DEV),
                      i32(bt).view(1, -1), self.page, i32(range(first, first + count)), i32([0] * count), self.H, self.G, self.D, self.scale,
                      None if self.size is None else self.size - 1, plan=p if plan else None, value_dim=self.Dv, softcap=self.cap)
        torch.cuda.synchronize()
        entry, ops.ledger = ops.ledger[0][0], None
        return out, entry


@pytest.mark.parametrize("cap, size", [(9.0, 40), (None, 33), (4.0, None), (20.0, 1), (15.0, 17)])
@pytest.mark.parametrize("H, G, D, Dv, page", [(4, 2, 16, 24, 8), (3, 1, 10, 6, 4), (6, 2, 64, 64, 16), (16, 1, 64, 32, 32)])
def test_capped_attention_float32(H, G, D, Dv, page, cap, size):
    ops = ops_for(torch.float32)
    c = Capped(H, G, D, Dv, 150, page, torch.float32, D, cap, size, far=(17, 64, 101, 120))
    for first, count in ((0, 150), (0, 1), (1, 2), (55, 3), (56, 1), (57, 1), (127, 5), (140, 1), (141, 1)):
        out, entry = c.run(ops, first, count)
        assert entry == "mv_attention_ref"
        close(out, c.want(first, count), 2e-5, f"{count} queries from {first}")


@pytest.mark.parametrize("cap, size", [(9.0, 40), (None, 33), (4.0, None), (20.0, 1), (15.0, 130)])
@pytest.mark.parametrize("variant", [(1, 1), (2, 1), (1, 2), (2, 2)])
@pytest.mark.parametrize("H, G, D, page", [(6, 2, 64, 16), (2, 1, 128, 32), (16, 1, 64, 64), (4, 4, 128, 16)])
def test_capped_attention_prompts(H, G, D, page, variant, cap, size):
    ops = ops_for(torch.bfloat16)
    c = Capped(H, G, D, D, 300, page, torch.bfloat16, H + D, cap, size, far=(15, 64, 101, 170, 226))
    for first, count in ((0, 300), (0, 2), (3, 40), (95, 66), (103, 2), (140, 2), (250, 33)):
        out, entry = c.run(ops, first, count, variant=variant)
        assert entry == "mv_attention_prefill"
        close(out, c.want(first, count), 1.2e-2, f"{count} queries from {first}")


@pytest.mark.parametrize("cap, size", [(9.0, 40), (None, 33), (4.0, None), (20.0, 1), (15.0, 400)])
@pytest.mark.parametrize("splits", [None, 1, 3, 16])
@pytest.mark.parametrize("H, G, D, page", [(6, 2, 64, 16), (2, 1, 128, 32), (16, 1, 64, 64), (4, 4, 128, 16)])
def test_capped_attention_single_tokens(H, G, D, page, splits, cap, size):
    ops = ops_for(torch.bfloat16)
    c = Capped(H, G, D, D, 700, page, torch.bfloat16, H + D + 1, cap, size, far=(0, 20, 100, 270, 512))
    for first in (0, 1, 31, 32, 39, 40, 52, 53, 59, 60, 139, 140, 499, 500, 551, 552, 699):
        out, entry = c.run(ops, first, 1, splits=splits)
        assert entry == "mv_attention_decode"
        close(out, c.want(first, 1), 1.2e-2, f"position {first}")


# ---------------------------------------------------------------------------------------
# attention over a latent
# ---------------------------------------------------------------------------------------
LATENT_SIZES = [(3, 12, 20, 24, 16), (4, 32, 64, 64, 16), (18, 64, 32, 96, 8), (1, 6, 10, 13, 4), (16, 128, 64, 256, 16), (5, 16, 16, 512, 32)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, d, dv, R, page", LATENT_SIZES)
@pytest.mark.parametrize("size", [1, 21, 64, None])
def test_latent_attention_under_a_window(dtype, H, d, dv, R, page, size):
    """The part whole: two requests side by side, prompts in portions (down to two tokens) and single tokens, on scattered
    pages that hold NaN before they are written and again once the window has let go of them."""
    from minivllm_amd.parts.latent_attention import LatentAttention, LatentAttentionSpec
    rt = runtime(dtype)
    hid, eps = 64, 1e-5
    g = torch.Generator().manual_seed(H * 10 + R)
    shapes = {"q": (H * d, hid), "dkv": (R, hid), "dkv.norm": (R,), "uk": (H * d, R), "uv": (H * dv, R), "sink": (H,), "o": (hid, H * dv)}
    w = {k: (torch.randn(s, generator=g) / (s[1] ** 0.5 if len(s) == 2 else 1.0)).to(torch.bfloat16) for k, s in shapes.items()}
    w["dkv.norm"] = (1 + 0.2 * w["dkv.norm"].float()).to(torch.bfloat16)
    w["sink"] = (w["sink"].float() + 2.0).to(torch.bfloat16)
    m = {"heads": H, "dim": d, "vdim": dv, "kv_rank": R, "scale": 2.5 / d ** 0.5, "mask": None if size is None else {"size": size}}
    spec = LatentAttentionSpec(hidden_size=hid, num_heads=H, plain_dim=d, rot_dim=0, value_dim=dv, q_rank=0, kv_rank=R, scale=m["scale"],
                               norm_eps=eps, window=None if size is None else size - 1, sink=True)
    part = LatentAttention(spec, {k.replace(".", "_"): v.to(DEV) for k, v in w.items()}, rt)
    T = 130
    x = torch.randn(2, T, hid, generator=g).to(dtype)
    rnd = plain.keep if dtype == torch.float32 else plain.round_to_bfloat16
    want = [plain.latent_mixer(x[r].double(), {k: v.double() for k, v in w.items()}, "", m, eps, None, rnd)[0] for r in range(2)]
    blocks = -(-T // page)
    perm = torch.randperm(2 * blocks + 2, generator=g)
    pages = torch.full((2 * blocks + 2, page, R), float("nan"), dtype=dtype, device=DEV)
    pages_t = torch.full((2 * blocks + 2, R, page), float("nan"), dtype=dtype, device=DEV)
    done = [0, 0]
    tol = 3e-5 if dtype == torch.float32 else 3e-2
    for lens in ([40, 33], [2, 3], [1, 1], [1, 1], [30, 1], [1, 1], [2, 50], [1, 1], [1, 1], [1, 1], [40, 2], [1, 1], [1, 1]):
        lens = [min(k, T - p) for k, p in zip(lens, done)]
        table = torch.full((2, blocks), -1, dtype=torch.int32)
        for r in range(2):
            low = 0 if size is None else max(0, done[r] - size + 1)
            for b in range(blocks):
                if b >= low // page:
                    table[r, b] = perm[r * blocks + b]
                else:
                    pages[perm[r * blocks + b]] = float("nan")
                    pages_t[perm[r * blocks + b]] = float("nan")
        ctx = context(lens, [0, 1], {}, starts=list(done), kv=({"latent": pages, "latent_t": pages_t}, None, table.to(DEV)), page=page)
        y = part.forward(torch.cat([x[r, p:p + k] for r, (p, k) in enumerate(zip(done, lens))]).to(DEV), ctx, 0)
        y = y if isinstance(y, torch.Tensor) else y.materialize()
        torch.cuda.synchronize()
        close(y, torch.cat([want[r][p:p + k] for r, (p, k) in enumerate(zip(done, lens))]), tol, f"{lens} from {done}")
        done = [p + k for p, k in zip(done, lens)]


@pytest.mark.parametrize("R", [32, 64, 96, 128, 160, 192, 256, 384, 512])
@pytest.mark.parametrize("kernel", ["general", "split", "mfma", "split_mfma"])
@pytest.mark.parametrize("size", [1, 8, 50, 300])
def test_latent_kernels_find_the_first_key_of_a_window(R, kernel, size):
    """A key that the query singles out just inside the window, then just outside; with and without a sink that stands out."""
    from minivllm_amd.engine.step import AttentionPlan
    from minivllm_amd.parts.base import Workspace
    ops, page, H, n = ops_for(torch.bfloat16), 16, 17, 420
    g = torch.Generator().manual_seed(R + size)
    rows = torch.randn(n, R, generator=g)
    mark = torch.randn(R, generator=g)
    at = [400, 401, 407, 408, 415]
    rows = rows.to(torch.bfloat16)
    for pos in at:
        for edge in (pos - size + 1, pos - size):
            if edge < 0:
                continue
            keys = rows.clone()
            keys[edge] = mark.to(torch.bfloat16)
            q = (0.2 * torch.randn(1, H, R, generator=g) + mark).to(torch.bfloat16).float()
            scale = 12.0 / R
            perm = torch.randperm(-(-n // page), generator=g)
            low = max(0, pos - size + 1) // page
            pages = torch.full((len(perm), page, R), float("nan"), dtype=torch.bfloat16)
            for p in range(low * page, pos + 1):
                pages[perm[p // page], p % page] = keys[p]
            bt = torch.where(torch.arange(len(perm)) >= low, perm, torch.full_like(perm, -1)).to(torch.int32).view(1, -1).to(DEV)
            for sink in (None, torch.linspace(-1.0, 14.0, H)):
                plan = AttentionPlan(decode_only=kernel.startswith("split"), max_q_len=1, max_context_len=pos + 1, n_seqs=1, q_lens=[1],
                                     cu_seqlens=i32([0, 1]), workspace=Workspace(torch.device(DEV)))
                out = torch.empty(1, H, R, device=DEV)
                ops.ledger = []
                pages_dev = pages.to(DEV)
                ops.attention_latent(q.to(DEV), out, pages_dev, bt, page, i32([pos]), i32([0]), H, R, 0, scale,
                                     plan=None if kernel == "general" else plan, window=size - 1, sink=None if sink is None else sink.to(DEV),
                                     pages_t=pages_dev.transpose(1, 2).contiguous() if kernel.endswith("mfma") else None)
                torch.cuda.synchronize()
                ran, ops.ledger = ops.ledger[0][0], None
                # (key rows of 1,024 bytes do not fit the split kernel's LDS beside the queries)
                assert ran == {"general": "mv_attention_latent", "split": "mv_attention_latent_split" if R < 512 else "mv_attention_latent", "mfma": "mv_attention_latent_mfma", "split_mfma": "mv_attention_latent_split_mfma"}[kernel]
                s = [plain.windowed(q[0, h:h + 1].double() @ keys[:pos + 1].double().T * scale, pos, size) for h in range(H)]
                want = torch.cat([plain.sink_softmax(s[h], None if sink is None else sink[h].double()) for h in range(H)]) @ keys[:pos + 1].double()
                close(out[0], want, 1.2e-2, f"position {pos}, marked key {edge}")


# ---------------------------------------------------------------------------------------
# gated linear attention
# ---------------------------------------------------------------------------------------
def linear_case(H, dk, dv, rank, hid, seed, slow=0.0):
    g = torch.Generator().manual_seed(seed)
    shapes = {"q": (H * dk, hid), "k": (H * dk, hid), "v": (H * dv, hid), "g": (H * dv, hid), "o": (hid, H * dv), "norm": (dv,),
              "a1": (rank, hid), "a2": (H * dk, rank), "a2.b": (H * dk,)}
    w = {}
    for name, s in shapes.items():
        t = torch.randn(s, generator=g)
        if len(s) == 2:
            t = t / s[1] ** 0.5
        if name == "norm":
            t = 1 + 0.2 * t
        if name == "a2.b":
            t = t + slow
        w[name] = t.to(torch.bfloat16)
    return w


def build_linear(rt, w, H, dk, dv, rank, hid, eps, tau, out_scale=1.0):
    from minivllm_amd.parts.matrix_state import GatedLinear, GatedLinearSpec
    spec = GatedLinearSpec(hidden_size=hid, num_heads=H, key_dim=dk, value_dim=dv, decay_rank=rank, tau=tau, out_norm_eps=eps,
                           out_scale=out_scale)
    return GatedLinear(spec, {k.replace("a2.b", "a2_bias"): v.to(DEV) for k, v in w.items()}, rt)


def plain_linear(x, w, H, dk, dv, eps, tau, S, dtype):
    rnd = plain.keep if dtype == torch.float32 else plain.round_to_bfloat16
    y, new = plain.right_mixer(x.double(), {k: v.double() for k, v in w.items()}, "", {"heads": H, "dim": dk, "vdim": dv, "tau": tau}, eps,
                               None if S is None else {"S": S}, rnd)
    return y, new["S"]


def finished(y):
    y = y if isinstance(y, torch.Tensor) else y.materialize()
    torch.cuda.synchronize()
    return y


LINEAR_SIZES = [(3, 12, 20, 6, 8.0), (5, 6, 10, 3, 16.0), (2, 64, 64, 32, 16.0), (1, 8, 16, 1, 1.0), (4, 32, 100, 17, 3.0), (2, 128, 64, 40, 16.0),
                (1, 200, 7, 5, 2.0), (2, 70, 40, 9, 30.0), (16, 64, 64, 16, 16.0), (2, 16, 300, 4, 5.0), (1, 260, 12, 4, 4.0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, dk, dv, rank, tau", LINEAR_SIZES)
@pytest.mark.parametrize("q_lens", [[9, 1, 4, 2], [150, 3, 67, 64], [1, 130], [1, 1, 1, 1]])
def test_gated_linear_step(dtype, H, dk, dv, rank, tau, q_lens):
    """Requests on slots out of order from states that are not zero; prompt portions with padding rows and a padding sequence,
    and single tokens (one kernel where it serves the sizes)."""
    rt = runtime(dtype)
    hid, eps = 64, 1e-5
    w = linear_case(H, dk, dv, rank, hid, seed=H * 100 + dk)
    part = build_linear(rt, w, H, dk, dv, rank, hid, eps, tau)
    g = torch.Generator().manual_seed(3)
    slots, n = [2, 0, 3, 1][:len(q_lens)], sum(q_lens)
    single = max(q_lens) == 1
    pad = 0 if single else 2
    x = torch.randn(n + pad, hid, generator=g).to(dtype)
    S0 = torch.randn(5, H, dk, dv, generator=g)
    state = S0.transpose(2, 3).contiguous().to(DEV)
    rt.ops.ledger = []
    y = finished(part.forward(x.to(DEV), context(q_lens, slots, {"state": state}, pad, 1 if pad else 0), 0))
    ran, rt.ops.ledger = [e[0] for e in rt.ops.ledger], None
    stepped = single and dk <= 256 and dv <= 256
    assert ("mv_gated_linear_step" in ran) == stepped and ("mv_gated_linear_chunks" in ran) != stepped
    base = 0
    for qn, slot in zip(q_lens, slots):
        want, S = plain_linear(x[base:base + qn], w, H, dk, dv, eps, tau, S0[slot].double(), dtype)
        close(y[base:base + qn], want, 3e-5 if dtype == torch.float32 else 2e-2, f"request of {qn}")
        close(state[slot].transpose(1, 2), S, 3e-5 if dtype == torch.float32 else 6e-3, "state")
        base += qn
    untouched = sorted(set(range(5)) - set(slots))
    assert torch.equal(state[untouched].cpu(), S0[untouched].transpose(2, 3)), "a slot of nobody was touched"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tau, slow", [(16.0, 3.0), (1.0, -6.0), (1.0, 0.0)])
def test_gated_linear_portions_and_long_runs(dtype, tau, slow):
    """700 tokens whole against portions of many sizes, down to one token, with decays of almost one, decays that forget
    within a token (their products leave float32's range inside a chunk), and ordinary ones."""
    H, dk, dv, rank, hid, eps = 2, 64, 48, 12, 48, 1e-6
    rt = runtime(dtype)
    w = linear_case(H, dk, dv, rank, hid, seed=5, slow=slow)
    part = build_linear(rt, w, H, dk, dv, rank, hid, eps, tau, out_scale=0.6)
    x = torch.randn(700, hid, generator=torch.Generator().manual_seed(9)).to(dtype)
    want, S = plain_linear(x, w, H, dk, dv, eps, tau, None, dtype)
    tol = 5e-5 if dtype == torch.float32 else 2e-2
    for sizes in ([700], [64, 63, 65, 128, 127, 1, 2, 250], [2, 2, 3, 31, 32, 33, 15, 16, 17, 549], [600] + [1] * 100):
        state, p, out = torch.zeros(1, H, dv, dk, device=DEV), 0, []
        for n in sizes:
            out.append(finished(part.forward(x[p:p + n].to(DEV), context([n], [0], {"state": state}), 0)).clone())
            p += n
        close(torch.cat(out), 0.6 * want, tol, str(sizes[:5]))
        close(state[0].transpose(1, 2), S, 5e-5 if dtype == torch.float32 else 6e-3, "state")


@pytest.mark.parametrize("dtype", DTYPES)
def test_gated_linear_many_requests(dtype):
    """More requests than a workgroup has threads, of one to three tokens and a few chunks, in one step."""
    H, dk, dv, rank, hid, eps, tau = 2, 8, 12, 4, 32, 1e-5, 6.0
    rt = runtime(dtype)
    g = torch.Generator().manual_seed(2)
    q_lens = [int(v) for v in torch.randint(1, 4, (290,), generator=g)]
    q_lens[5], q_lens[256], q_lens[289] = 130, 70, 65
    w = linear_case(H, dk, dv, rank, hid, seed=1)
    part = build_linear(rt, w, H, dk, dv, rank, hid, eps, tau)
    x = torch.randn(sum(q_lens), hid, generator=g).to(dtype)
    state = torch.zeros(290, H, dv, dk, device=DEV)
    y = finished(part.forward(x.to(DEV), context(q_lens, list(range(289, -1, -1)), {"state": state}), 0))
    base = 0
    errors = []
    for s, n in enumerate(q_lens):
        want, S = plain_linear(x[base:base + n], w, H, dk, dv, eps, tau, None, dtype)
        errors.append(float((y[base:base + n].double().cpu() - want).abs().max()))
        close(state[289 - s].transpose(1, 2), S, 2e-5 if dtype == torch.float32 else 1e-2, f"state of request {s}")
        base += n
    # (a first token's output is its value times the sign of q.k: where that nearly vanishes, rounding decides)
    errors.sort()
    assert errors[int(len(errors) * 0.97)] <= (1e-4 if dtype == torch.float32 else 0.12), errors[-12:]


# ---------------------------------------------------------------------------------------
# the real-gated linear recurrent unit
# ---------------------------------------------------------------------------------------
def unit_case(W, B, taps, hid, seed):
    g = torch.Generator().manual_seed(seed)
    P = W // B
    shapes = {"y": (W, hid), "y.b": (W,), "x": (W, hid), "x.b": (W,), "conv": (W, taps), "conv.b": (W,), "ra": (B, P, P), "ra.b": (B, P),
              "ri": (B, P, P), "ri.b": (B, P), "lam": (W,), "o": (hid, W)}
    w = {}
    for name, s in shapes.items():
        t = torch.randn(s, generator=g)
        if name in ("y", "x", "o", "ra", "ri"):
            t = 1.3 * t / s[-1] ** 0.5
        if name == "lam":
            t = 1.5 * t - 3.0
        w[name] = t.to(torch.bfloat16)
    return w


def build_unit(rt, w, W, B, taps, hid):
    from minivllm_amd.parts.recurrent_unit import RecurrentUnit, RecurrentUnitSpec
    return RecurrentUnit(RecurrentUnitSpec(hidden_size=hid, width=W, blocks=B, conv_taps=taps),
                         {k.replace(".b", "_bias"): v.to(DEV) for k, v in w.items()}, rt)


def plain_unit(x, w, m, state, dtype):
    rnd = plain.keep if dtype == torch.float32 else plain.round_to_bfloat16
    w = {k: v.double() for k, v in w.items()}
    return plain.rglru_mixer(x.double(), w, "", m, 1e-5, state, rnd)


UNIT_SIZES = [(48, 3, 3), (33, 3, 1), (20, 1, 2), (192, 2, 4), (45, 5, 6), (512, 1, 4), (1024, 8, 4), (640, 1, 3), (24, 6, 4), (256, 4, 1)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W, B, taps", UNIT_SIZES)
@pytest.mark.parametrize("q_lens", [[9, 1, 4, 2], [70, 3, 33, 32], [1, 130], [1, 1, 1, 1]])
def test_recurrent_unit_step(dtype, W, B, taps, q_lens):
    rt = runtime(dtype)
    hid = 64
    w = unit_case(W, B, taps, hid, seed=W + taps)
    part = build_unit(rt, w, W, B, taps, hid)
    g = torch.Generator().manual_seed(3)
    slots, n = [2, 0, 3, 1][:len(q_lens)], sum(q_lens)
    single = max(q_lens) == 1
    pad = 0 if single else 2
    x = torch.randn(n + pad, hid, generator=g).to(dtype)
    S0 = torch.randn(5, W, generator=g)
    c0 = torch.randn(5, taps - 1, W, generator=g).to(dtype)
    state, conv = S0.clone().to(DEV), c0.clone().to(DEV)
    rt.ops.ledger = []
    y = finished(part.forward(x.to(DEV), context(q_lens, slots, {"state": state, "conv": conv}, pad, 1 if pad else 0), 0))
    ran, rt.ops.ledger = [e[0] for e in rt.ops.ledger], None
    stepped = single and (W // B) % 4 == 0 and W // B <= 512
    assert ("mv_unit_step" in ran) == stepped and ("mv_unit_scan" in ran) != stepped
    base = 0
    for qn, slot in zip(q_lens, slots):
        want, new = plain_unit(x[base:base + qn], w, {}, {"S": S0[slot].double(), "conv": c0[slot].double()}, dtype)
        close(y[base:base + qn], want, 2e-5 if dtype == torch.float32 else 2e-2, f"request of {qn}")
        close(state[slot], new["S"], 1e-5 if dtype == torch.float32 else 1e-2, "state")
        if taps > 1:
            close(conv[slot], new["conv"], 1e-6 if dtype == torch.float32 else 8e-3, "kept inputs")
        base += qn
    untouched = sorted(set(range(5)) - set(slots))
    assert torch.equal(state[untouched].cpu(), S0[untouched]) and torch.equal(conv[untouched].cpu(), c0[untouched])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [3, 70, 333])
def test_recurrent_unit_many_single_tokens(dtype, rows):
    """Two rows a workgroup once the rows fill the chip (an odd number of rows among them), on slots in reverse order."""
    W, B, taps, hid = 128, 8, 4, 64
    rt = runtime(dtype)
    w = unit_case(W, B, taps, hid, seed=1)
    part = build_unit(rt, w, W, B, taps, hid)
    g = torch.Generator().manual_seed(4)
    x, S0, c0 = torch.randn(rows, hid, generator=g).to(dtype), torch.randn(rows, W, generator=g), torch.randn(rows, taps - 1, W, generator=g).to(dtype)
    state, conv = S0.clone().to(DEV), c0.clone().to(DEV)
    y = finished(part.forward(x.to(DEV), context([1] * rows, list(range(rows - 1, -1, -1)), {"state": state, "conv": conv}), 0))
    for r in list(range(0, rows, 7)) + [rows - 1]:
        slot = rows - 1 - r
        want, new = plain_unit(x[r:r + 1], w, {}, {"S": S0[slot].double(), "conv": c0[slot].double()}, dtype)
        close(y[r:r + 1], want, 2e-5 if dtype == torch.float32 else 3e-2, f"row {r}")
        close(state[slot], new["S"], 1e-5 if dtype == torch.float32 else 1e-2, "state")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("B", [2, 5])
def test_recurrent_unit_portions_and_long_runs(dtype, B):
    """500 tokens whole, in portions down to one token, and mostly one by one; blocks of a size that the one-launch kernel
    serves and of one that it does not."""
    W, taps, hid = (96, 4, 48) if B == 2 else (45, 4, 48)
    rt = runtime(dtype)
    w = unit_case(W, B, taps, hid, seed=8)
    part = build_unit(rt, w, W, B, taps, hid)
    x = torch.randn(500, hid, generator=torch.Generator().manual_seed(2)).to(dtype)
    want, new = plain_unit(x, w, {}, None, dtype)
    for sizes in ([500], [2, 3, 2, 31, 32, 33, 1, 1, 64, 65, 266], [100] + [1] * 400):
        state, conv = torch.zeros(1, W, device=DEV), torch.zeros(1, taps - 1, W, dtype=dtype, device=DEV)
        out, p = [], 0
        for n in sizes:
            out.append(finished(part.forward(x[p:p + n].to(DEV), context([n], [0], {"state": state, "conv": conv}), 0)).clone())
            p += n
        close(torch.cat(out), want, 3e-5 if dtype == torch.float32 else 2e-2, str(sizes[:6]))
        close(state[0], new["S"], 3e-5 if dtype == torch.float32 else 1e-2, "state")


def test_recurrent_unit_constants_by_hand():
    """One channel: a gate at one half, softplus(0) = ln 2, so a = exp(-8 ln 2 / 2) = 1/16; no special first token."""
    rt = runtime(torch.float32)
    w = {k: torch.zeros(s) for k, s in {"y": (1, 1), "y.b": (1,), "x": (1, 1), "x.b": (1,), "conv": (1, 1), "conv.b": (1,), "ra": (1, 1, 1),
                                        "ra.b": (1, 1), "ri": (1, 1, 1), "ri.b": (1, 1), "lam": (1,), "o": (1, 1)}.items()}
    w["y.b"][:], w["x"][:], w["conv"][:], w["o"][:] = 2.0, 1.0, 1.0, 1.0
    part = build_unit(rt, {k: v.float() for k, v in w.items()}, 1, 1, 1, 1)
    state = torch.zeros(1, 1, device=DEV)
    y = finished(part.forward(torch.tensor([[1.0], [3.0]], device=DEV), context([2], [0], {"state": state}), 0)).cpu().double()
    gain = math.sqrt(1 - 1 / 256) * 0.5
    act = float(plain.gelu_tanh(torch.tensor(2.0, dtype=torch.float64)))
    want = torch.tensor([[gain * act], [(gain / 16 + 3 * gain) * act]], dtype=torch.float64)
    close(y, want, 1e-6, "two tokens")


# ---------------------------------------------------------------------------------------
# feed-forward, block
# ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype, hid, ff, rows", [
    (torch.float32, 50, 30, 7), (torch.float32, 64, 96, 65), (torch.bfloat16, 50, 30, 9), (torch.bfloat16, 64, 96, 1), (torch.bfloat16, 64, 96, 300),
    (torch.bfloat16, 192, 256, 40), (torch.bfloat16, 1024, 4608, 1), (torch.bfloat16, 1024, 4608, 8), (torch.bfloat16, 1024, 4608, 16),
    (torch.bfloat16, 1024, 4608, 64), (torch.bfloat16, 1024, 4608, 200), (torch.bfloat16, 2048, 3072, 20), (torch.bfloat16, 1024, 4608, 2000),
    (torch.bfloat16, 4096, 4608, 8), (torch.bfloat16, 4096, 4608, 64), (torch.bfloat16, 4096, 18432, 8)])
@pytest.mark.parametrize("bias", [True, False])
def test_squared_relu(dtype, hid, ff, rows, bias):
    """... which the weight-streaming and the tiled product apply themselves, the latter where it does not split K."""
    from minivllm_amd.parts.mlp import SquaredReLU, SquaredReLUSpec
    rt = runtime(dtype)
    g = torch.Generator().manual_seed(hid + ff)
    some = torch.randn(min(ff, 2048), hid, generator=g).repeat(-(-ff // 2048), 1)[:ff]          # (many rows: the same ones again)
    w = {"up": some / hid ** 0.5, "down": torch.randn(hid, ff, generator=g) / ff ** 0.5, "up.b": 0.8 * torch.randn(ff, generator=g), "down.b": 0.8 * torch.randn(hid, generator=g)}
    w = {k: (v if bias or not k.endswith(".b") else 0 * v).to(torch.bfloat16) for k, v in w.items()}
    part = SquaredReLU(SquaredReLUSpec(hidden_size=hid, intermediate_size=ff, bias=bias),
                       {k.replace(".b", "_bias"): v.to(DEV) for k, v in w.items() if bias or not k.endswith(".b")}, rt)
    x = torch.randn(rows, hid, generator=torch.Generator().manual_seed(rows)).to(dtype)
    rt.ops.ledger = []
    y = finished(part.forward(x.to(DEV), None))
    ran, rt.ops.ledger = [e[0] for e in rt.ops.ledger], None
    fused = ran[0] == "mv_gemm_skinny" or (ran[0] == "mv_gemm_tile" and rt.ops.lib.dll.mv_gemm_tile_splits(rows, ff, hid, 0, 0) == 1)
    assert ("mv_squared_relu" in ran) != fused, ran
    if ff == 18432:
        assert ran[0] == "mv_gemm_tile" and fused, ran
    want = plain.feed_forward(x.double(), {k: v.double() for k, v in w.items()}, "")
    close(y, want, 1e-5 if dtype == torch.float32 else 1.2e-2, f"{rows} rows")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [64, 50, 1024, 2056, 4096, 8200])
@pytest.mark.parametrize("rows", [1, 5, 200])
@pytest.mark.parametrize("with_copy", [True, False])
def test_norm_behind_a_sublayer(dtype, W, rows, with_copy):
    """resid += norm(y) in float32, and the residual's rows in the activation type with it."""
    ops = ops_for(dtype)
    g = torch.Generator().manual_seed(W)
    y, x0, w = (3 * torch.randn(rows, W, generator=g)).to(dtype), torch.randn(rows, W, generator=g), 1 + 0.2 * torch.randn(W, generator=g)
    w = w.to(torch.bfloat16)
    resid = x0.to(DEV)
    copy = torch.empty(rows, W, dtype=dtype, device=DEV) if with_copy else None
    ops.norm_add_norm(y.to(DEV), (w.to(DEV), 1e-5, False), resid, None, copy)
    torch.cuda.synchronize()
    want = x0.double() + plain.rms_norm(y.double(), w.double(), 1e-5)
    close(resid, want, 1e-6, "residual")
    if with_copy:
        assert torch.equal(copy, resid.to(dtype)), "the copy is not the residual rounded"
    rounded = torch.empty(rows, W, dtype=dtype, device=DEV)
    ops.round_rows(resid, rounded)
    assert torch.equal(rounded, resid.to(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [((4, 2, 16, 24), (3, 12, 20)), ((3, 1, 10, 6), (5, 6, 10)), ((2, 1, 64, 64), (2, 32, 32)), ((1, 1, 8, 5), (1, 8, 3))])
def test_two_mixers_summed(dtype, sizes):
    """The part whole, a portion and single tokens behind it, for rows of the joined heads that need gaps and for rows that
    need none; the constants on the two sides differ and one is negative."""
    from minivllm_amd.parts.attention import AttentionSpec
    from minivllm_amd.parts.matrix_state import GatedLinearSpec
    from minivllm_amd.parts.parallel import ParallelSum, ParallelSumSpec
    from minivllm_amd.parts.rope import RotaryEmbedding, RotarySpec
    (H, G, D, Dv), (R, dk, dv) = sizes
    rt = runtime(dtype)
    hid, eps, taps, size, rank, page = 48, 1e-5, 3, 14, 5, 16
    g = torch.Generator().manual_seed(H + dk)
    w = {"right." + k: v for k, v in linear_case(R, dk, dv, rank, hid, seed=2).items()}
    for name, s in {"q": (H * D, hid), "k": (G * D, hid), "v": (G * Dv, hid), "o": (hid, H * Dv)}.items():
        w["left." + name] = (torch.randn(s, generator=g) / s[1] ** 0.5).to(torch.bfloat16)
        if name != "o":
            w[f"left.{name}.conv"] = (0.6 * torch.randn(s[0], taps, generator=g)).to(torch.bfloat16)
    rot = {"dims": D // 4 * 2, "base": 100.0}
    m = {"left": {"heads": H, "kv_heads": G, "dim": D, "vdim": Dv, "scale": 0.5, "softcap": 5.0, "mask": {"size": size}, "rot": rot},
         "right": {"heads": R, "dim": dk, "vdim": dv, "tau": 5.0}, "left_scale": 0.8, "right_scale": -0.6}
    rope = RotarySpec(rotary_dim=rot["dims"], theta=100.0)
    spec = ParallelSumSpec(hidden_size=hid,
                           left=AttentionSpec(hidden_size=hid, num_heads=H, num_kv_heads=G, head_dim=D, value_dim=Dv, scale=0.5, qk_norm_eps=eps,
                                              window=size - 1, position=rope, unit_norm_after_rotation=True, softcap=5.0, conv_taps=taps,
                                              out_scale=0.8),
                           right=GatedLinearSpec(hidden_size=hid, num_heads=R, key_dim=dk, value_dim=dv, decay_rank=rank, tau=5.0,
                                                 out_norm_eps=eps, out_scale=-0.6))
    rename = lambda k: k.replace("a2.b", "a2_bias").replace(".conv", "_conv")
    part = ParallelSum(spec, {rename(k): v.to(DEV) for k, v in w.items()}, rt, position=RotaryEmbedding(rope, {}, rt))
    T = 60
    x = torch.randn(T, hid, generator=g).to(dtype)
    rnd = plain.keep if dtype == torch.float32 else plain.round_to_bfloat16
    want, _ = plain.parallel_mixer(x.double(), {k: v.double() for k, v in w.items()}, "", m, eps, None, rnd)
    blocks = -(-T // page)
    pages = {"k": torch.full((blocks, G, page, D), float("nan"), dtype=dtype, device=DEV),
             "v": torch.full((blocks, G, Dv, page), float("nan"), dtype=dtype, device=DEV)}
    states = {"conv": torch.zeros(1, taps - 1, spec.left.conv_channels, dtype=dtype, device=DEV), "state": torch.zeros(1, R, dv, dk, device=DEV)}
    table = torch.randperm(blocks, generator=g).to(torch.int32).view(1, -1).to(DEV)
    p, out = 0, []
    for n in [30, 2, 1, 1, 17] + [1] * 9:
        ctx = context([n], [0], states, starts=[p], kv=(pages, None, table), page=page)
        out.append(finished(part.forward(x[p:p + n].to(DEV), ctx, 0)).clone())
        p += n
    close(torch.cat(out), want, 3e-5 if dtype == torch.float32 else 3e-2, "sum")
