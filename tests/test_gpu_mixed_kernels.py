"""The mixed-layer decoder's kernels one by one, through the C ABI, against the
plain float64 statement of each mechanism."""
import ctypes

import numpy as np
import pytest
import torch

import mixed_model as mm
import mixer_oracle as mo
import qllm_hip as qh
from kernel_util import BF16, F32, close, on, packed, padded, steps, torch_type

pytestmark = pytest.mark.gpu

# ---- linear --------------------------------------------------------------------


def padded_input(device, x, columns, element):
    out = torch.zeros((x.shape[0], padded(columns, 64)), dtype=torch_type(element), device=device)
    out[:, :x.shape[1]] = on(device, x)
    return out


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("batch", [1, 2, 16, 17, 33, 64, 65, 130, 300])
def test_linear_segments_of_every_epilogue(device, element, batch):
    rng = np.random.default_rng(batch)
    shapes = [(70, 200), (33, 90)]
    matrices = [mm.bf16(rng.standard_normal(s) / np.sqrt(s[1])) for s in shapes]
    gate, up = (mm.bf16(rng.standard_normal((45, 200)) / 14) for _ in range(2))
    inputs = [mm.bf16(rng.standard_normal((batch, s[1]))) for s in shapes]
    first = packed(device, [(matrices[0], 0, 1, 0)], 70, 200)
    second = packed(device, [(matrices[1], 0, 1, 0)], 33, 90)
    pair = packed(device, [(gate, 0, 2, 0), (up, 1, 2, 0)], 96, 200)
    x0 = padded_input(device, inputs[0], 200, element)
    x1 = padded_input(device, inputs[1], 90, element)
    base = rng.standard_normal((batch, 36)).astype(np.float32)
    store = torch.full((batch, 72), 7.0, device=device)
    add = on(device, base)
    gated = torch.zeros((batch, 64), dtype=torch_type(element), device=device)
    segments = (qh.LinearSegment * 3)(
        qh.LinearSegment(qh.ptr(first), qh.ptr(x0), qh.ptr(store), 80, 256, 256, 72, 70,
                         qh.LINEAR_STORE, 0, 0),
        qh.LinearSegment(qh.ptr(second), qh.ptr(x1), qh.ptr(add), 48, 128, 128, 36, 33,
                         qh.LINEAR_ADD, 0, 0),
        qh.LinearSegment(qh.ptr(pair), qh.ptr(x0), qh.ptr(gated), 96, 256, 256, 64, 45,
                         qh.LINEAR_GATED, 0, 0))
    qh.call("qllm_linear_batch", segments, 3, batch, element, None)
    torch.cuda.synchronize()
    products = [x.astype(np.float64) @ m.T.astype(np.float64)
                for x, m in zip(inputs, matrices)]
    # bf16 inputs and weights, F32 sums: both modes give the product itself
    close(store[:, :70], products[0], F32, "store")
    assert torch.all(store[:, 70:] == 7.0)
    close(add[:, :33], base[:, :33] + products[1], F32, "add")
    assert np.array_equal(add[:, 33:].cpu().numpy(), base[:, 33:])
    x = inputs[0].astype(np.float64)
    want = mo.gelu_tanh(x @ gate.T.astype(np.float64)) * (x @ up.T.astype(np.float64))
    close(gated[:, :45], want, element, "gated")
    assert torch.all(gated[:, 45:] == 0)


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("splits", [1, 3, 7])
def test_linear_partials_and_side_by_side_columns(device, element, splits):
    rng = np.random.default_rng(splits)
    left, right = (mm.bf16(rng.standard_normal((50, n)) / 12) for n in (70, 100))
    weights = packed(device, [(left, 0, 1, 0), (right, 0, 1, 128)], 50, 256)
    x = np.zeros((5, 256), dtype=np.float32)
    x[:, :70] = mm.bf16(rng.standard_normal((5, 70)))
    x[:, 128:228] = mm.bf16(rng.standard_normal((5, 100)))
    d_x = padded_input(device, x, 256, element)
    out = torch.zeros((splits, 5, 52), device=device)
    segment = qh.LinearSegment(qh.ptr(weights), qh.ptr(d_x), qh.ptr(out), 64, 256, 256, 52, 50,
                               qh.LINEAR_PARTIALS, 0, splits)
    qh.call("qllm_linear_batch", ctypes.byref(segment), 1, 5, element, None)
    torch.cuda.synchronize()
    want = x[:, :70].astype(np.float64) @ left.T + x[:, 128:228].astype(np.float64) @ right.T
    close(out.sum(0)[:, :50], want, F32)


def test_linear_tall_tiles_of_all_sizes(device):
    rng = np.random.default_rng(3)
    for rows, columns, batch in ((2100, 128, 700), (4096, 64, 1030), (300, 320, 129)):
        w = mm.bf16(rng.standard_normal((rows, columns)) / 12)
        x = mm.bf16(rng.standard_normal((batch, columns)))
        weights = packed(device, [(w, 0, 1, 0)], rows, columns)
        d_x = padded_input(device, x, columns, BF16)
        out = torch.zeros((batch, padded(rows, 4)), device=device)
        segment = qh.LinearSegment(qh.ptr(weights), qh.ptr(d_x), qh.ptr(out), padded(rows, 16),
                                   padded(columns, 64), padded(columns, 64), padded(rows, 4),
                                   rows, qh.LINEAR_STORE, 0, 0)
        qh.call("qllm_linear_batch", ctypes.byref(segment), 1, batch, BF16, None)
        torch.cuda.synchronize()
        close(out[:, :rows], x.astype(np.float64) @ w.T.astype(np.float64), F32)


# ---- stream ---------------------------------------------------------------------


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("width", [64, 90, 132])
def test_embedding_norms_partials_and_gather(device, element, width):
    rng = np.random.default_rng(width)
    table = mm.bf16(rng.standard_normal((30, width)))
    tokens = np.array([3, 29, 0, 3, 17], dtype=np.int32)
    x = torch.zeros((5, width), device=device)
    d_table, d_tokens = on(device, table, torch.bfloat16), on(device, tokens, torch.int32)
    qh.call("qllm_embedding_bf16_batch", qh.ptr(d_table), 30, qh.ptr(d_tokens), qh.ptr(x), 5,
            width, 0.75, None)
    torch.cuda.synchronize()
    assert np.array_equal(x.cpu().numpy(), table[tokens] * np.float32(0.75))

    stride = padded(width, 64)
    partials = rng.standard_normal((9, 5, padded(width, 4))).astype(np.float32)
    weights = rng.standard_normal((2, width)).astype(np.float32)
    d_weights = [on(device, w) for w in weights]
    outs = [torch.full((5, stride), 9.0, dtype=torch_type(element), device=device)
            for _ in range(2)]
    summed = torch.zeros((5, width), device=device)
    d_partials = on(device, partials)
    launch = qh.StreamNormLaunch(
        qh.ptr(x), qh.ptr(summed), qh.ptr(d_partials), 9, padded(width, 4),
        (ctypes.c_void_p * 2)(*map(qh.ptr, d_weights)),
        (ctypes.c_void_p * 2)(*map(qh.ptr, outs)), (ctypes.c_uint32 * 2)(stride, stride),
        5, width, 1e-5, element, None, None, None)
    qh.call("qllm_stream_norm", ctypes.byref(launch), None)
    torch.cuda.synchronize()
    stream = table[tokens].astype(np.float64) * 0.75 + partials[:, :, :width].sum(0)
    close(summed, stream, F32)
    for out, w in zip(outs, weights):
        close(out[:, :width], mo.rms(stream, 1e-5) * w, element)
        assert torch.all(out[:, width:] == 0)

    rows = torch.tensor([4, 0, 4], dtype=torch.int32, device=device)
    picked = torch.zeros((3, stride), dtype=torch_type(element), device=device)
    launch = qh.StreamNormLaunch(
        qh.ptr(summed), None, None, 0, 0, (ctypes.c_void_p * 2)(qh.ptr(d_weights[0]), None),
        (ctypes.c_void_p * 2)(qh.ptr(picked), None), (ctypes.c_uint32 * 2)(stride, 0),
        3, width, 1e-5, element, None, qh.ptr(rows), None)
    qh.call("qllm_stream_norm", ctypes.byref(launch), None)
    torch.cuda.synchronize()
    close(picked[:, :width], (mo.rms(stream, 1e-5) * weights[0])[[4, 0, 4]], element)


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("width", [64, 90])
def test_token_shift_carries_the_last_norm(device, element, width):
    rng = np.random.default_rng(width)
    x = rng.standard_normal((7, width)).astype(np.float32)
    weight, *mus = rng.uniform(0.1, 1.0, (4, width)).astype(np.float32)
    stride = padded(width, 64)
    slot_stride = padded(width, 4) + 8
    carried = torch.zeros(2 * slot_stride, device=device)
    last = torch.zeros(padded(width, 4), device=device)
    d_weight, d_mus = on(device, weight), [on(device, mu) for mu in mus]
    normed = mo.rms(x.astype(np.float64), 1e-5) * weight
    before = np.zeros(width)
    for first, count in ((0, 1), (1, 2), (3, 4)):
        d_x = on(device, x[first:first + count])
        outs = [torch.zeros((count, stride), dtype=torch_type(element), device=device)
                for _ in mus]
        shift = qh.TokenShift(3, (ctypes.c_void_p * 6)(*map(qh.ptr, d_mus)),
                              (ctypes.c_void_p * 6)(*map(qh.ptr, outs)), qh.ptr(carried),
                              slot_stride, qh.ptr(last))
        step = steps(device, first, slot=1)
        launch = qh.StreamNormLaunch(
            qh.ptr(d_x), None, None, 0, 0, (ctypes.c_void_p * 2)(qh.ptr(d_weight), None),
            (ctypes.c_void_p * 2)(None, None), (ctypes.c_uint32 * 2)(stride, 0), count, width,
            1e-5, element, ctypes.pointer(shift), None, qh.ptr(step))
        qh.call("qllm_stream_norm", ctypes.byref(launch), None)
        torch.cuda.synchronize()
        part = normed[first:first + count]
        for out, mu in zip(outs, mus):
            close(out[:, :width], mo.shift_mix(part, before, mu), element)
        before = part[-1]
        close(last[:width], before, F32)
        carried[slot_stride:slot_stride + width] = last[:width]


# ---- attention -------------------------------------------------------------------


class Attention:
    """Pages, table and launches of one attention layer; rows are fed in any
    portions, outputs come back in order."""

    def __init__(self, device, element, heads, kv, dim, vdim, window, sinks, mix, scale,
                 rotary=0, base=1000.0, page_tokens=64, context=512, slots=1, strides=None):
        self.device, self.element = device, element
        self.heads, self.kv, self.dim, self.vdim = heads, kv, dim, vdim
        self.stride = (heads + kv) * dim + kv * vdim + heads
        self.stride += -self.stride % 4
        key, value = strides or (padded(dim, 64), padded(vdim, 64))
        key, value = (128 if 64 < s <= 128 else 256 if 128 < s <= 256 else s
                      for s in (key, value))
        self.key, self.mix = key, None if mix is None else on(device, mix)
        pages = context // page_tokens
        layer = qh.call("qllm_windowed_layer_bytes", page_tokens, kv, key, value, element)
        self.offset = 64
        self.pages = [torch.zeros(layer + 64, dtype=torch.uint8, device=device)
                      for _ in range(pages * slots)]
        # pages in no particular order
        order = np.random.default_rng(0).permutation(len(self.pages))
        self.table = torch.tensor([self.pages[i].data_ptr() for i in order],
                                  dtype=torch.int64, device=device)
        self.step = steps(device, 0)
        self.rotary, self.base = rotary, base
        self.frequencies = torch.tensor(
            [base ** (-2.0 * i / rotary) for i in range(rotary // 2)] or [0.0],
            dtype=torch.float64, device=device)
        self.layer = qh.WindowedAttention(
            heads, kv, dim, vdim, key, value, window, sinks, scale, qh.ptr(self.mix),
            page_tokens, pages, self.offset, qh.ptr(self.table), qh.ptr(self.step), element)

    def run(self, projections, position, slot=0, first=None, share=None):
        rows = projections.shape[0]
        d = on(self.device, projections)
        self.step.copy_(torch.tensor([position, slot, rows, 0], dtype=torch.int32))
        query = torch.zeros((rows, self.heads, self.key), dtype=torch_type(self.element),
                            device=self.device)
        kept = torch.zeros((rows, self.kv * self.vdim), device=self.device)
        at = self.heads * self.dim, (self.heads + self.kv) * self.dim
        gate = at[1] + self.kv * self.vdim
        d_first = None if first is None else on(self.device, first)
        d_share = None if share is None else torch.tensor([share], device=self.device)
        store = qh.RopeStoreLaunch(
            qh.ptr(d), self.stride, 0, at[0], at[1], self.rotary, qh.ptr(self.frequencies),
            qh.ptr(d_first), qh.ptr(d_share), qh.ptr(kept), qh.ptr(query), rows)
        qh.call("qllm_windowed_rope_store", ctypes.byref(self.layer), ctypes.byref(store), None)
        size = qh.call("qllm_windowed_attention_workspace_bytes", ctypes.byref(self.layer),
                       rows, position + rows - 1)
        workspace = torch.zeros(max(size, 16), dtype=torch.uint8, device=self.device)
        out = torch.zeros((rows, self.heads * self.vdim), dtype=torch_type(self.element),
                          device=self.device)
        launch = qh.AttentionLaunch(
            qh.ptr(query), d.data_ptr() + 4 * gate, self.stride, qh.ptr(out),
            self.heads * self.vdim, rows, position + rows - 1, qh.ptr(workspace), size)
        qh.call("qllm_windowed_attention_rows", ctypes.byref(self.layer), ctypes.byref(launch),
                None)
        torch.cuda.synchronize()
        assert np.array_equal(
            kept.cpu().numpy(),
            projections[:, at[1]:at[1] + self.kv * self.vdim])
        return out.float().cpu().numpy().astype(np.float64)

    def expected(self, projections, window, sinks, mix, scale, first=None, share=None):
        p = projections.astype(np.float64)
        rows = p.shape[0]
        at = self.heads * self.dim, (self.heads + self.kv) * self.dim
        where = np.arange(rows, dtype=np.float64)
        q = mo.rotate_interleaved(p[:, :at[0]].reshape(rows, self.heads, self.dim), where,
                                  self.rotary, self.base)
        k = mo.rotate_interleaved(p[:, at[0]:at[1]].reshape(rows, self.kv, self.dim), where,
                                  self.rotary, self.base)
        v = p[:, at[1]:at[1] + self.kv * self.vdim]
        if first is not None:
            v = (1.0 - share) * v + share * first
        v = v.reshape(rows, self.kv, self.vdim)
        gate = p[:, at[1] + self.kv * self.vdim:][:, :self.heads]
        out = mo.attention_core(q, k, v, where, where, scale, window or rows, sinks,
                                np.eye(self.heads) if mix is None else mix)
        return (out * mo.sigmoid(gate)[:, :, None]).reshape(rows, -1)


def stand_out(rng, layer, projections, pairs, head, strength=None):
    """Makes the score of (query row, key row) of one head stand out: the key
    becomes the query direction (unrotated dimensions or rotary 0 assumed)."""
    dim, group = layer.dim, layer.heads // layer.kv
    key_at = layer.heads * dim + head // group * dim
    for query, key in pairs:
        direction = mm.bf16(rng.standard_normal(dim))
        direction *= np.float32((strength or 5.0) / np.linalg.norm(direction) * dim ** 0.25)
        projections[query, head * dim:(head + 1) * dim] = direction
        projections[key, key_at:key_at + dim] = direction


SHAPES = [
    # heads, kv, dim, vdim, window, sinks, rotary, page tokens
    (6, 2, 56, 44, 40, 5, 56, 64),
    (3, 1, 24, 40, 33, 0, 16, 32),
    (12, 4, 48, 64, 64, 1, 48, 64),
    (16, 4, 128, 128, 70, 37, 64, 64),
    (20, 4, 80, 24, 31, 33, 32, 96),
    (32, 8, 64, 64, 90, 4, 64, 64),
    (24, 8, 128, 96, 1, 2, 0, 32),
    (8, 8, 32, 32, 0, 0, 32, 64),
    (9, 3, 16, 128, 50, 64, 16, 64),
    (6, 6, 160, 72, 48, 3, 20, 64),
    (36, 12, 40, 40, 45, 8, 40, 64),
    (40, 2, 32, 32, 45, 7, 20, 64),
    (64, 8, 128, 120, 35, 3, 64, 64),
]


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("shape", SHAPES, ids=lambda s: "x".join(map(str, s)))
def test_windowed_attention_in_portions(device, element, shape):
    heads, kv, dim, vdim, window, sinks, rotary, page_tokens = shape
    rng = np.random.default_rng(heads * dim + window)
    total, scale = 230, 1.3 / np.sqrt(dim)
    mix = mm.bf16(np.eye(heads) + 0.4 * rng.standard_normal((heads, heads)))
    layer = Attention(device, element, heads, kv, dim, vdim, window, sinks, mix, scale, rotary,
                      page_tokens=page_tokens, context=page_tokens * (1 + 256 // page_tokens))
    projections = mm.bf16(rng.standard_normal((total, layer.stride)))
    first = rng.standard_normal((total, kv * vdim)).astype(np.float32)
    want = layer.expected(projections, window, sinks, mix.astype(np.float64), scale, first, 0.3)
    at = 0
    got = []
    for count in (1, 2, 31, 3, 64, 4, 5, 1, 80, 17, 1, 1, 20):
        got.append(layer.run(projections[at:at + count], at, first=first[at:at + count],
                             share=0.3))
        at += count
    assert at == total
    close(np.concatenate(got), want, element, str(shape))


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("rows", [1, 3, 16])
@pytest.mark.parametrize("heads,kv,dim", [(4, 2, 64), (20, 4, 64)])
def test_edges_of_window_pages_and_kept_tokens(device, element, rows, heads, kv, dim):
    """One score stands out per case: a key just inside or outside the window,
    among or after the kept first tokens, at a page's border, at the query
    itself.  A mask off by one changes the output by its whole magnitude."""
    window, sinks, total = 48, 5, 192
    scale = dim ** -0.5
    rng = np.random.default_rng(rows)
    mix = mm.bf16(np.eye(heads) + 0.5 * rng.standard_normal((heads, heads)))
    query = total - 1
    keys = [query, query - 1, query - window + 1, query - window, query - window - 1,
            0, sinks - 1, sinks, sinks + 1, 127, 128, 63, 64, 159, 160]
    for head in (0, heads - 1):
        base = mm.bf16(0.5 * rng.standard_normal((total, 4 * heads * dim)))
        for key in keys:
            layer = Attention(device, element, heads, kv, dim, 32, window, sinks, mix, scale)
            projections = base[:, :layer.stride].copy()
            stand_out(rng, layer, projections, [(query, key)], head)
            want = layer.expected(projections, window, sinks, mix.astype(np.float64), scale)
            for wrong in ((window + 1, sinks), (window - 1, sinks), (window, sinks + 1),
                          (window, sinks - 1)):
                # the case would show such a mask: at the keys it is about the
                # planted score appears or goes
                if key in (query - window + 1, query - window, sinks - 1, sinks):
                    other = layer.expected(projections, *wrong, mix.astype(np.float64), scale)
                    shows = {(window + 1, sinks): query - window,
                             (window - 1, sinks): query - window + 1,
                             (window, sinks + 1): sinks,
                             (window, sinks - 1): sinks - 1}[wrong] == key
                    change = np.abs(other[-1] - want[-1]).max() / np.abs(want[-1]).max()
                    assert not shows or change > 0.2
            cut = total - rows
            layer.run(projections[:cut], 0)
            got = layer.run(projections[cut:], cut)
            close(got, want[cut:], element, f"head {head} key {key}")


def test_pages_and_slots_used_again(device):
    rng = np.random.default_rng(5)
    layer = Attention(device, BF16, 4, 2, 64, 64, 32, 2, None, 0.125, context=128, slots=2)
    long = mm.bf16(3.0 * rng.standard_normal((120, layer.stride)))
    short = mm.bf16(rng.standard_normal((40, layer.stride)))
    layer.run(long, 0, slot=1)
    for slot in (1, 0):
        want = layer.expected(short, 32, 2, None, 0.125)
        got = np.concatenate([layer.run(short[:33], 0, slot=slot),
                              layer.run(short[33:34], 33, slot=slot),
                              layer.run(short[34:], 34, slot=slot)])
        close(got, want, BF16, f"slot {slot}")


# ---- recurrences ------------------------------------------------------------------


class Recurrence:
    def __init__(self, device, element, kind, heads, dim, rank, rng, slots=2):
        self.device, self.element, self.kind = device, element, kind
        self.heads, self.dim, self.rank = heads, dim, rank
        n = heads * dim
        self.up = mm.bf16(rng.standard_normal((n, rank)) / np.sqrt(rank))
        self.base = mm.bf16(rng.standard_normal(n) - 1.0)
        self.bias, self.bonus, self.norm = mm.bf16(rng.standard_normal((3, n)))
        self.columns = [i * (n + 3) for i in range(5)]     # r k v gate rate, then low
        self.low = 5 * (n + 3)
        self.stride = self.low + rank + (-(self.low + rank)) % 4
        self.keep = [on(device, self.up, torch.bfloat16)] + [
            on(device, v) for v in (self.base, self.bias, self.bonus, self.norm)]
        self.slot_stride = n * dim + 12
        self.state = torch.zeros(slots * self.slot_stride, device=device)
        self.step = steps(device, 0)
        up, base, bias, bonus, norm = map(qh.ptr, self.keep)
        self.layer = qh.Recurrence(kind, heads, dim, rank, kind, 1e-5, 1e-6,
                                   -np.exp(-0.5), up, base, bias, bonus, norm,
                                   qh.ptr(self.state), self.slot_stride, qh.ptr(self.step),
                                   element)

    def run(self, projections, slot=1):
        rows = projections.shape[0]
        d = on(self.device, projections)
        self.step.copy_(torch.tensor([0, slot, rows, 0], dtype=torch.int32))
        size = qh.call("qllm_recurrence_workspace_bytes", ctypes.byref(self.layer), rows)
        workspace = torch.zeros(max(size, 16), dtype=torch.uint8, device=self.device)
        out = torch.zeros((rows, self.heads * self.dim), dtype=torch_type(self.element),
                          device=self.device)
        r, k, v, gate, rate = self.columns
        launch = qh.RecurrenceLaunch(qh.ptr(d), self.stride, r, k, v, gate, rate, self.low,
                                     qh.ptr(out), self.heads * self.dim, rows, None, None, 0,
                                     qh.ptr(workspace), size)
        qh.call("qllm_recurrence_rows", ctypes.byref(self.layer), ctypes.byref(launch), None)
        torch.cuda.synchronize()
        return out.float().cpu().numpy().astype(np.float64)

    def expected(self, projections):
        p = projections.astype(np.float64)
        rows, n = p.shape[0], self.heads * self.dim
        shape = (rows, self.heads, self.dim)
        r, k, v, gate, rate = (p[:, c:c + n] for c in self.columns)
        inner = np.tanh(p[:, self.low:self.low + self.rank]) @ self.up.T.astype(
            np.float64) + self.base
        zero = np.zeros((self.dim, self.dim))
        out = np.empty(shape)
        if self.kind == qh.RECURRENCE_DELTA:
            w = np.exp(-np.exp(-0.5) * mo.sigmoid(inner)).reshape(shape)
            a = mo.sigmoid(rate + self.bias).reshape(shape)
        else:
            w = np.exp(-np.exp(inner)).reshape(shape)
        r, k, v = (x.reshape(shape) for x in (r, k, v))
        states = []
        for h in range(self.heads):
            if self.kind == qh.RECURRENCE_DELTA:
                out[:, h], state = mo.delta_recurrence(r[:, h], k[:, h], v[:, h], w[:, h],
                                                       a[:, h], zero)
            else:
                out[:, h], state = mo.wkv_recurrence(
                    r[:, h], k[:, h], v[:, h], w[:, h],
                    self.bonus[h * self.dim:(h + 1) * self.dim].astype(np.float64), zero)
            states.append(state)
        gated = mo.sigmoid(gate) if self.kind == qh.RECURRENCE_DELTA else mo.silu(gate)
        return mo.rms(out, 1e-5).reshape(rows, n) * self.norm * gated, np.stack(states)


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("kind", [qh.RECURRENCE_DELTA, qh.RECURRENCE_BONUS])
@pytest.mark.parametrize("heads,dim,rank", [(3, 64, 16), (2, 24, 8), (1, 128, 40), (5, 16, 1),
                                            (2, 80, 64), (1, 144, 33), (7, 5, 3)])
def test_recurrences_in_portions(device, element, kind, heads, dim, rank):
    rng = np.random.default_rng(heads * dim + kind)
    layer = Recurrence(device, element, kind, heads, dim, rank, rng)
    projections = mm.bf16(rng.standard_normal((150, layer.stride)))
    projections[:, layer.columns[1]:layer.columns[2]] *= np.float32(2 / np.sqrt(dim))
    want, states = layer.expected(projections)
    at, got = 0, []
    for count in (1, 1, 2, 37, 3, 16, 64, 1, 7, 17, 1):
        got.append(layer.run(projections[at:at + count]))
        at += count
    assert at == 150
    close(np.concatenate(got), want, element, "outputs", factor=2.0)
    n = heads * dim * dim
    state = layer.state[layer.slot_stride:layer.slot_stride + n].cpu().numpy()
    close(state.reshape(heads, dim, dim).astype(np.float64), states, F32, "state", factor=4.0)
    # the other slot was not touched
    assert torch.all(layer.state[:layer.slot_stride] == 0)
    # the same prompt in one piece, in a slot that holds another request's state
    layer.state[layer.slot_stride:] = 0
    close(layer.run(projections), want, element, "whole", factor=2.0)


@pytest.mark.parametrize("element", [F32, BF16])
@pytest.mark.parametrize("kind", [qh.RECURRENCE_DELTA, qh.RECURRENCE_BONUS])
@pytest.mark.parametrize("heads,dim", [(2, 64), (1, 24), (1, 130)])
def test_recurrences_over_long_prompts(device, element, kind, heads, dim):
    rng = np.random.default_rng(dim + kind)
    layer = Recurrence(device, element, kind, heads, dim, 6, rng)
    projections = mm.bf16(rng.standard_normal((1300, layer.stride)))
    projections[:, layer.columns[1]:layer.columns[2]] *= np.float32(2 / np.sqrt(dim))
    want, states = layer.expected(projections)
    n = heads * dim * dim
    for counts in ([1300], [600, 1, 699], [100, 530, 515, 155]):
        layer.state.zero_()
        got, at = [], 0
        for count in counts:
            got.append(layer.run(projections[at:at + count]))
            at += count
        close(np.concatenate(got), want, element, str(counts), factor=2.0)
        state = layer.state[layer.slot_stride:layer.slot_stride + n].cpu().numpy()
        close(state.reshape(heads, dim, dim).astype(np.float64), states, F32, "state",
              factor=4.0)
        assert torch.all(layer.state[:layer.slot_stride] == 0)


def test_launches_turn_down_what_does_not_fit(device):
    layer = Attention(device, BF16, 4, 2, 64, 64, 32, 2, None, 0.125, context=128)
    bad = qh.RopeStoreLaunch(layer.table.data_ptr(), 8, 0, 0, 0, 0, None, None, None, None,
                             layer.table.data_ptr(), 1)
    with pytest.raises(qh.QllmError):
        qh.call("qllm_windowed_rope_store", ctypes.byref(layer.layer), ctypes.byref(bad), None)
    launch = qh.AttentionLaunch(layer.table.data_ptr(), None, 0, layer.table.data_ptr(), 256, 1,
                                100, None, 0)
    with pytest.raises(qh.QllmError, match="workspace"):
        qh.call("qllm_windowed_attention_rows", ctypes.byref(layer.layer),
                ctypes.byref(launch), None)
    segment = qh.LinearSegment(layer.table.data_ptr(), layer.table.data_ptr(),
                               layer.table.data_ptr(), 15, 64, 64, 16, 15, 0, 0, 0)
    with pytest.raises(qh.QllmError, match="segment"):
        qh.call("qllm_linear_batch", ctypes.byref(segment), 1, 1, BF16, None)
