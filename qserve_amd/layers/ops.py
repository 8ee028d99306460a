"""The operations the served models are made of, in two forms with one signature:

* `HipOps`   - the product path: one launch of libqserve_serve.so per call (include/qserve_serve.h), on the current stream;
* `TorchOps` - the same operations written with unfused torch tensor ops on any device.  It exists to bring a layer up and
  to test host logic (cache, scheduler, batching) where no GPU is; an engine only uses it when asked to by name - a model on
  a GPU never falls back to it.

Conventions: `x` is the float residual stream [T, D]; `h` and every other activation is in the storage type (bfloat16 or
float32); matrix products are the vendor's (`linear`), with float accumulation.
"""
import torch

BF16, F32 = 0, 1


def dtype_code(dtype):
    if dtype == torch.bfloat16:
        return BF16
    if dtype == torch.float32:
        return F32
    raise ValueError(f"the serving kernels store bfloat16 or float32, not {dtype}")


def linear(x, w):
    """x [T, in] @ w [out, in]^T in the storage type (hipBLASLt / rocBLAS through torch; float accumulation)."""
    return torch.matmul(x, w.t())


class HipOps:
    name = "hip"

    def __init__(self, dtype):
        from ..serving._lib import check, lib
        self.dtype, self.code = dtype, dtype_code(dtype)
        self.L, self.check = lib(), check

    @staticmethod
    def _s():
        return torch.cuda.current_stream().cuda_stream

    def _need(self, *ts):
        for t in ts:
            if t is not None and not (t.is_cuda and t.is_contiguous()):
                raise RuntimeError("serving kernels need contiguous tensors on the GPU")

    def embed(self, tokens, table):
        T, D = tokens.numel(), table.size(1)
        x = torch.empty((T, D), dtype=torch.float32, device=table.device)
        h = torch.empty((T, D), dtype=self.dtype, device=table.device)
        self._need(tokens, table)
        self.check(self.L.qsv_embed(x.data_ptr(), h.data_ptr(), table.data_ptr(), tokens.data_ptr(), T, D, self.code, self._s()),
                   "embed")
        return x, h

    def add_layer_norm(self, x, y, w, eps):
        """x += layer_norm(y) * w in place; returns x in the storage type."""
        h = torch.empty(x.shape, dtype=self.dtype, device=x.device)
        self._need(x, y, w)
        assert y.shape == x.shape and y.dtype == self.dtype and x.dtype == torch.float32
        self.check(self.L.qsv_add_layer_norm(x.data_ptr(), h.data_ptr(), y.data_ptr(), w.data_ptr(), eps, x.size(0), x.size(1),
                                             self.code, self._s()), "add_layer_norm")
        return h

    def layer_norm_rows(self, x, rows, w, eps):
        n = x.size(0) if rows is None else rows.numel()
        out = torch.empty((n, x.size(1)), dtype=self.dtype, device=x.device)
        self._need(x, rows, w)
        self.check(self.L.qsv_layer_norm_rows(out.data_ptr(), x.data_ptr(), 0 if rows is None else rows.data_ptr(), w.data_ptr(),
                                              eps, n, x.size(1), self.code, self._s()), "layer_norm_rows")
        return out

    def latent_prep(self, down, q_off, q_rank, q_w, kv_off, kv_rank, kv_w, rot_dim, rot_n, rope, pool, slot, pos, eps):
        T = down.size(0)
        cq = torch.empty((T, q_rank), dtype=self.dtype, device=down.device)
        self._need(down, q_w, kv_w, rope, pool, slot, pos)
        assert pool.size(-1) == kv_rank + rot_dim and slot.dtype == torch.int64 and pos.dtype == torch.int32
        assert rope is None or (rope.dtype == torch.float32 and rope.size(-1) * 2 == rot_n)
        self.check(self.L.qsv_latent_prep(down.data_ptr(), down.stride(0), q_off, q_rank, q_w.data_ptr(), cq.data_ptr(), kv_off,
                                          kv_rank, kv_w.data_ptr(), rot_dim, rot_n, 0 if rope is None else rope.data_ptr(),
                                          pool.data_ptr(), slot.data_ptr(), pos.data_ptr(), eps, T, self.code, self._s()),
                   "latent_prep")
        return cq

    def latent_query(self, q, q_abs, rope, pos, scale, heads, dim, rot_dim, rot_n, rank):
        T = q.size(0)
        qf = torch.empty((T, heads, rank + rot_dim), dtype=torch.float32, device=q.device)
        self._need(q, q_abs, rope, pos)
        assert q.numel() == T * heads * (dim + rot_dim) and q_abs.shape == (heads, T, rank)
        self.check(self.L.qsv_latent_query(qf.data_ptr(), q.data_ptr(), q_abs.data_ptr(), 0 if rope is None else rope.data_ptr(),
                                           pos.data_ptr(), scale, T, heads, dim, rot_dim, rot_n, rank, self.code, self._s()),
                   "latent_query")
        return qf

    attention_split_target = 512        # workgroups a launch of the matrix-core attention should at least have

    def latent_attention(self, qf, pool, batch, window, rank, page, variant=0, key_splits=None, q_first=0, chunk=None, bias=None,
                         keep_first=0, sink=None, pooled=None, pool_block=0, slopes=None):
        """batch: the step's StepBatch (block table, sequence slot and position per token, work tiles).  variant: 0 = the
        matrix-core kernel where it takes the sizes, 1 = always the wave kernel.  key_splits: None = chosen from the number
        of workgroups and the context.  q_first: the caller's promise that every query is zero before that element.
        pool [rows, R]: one pool for all heads; [G, rows, R]: head h reads pool h // (H / G), all in one launch.
        chunk: a query sees only the keys of its own chunk of that many positions.  bias: float [H, n], bias[h, min(i - j, n - 1)]
        is added to the score of query i and key j.  keep_first: the first that many positions of the sequence stay visible
        behind the window.  sink float [H]: exp(sink[h]) joins the softmax's denominator (no key, no value).  pooled (shaped like
        pool, ceil(page / pool_block) rows per page, written by `pool_blocks`): one more key / value row per block of pool_block
        positions that lies wholly before the window.  slopes float [H]: slopes[h] * (i - j) is taken off the score."""
        T, H, R = qf.shape
        assert slopes is None or (slopes.dtype == torch.float32 and slopes.numel() == H and slopes.is_contiguous() and pooled is None)
        assert sink is None or (sink.dtype == torch.float32 and sink.numel() == H and sink.is_contiguous())
        assert pooled is None or (window and pool_block > 0 and bias is None and not chunk and not keep_first and pooled.dim() == pool.dim()
                                  and pooled.dtype == pool.dtype and pooled.size(-1) == R)
        assert not keep_first or (window and not chunk)
        per_page = (page + pool_block - 1) // pool_block if pooled is not None else 0
        assert pooled is None or pooled.size(-2) == pool.size(-2) // page * per_page
        more = (int(keep_first or 0), 0 if sink is None else sink.data_ptr(), 0 if pooled is None else pooled.data_ptr(),
                0 if pooled is None or pooled.dim() == 2 else pooled.stride(0), int(pool_block) if pooled is not None else 0, per_page,
                0 if slopes is None else slopes.data_ptr())
        assert bias is None or (bias.dtype == torch.float32 and bias.dim() == 2 and bias.size(0) == H and bias.is_contiguous())
        extra = (int(chunk or 0), 0 if bias is None else bias.data_ptr(), 0 if bias is None else bias.size(1))
        block_table, seq, pos = batch.block_table, batch.seq, batch.pos
        out = torch.empty((T, H, rank), dtype=self.dtype, device=qf.device)
        self._need(qf, pool, block_table, seq, pos, pooled)
        assert pool.size(-1) == R and block_table.dtype == torch.int32 and seq.dtype == torch.int32
        per, pool_stride = (H, 0) if pool.dim() == 2 else (H // pool.size(0), pool.stride(0))
        assert pool.dim() == 2 or H % pool.size(0) == 0
        if variant == 0 and page % 32 == 0 and self.L.qsv_latent_attention_mfma_ok(rank, R, self.code):
            tiles = batch.tiles(self.L.qsv_latent_attention_tile_tokens(per))
            # few workgroups and long contexts (decoding): cut the keys over several workgroups, merged by a second launch
            groups = tiles.size(0) * (H // per) * ((per + 31) // 32)
            span = min(batch.max_pos + 1, int(window)) if window else batch.max_pos + 1
            span = min(span, int(chunk)) if chunk else span
            span += int(keep_first or 0) + (batch.max_pos // pool_block if pooled is not None else 0)
            # (rows wider than 320 elements: one workgroup per CU at a time - a launch of one round of workgroups is the aim)
            target = self.attention_split_target // 2 if R > 320 else self.attention_split_target
            splits = max(1, min(target // max(groups, 1), span // 128, 32)) if key_splits is None else key_splits
            po = pm = None
            if splits > 1:
                po = torch.empty((splits, T, H, rank), dtype=torch.float32, device=qf.device)
                pm = torch.empty((splits, T, H, 2), dtype=torch.float32, device=qf.device)
            self.check(self.L.qsv_latent_attention_mfma(out.data_ptr(), qf.data_ptr(), pool.data_ptr(), block_table.data_ptr(),
                                                        block_table.stride(0), pos.data_ptr(), tiles.data_ptr(), tiles.size(0),
                                                        int(window or 0), H, rank, R, page, splits,
                                                        0 if po is None else po.data_ptr(), 0 if pm is None else pm.data_ptr(), T,
                                                        int(q_first), per, pool_stride, *extra, *more, self._s()), "latent_attention_mfma")
            return out
        self.check(self.L.qsv_latent_attention(out.data_ptr(), qf.data_ptr(), pool.data_ptr(), block_table.data_ptr(),
                                               block_table.stride(0), seq.data_ptr(), pos.data_ptr(), int(window or 0), T, H,
                                               rank, R, page, per, pool_stride, *extra, *more, self.code, variant, self._s()),
                   "latent_attention")
        return out

    def sigmoid_gate(self, o, g):
        """o [T, n] *= sigmoid(g [T, n]) in place; g may be a column slice of a wider matrix."""
        self._need(o)
        assert g.is_cuda and g.stride(1) == 1 and g.shape == o.shape
        self.check(self.L.qsv_sigmoid_gate(o.data_ptr(), g.data_ptr(), g.stride(0), o.size(0), o.size(1), self.code, self._s()),
                   "sigmoid_gate")
        return o

    # ---- streams, position-free norm, token shift -----------------------------------------------------------------------------
    def embed_streams(self, tokens, table, scale, streams):
        T, D = tokens.numel(), table.size(1)
        x = torch.empty((T, streams, D), dtype=torch.float32, device=table.device)
        self._need(tokens, table)
        self.check(self.L.qsv_embed_streams(x.data_ptr(), table.data_ptr(), tokens.data_ptr(), float(scale), T, streams, D, self.code,
                                            self._s()), "embed_streams")
        return x

    def hc_read(self, x, w_in, norm, shift=None, batch=None, prev=None):
        """-> the sublayer's input [T, D] (storage type): norm(sum_s w_in[s] x[:, s]), token-shifted if `shift` is given (then
        `prev` is the sequences' two-copy state [2 slots, D] and `batch` names each token's run and state rows)."""
        w, b, alpha = norm
        T, S, D = x.shape
        h = torch.empty((T, D), dtype=self.dtype, device=x.device)
        self._need(x, w_in, w, b, shift, prev)
        assert x.dtype == torch.float32 and w_in.dtype == torch.float32 and w_in.numel() == S
        p = [0, 0, 0, 0, 0]
        if shift is not None:
            assert prev.dtype == torch.float32 and prev.size(-1) == D and shift.dtype == self.dtype
            p = [shift.data_ptr(), prev.data_ptr(), batch.run_off.data_ptr(), batch.state_rd.data_ptr(), batch.state_wr.data_ptr()]
        self.check(self.L.qsv_hc_read(h.data_ptr(), x.data_ptr(), w_in.data_ptr(), w.data_ptr(), b.data_ptr(), float(alpha), *p,
                                      T, S, D, self.code, self._s()), "hc_read")
        return h

    def hc_write(self, x, y, w_mix, w_out, then_read=None):
        """All streams rewritten in place from the sublayer's output y.  then_read = (w_in, norm) of the NEXT sublayer, if it
        reads without a token shift: its input comes out of the same pass -> h [T, D] (else None)."""
        T, S, D = x.shape
        self._need(x, y, w_mix, w_out)
        assert y.shape == (T, D) and y.dtype == self.dtype and w_mix.dtype == torch.float32 and w_mix.shape == (S, S)
        h, nxt = None, [0, 0, 0, 0, 0.0]
        if then_read is not None:
            w_in, (w, b, alpha) = then_read
            h = torch.empty((T, D), dtype=self.dtype, device=x.device)
            nxt = [h.data_ptr(), w_in.data_ptr(), w.data_ptr(), b.data_ptr(), float(alpha)]
        self.check(self.L.qsv_hc_write(x.data_ptr(), y.data_ptr(), w_mix.data_ptr(), w_out.data_ptr(), T, S, D, *nxt, self.code,
                                       self._s()), "hc_write")
        return h

    def dyt_sum_rows(self, x, rows, norm):
        w, b, alpha = norm
        T, S, D = x.shape
        n = T if rows is None else rows.numel()
        out = torch.empty((n, D), dtype=self.dtype, device=x.device)
        self._need(x, rows, w, b)
        self.check(self.L.qsv_dyt_sum_rows(out.data_ptr(), x.data_ptr(), 0 if rows is None else rows.data_ptr(), w.data_ptr(),
                                           b.data_ptr(), float(alpha), n, S, D, self.code, self._s()), "dyt_sum_rows")
        return out

    def rms_pair_mean(self, a, wa, b, wb, eps):
        out = torch.empty_like(a)
        self._need(a, wa, b, wb)
        assert a.shape == b.shape and a.dtype == self.dtype and b.dtype == self.dtype
        self.check(self.L.qsv_rms_pair_mean(out.data_ptr(), a.data_ptr(), wa.data_ptr(), b.data_ptr(), wb.data_ptr(), eps, a.size(0),
                                            a.size(1), self.code, self._s()), "rms_pair_mean")
        return out

    GLU_ACTS = {"silu": 0, "gelu_tanh": 1, "clamped": 2}

    def glu(self, a, act="silu", limit=0.0, row_scale=None, scale_index=None):
        """a [n, 2 ff] with (gate, up) as neighbours -> act(gate) * up [n, ff]; act: silu, gelu_tanh (gelu in its tanh form), or
        clamped: g = min(gate, limit), u = clamp(up, -limit, limit) -> g sigmoid(1.702 g) (u + 1).  row_scale (float): row r
        of a is first multiplied by row_scale[scale_index[r]] (scale_index int64, None: r)."""
        n, ff = a.size(0), a.size(1) // 2
        out = torch.empty((n, ff), dtype=self.dtype, device=a.device)
        self._need(a, row_scale, scale_index)
        assert row_scale is None or row_scale.dtype == torch.float32
        self.check(self.L.qsv_glu(out.data_ptr(), a.data_ptr(), n, ff, self.GLU_ACTS[act], float(limit),
                                  0 if row_scale is None else row_scale.data_ptr(), 0 if scale_index is None else scale_index.data_ptr(),
                                  self.code, self._s()), "glu")
        return out

    # ---- sinusoidal positions, RMS-normed residual, whole-projection query / key norms ----------------------------------------------
    def embed_sinusoid(self, tokens, pos, table, freq, scale):
        """-> float x [T, D] = table[tokens] * scale + the sinusoidal vector of each position (freq float [(D + 1) // 2])."""
        T, D = tokens.numel(), table.size(1)
        x = torch.empty((T, D), dtype=torch.float32, device=table.device)
        self._need(tokens, pos, table, freq)
        assert freq.dtype == torch.float32 and freq.numel() == (D + 1) // 2
        self.check(self.L.qsv_embed_sinusoid(x.data_ptr(), table.data_ptr(), tokens.data_ptr(), pos.data_ptr(), freq.data_ptr(),
                                             float(scale), T, D, self.code, self._s()), "embed_sinusoid")
        return x

    def add_rms_norm(self, x, ys, w, eps):
        """x += sum of ys (up to three sublayer outputs, storage type) in place; -> rms_norm(x) * w in the storage type (None if
        w is None)."""
        ys = [y for y in ys if y is not None]
        assert len(ys) <= 3 and all(y.shape == x.shape and y.dtype == self.dtype for y in ys) and x.dtype == torch.float32
        h = None if w is None else torch.empty(x.shape, dtype=self.dtype, device=x.device)
        self._need(x, w, *ys)
        p = [y.data_ptr() for y in ys] + [0] * (3 - len(ys))
        self.check(self.L.qsv_add_rms_norm(x.data_ptr(), 0 if h is None else h.data_ptr(), *p, 0 if w is None else w.data_ptr(),
                                           float(eps), x.size(0), x.size(1), self.code, self._s()), "add_rms_norm")
        return h

    def rms_norm_rows(self, x, rows, w, eps):
        """w: storage type or float."""
        n = x.size(0) if rows is None else rows.numel()
        out = torch.empty((n, x.size(1)), dtype=self.dtype, device=x.device)
        self._need(x, rows, w)
        self.check(self.L.qsv_rms_norm_rows(out.data_ptr(), x.data_ptr(), 0 if rows is None else rows.data_ptr(), w.data_ptr(),
                                            dtype_code(w.dtype), float(eps), n, x.size(1), self.code, self._s()), "rms_norm_rows")
        return out

    def scaled_sum_rms_norms(self, x, parts, gains, eps, tokens=None, table=None):
        """x += sum of scale * y over parts [(y, scale)] (up to three; y storage type, scale per coordinate in the storage type or None) in
        place, or, with tokens, x <- table[tokens] (+ the parts; x None: made here); -> (x, [rms_norm(x) * g in the storage type for the (up to
        two) float gains g]), all from one statistic."""
        assert len(parts) <= 3 and len(gains) <= 2
        if tokens is not None and x is None:
            x = torch.empty((tokens.numel(), table.size(1)), dtype=torch.float32, device=table.device)
        T, D = x.shape
        hs = [torch.empty((T, D), dtype=self.dtype, device=x.device) for _ in gains]
        self._need(x, tokens, table, *gains, *[v for p in parts for v in p])
        assert x.dtype == torch.float32 and all(g.dtype == torch.float32 and g.numel() == D for g in gains)
        for y, s in parts:
            assert y.shape == x.shape and y.dtype == self.dtype and (s is None or (s.dtype == self.dtype and s.numel() == D))
        p = [0 if v is None else v.data_ptr() for part in parts for v in part] + [0] * (6 - 2 * len(parts))
        hp, gp = ([v.data_ptr() for v in vs] + [0] * (2 - len(vs)) for vs in (hs, gains))
        self.check(self.L.qsv_scaled_sum_rms_norms(x.data_ptr(), *hp, *p, *gp, 0 if tokens is None else tokens.data_ptr(),
                                                   0 if table is None else table.data_ptr(), float(eps), T, D, self.code, self._s()),
                   "scaled_sum_rms_norms")
        return x, hs

    def normed_attention_prep(self, proj, q_off, k_off, v_off, heads, kv_heads, dim, vdim, q_w, k_w, eps, scale, v_first, mix, pool,
                              batch):
        """-> float queries [T, heads, vdim + dim] = [0 | normed q * scale]; writes the cache rows [v' | normed k] of the step's
        tokens.  v_first: [T, kv_heads * vdim] (a column slice is fine) or None; mix: the blend's weight on v_first."""
        T = proj.size(0)
        qf = torch.empty((T, heads, vdim + dim), dtype=torch.float32, device=proj.device)
        self._need(proj, q_w, k_w, pool, batch.slot)
        assert pool.shape[0] == kv_heads and pool.shape[2] == vdim + dim and pool.dtype == self.dtype and proj.dtype == self.dtype
        assert v_first is None or (v_first.dtype == self.dtype and v_first.stride(1) == 1 and v_first.shape == (T, kv_heads * vdim))
        self.check(self.L.qsv_normed_attention_prep(qf.data_ptr(), pool.data_ptr(), pool.size(1), proj.data_ptr(), proj.stride(0),
                                                    q_off, k_off, v_off, heads, kv_heads, dim, vdim, q_w.data_ptr(), k_w.data_ptr(),
                                                    float(eps), float(scale), 0 if v_first is None else v_first.data_ptr(),
                                                    0 if v_first is None else v_first.stride(0), float(mix), batch.slot.data_ptr(),
                                                    T, self.code, self._s()), "normed_attention_prep")
        return qf

    def max_gates(self, proj, i_off, f_off, bias_i, bias_f, cap, m_state, batch, heads):
        """Exponential gates with a running maximum from the pre-activations proj[:, i_off : i_off + heads] / [f_off : ...]; m_state
        float [slots, heads].  -> (decay a, input scale b, maximum m), float [T, heads] each."""
        T = proj.size(0)
        a, b, m = (torch.empty((T, heads), dtype=torch.float32, device=proj.device) for _ in range(3))
        self._need(bias_i, bias_f, m_state)
        assert proj.stride(1) == 1 and proj.dtype == self.dtype and bias_i.dtype == bias_f.dtype == m_state.dtype == torch.float32
        assert m_state.shape[1:] == (heads,) and bias_i.numel() == bias_f.numel() == heads
        runs = batch.runs()
        el = proj.element_size()
        self.check(self.L.qsv_max_gates(a.data_ptr(), b.data_ptr(), m.data_ptr(), proj.data_ptr() + i_off * el,
                                        proj.data_ptr() + f_off * el, proj.stride(0), bias_i.data_ptr(), bias_f.data_ptr(), float(cap),
                                        m_state.data_ptr(), runs.data_ptr(), runs.size(0), heads, self.code, self._s()), "max_gates")
        return a, b, m

    # ---- attention with rotated keys and values: rotations + cache write ---------------------------------------------------------
    def attention_prep(self, proj, q_off, k_off, v_off, heads, kv_heads, dim, vdim, rot_n, rope_k, rope_v, scale, pool, batch):
        T = proj.size(0)
        qf = torch.empty((T, heads, vdim + dim), dtype=torch.float32, device=proj.device)
        self._need(proj, rope_k, rope_v, pool, batch.slot, batch.pos)
        assert pool.shape[0] == kv_heads and pool.shape[2] == vdim + dim and pool.dtype == self.dtype and proj.dtype == self.dtype
        assert rope_k.size(-1) * 2 == rot_n and rope_v.size(-1) * 2 == vdim and rope_k.size(0) > batch.max_pos < rope_v.size(0)
        self.check(self.L.qsv_attention_prep(qf.data_ptr(), pool.data_ptr(), pool.size(1), proj.data_ptr(), proj.stride(0), q_off,
                                             k_off, v_off, heads, kv_heads, dim, vdim, rot_n, rope_k.data_ptr(), rope_v.data_ptr(),
                                             float(scale), batch.slot.data_ptr(), batch.pos.data_ptr(), T, self.code, self._s()),
                   "attention_prep")
        return qf

    def rotate_heads(self, o, rope, pos, sign):
        T, H, n = o.shape
        self._need(o, rope, pos)
        assert rope.size(-1) * 2 == n and o.dtype == self.dtype
        self.check(self.L.qsv_rotate_heads(o.data_ptr(), rope.data_ptr(), pos.data_ptr(), float(sign), T, H, n, self.code, self._s()),
                   "rotate_heads")
        return o


    # ---- sandwich norms, sink / kept-first / pooled-block attention, element-wise gated recurrence -----------------------------------
    def add_normed_rms_norm(self, x, y, w_post, w_next, eps):
        """x += rms_norm(y) * w_post in place (y None: nothing is added); -> rms_norm(x) * w_next in the storage type (None if
        w_next is None).  The weights hold one number (a gain for all coordinates) or one per coordinate."""
        T, D = x.shape
        h = None if w_next is None else torch.empty((T, D), dtype=self.dtype, device=x.device)
        self._need(x, y, w_post, w_next)
        assert x.dtype == torch.float32 and (y is None or (y.shape == x.shape and y.dtype == self.dtype and w_post is not None))
        for w in (w_post, w_next):
            assert w is None or (w.dtype == self.dtype and w.numel() in (1, D))
        self.check(self.L.qsv_add_normed_rms_norm(x.data_ptr(), 0 if h is None else h.data_ptr(), 0 if y is None else y.data_ptr(),
                                                  0 if y is None else w_post.data_ptr(), int(y is not None and w_post.numel() != 1),
                                                  0 if w_next is None else w_next.data_ptr(),
                                                  int(w_next is not None and w_next.numel() != 1), float(eps), T, D, self.code,
                                                  self._s()), "add_normed_rms_norm")
        return h

    def relu_sq(self, a):
        """a <- relu(a)^2 in place."""
        self._need(a)
        self.check(self.L.qsv_relu_sq(a.data_ptr(), a.numel(), self.code, self._s()), "relu_sq")
        return a

    def qk_norm_rope_prep(self, q, k, v, heads, kv_heads, dim, vdim, q_w, k_w, per_head, eps, rope, rot_n, scale, pool, batch,
                          q_b=None, k_b=None, v_b=None, halves=False, head_scale=None, q_pad=None, rot_gain=0.0, q_store=False):
        """q [T, heads * dim], k [T, kv_heads * dim], v [T, kv_heads * vdim] (float or storage type, column slices are fine; k and v
        None: the layer caches nothing; v may be k itself: values that are the projected keys).  q_b, k_b, v_b (one per channel) are added
        first.  Queries and keys are RMS-normed per head (weight [dim], shared by the heads) or over the whole projection (weight as wide
        as it), then the first rot_n dimensions of every head turn with the position (pairs of neighbours, or with `halves` (i, i + rot_n
        / 2); rope float [positions, 2, rot_n / 2] or None).  -> float queries [T, heads, q_pad + dim] = [0 | q * scale *
        head_scale[h]] (q_pad None: vdim); writes the cache rows [v | k] of the step's tokens into pool [kv_heads, rows, vdim + dim].
        q_w = k_w = None: norms (per head) without weights; rot_gain > 0: those norms follow the rotation, whose cos and sin carry the
        magnitude sqrt(rot_gain); q_store: the queries come in the storage type."""
        T = q.size(0)
        q_pad = vdim if q_pad is None else int(q_pad)
        qf = torch.empty((T, heads, q_pad + dim), dtype=self.dtype if q_store else torch.float32, device=q.device)
        self._need(q_w, k_w, rope, pool, batch.slot, batch.pos, q_b, k_b, v_b, head_scale)
        assert q.stride(1) == 1 and q.size(1) == heads * dim and (per_head or q_w is not None) and (k is None or (q_w is None) == (k_w is None))
        assert q_w is None or (q_w.dtype == self.dtype and q_w.numel() == (dim if per_head else heads * dim))
        assert rope is None or (rope.dtype == torch.float32 and rope.size(-1) * 2 == rot_n and rot_n <= dim and rope.size(0) > batch.max_pos)
        for b, n in ((q_b, heads * dim), (k_b, kv_heads * dim), (v_b, kv_heads * vdim)):
            assert b is None or (b.dtype == self.dtype and b.numel() == n)
        assert head_scale is None or (head_scale.dtype == torch.float32 and head_scale.numel() == heads)
        kp = [0, 0, 0, 0, 0, 0, 0]
        if k is not None:
            assert k.dtype == v.dtype == q.dtype and k.stride(1) == v.stride(1) == 1 and k.size(1) == kv_heads * dim
            assert v.size(1) == kv_heads * vdim
            assert k_w is None or (k_w.dtype == self.dtype and k_w.numel() == (dim if per_head else kv_heads * dim))
            assert pool.shape[0] == kv_heads and pool.shape[2] == vdim + dim and pool.dtype == self.dtype
            kp = [k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0), 0 if k_w is None else k_w.data_ptr(), pool.data_ptr(), pool.size(1)]
        opt = [0 if b is None else b.data_ptr() for b in (q_b, k_b, v_b)]
        self.check(self.L.qsv_qk_norm_rope_prep(qf.data_ptr(), q.data_ptr(), q.stride(0), *kp[:4], dtype_code(q.dtype), heads, kv_heads,
                                                dim, vdim, 0 if q_w is None else q_w.data_ptr(), kp[4], int(bool(per_head)), float(eps),
                                                0 if rope is None else rope.data_ptr(), int(rot_n if rope is not None else 0),
                                                float(scale), kp[5], kp[6], batch.slot.data_ptr(), batch.pos.data_ptr(), T, *opt,
                                                int(bool(halves)), 0 if head_scale is None else head_scale.data_ptr(), q_pad,
                                                float(rot_gain), int(bool(q_store)), self.code,
                                                self._s()), "qk_norm_rope_prep")
        return qf

    def pool_blocks(self, pool, pooled, batch, block, page):
        """For every token of the step that completes a block of `block` positions: the mean of the block's cache rows (as the pool
        holds them) goes into `pooled` [kv_heads, pages * ceil(page / block), row]: the block that starts in page p at offset o
        has row p * ceil(page / block) + o // block."""
        per_page = (page + block - 1) // block
        self._need(pool, pooled, batch.block_table, batch.seq, batch.pos)
        assert pool.dim() == 3 and pooled.dim() == 3 and pooled.size(0) == pool.size(0) and pooled.size(2) == pool.size(2)
        assert pooled.size(1) == pool.size(1) // page * per_page and pooled.dtype == pool.dtype == self.dtype
        self.check(self.L.qsv_pool_blocks(pooled.data_ptr(), pooled.size(1), pool.data_ptr(), pool.size(1), batch.block_table.data_ptr(),
                                          batch.block_table.stride(0), batch.seq.data_ptr(), batch.pos.data_ptr(), batch.n_tokens,
                                          pool.size(0), pool.size(2), int(block), int(page), per_page, self.code, self._s()),
                   "pool_blocks")

    def min_gru_scan(self, proj, z_off, x_off, g_off, b_z, b_x, state, batch, width):
        """Element-wise gated recurrence S <- (1 - z) S + z c with z = sigmoid(proj[:, z_off ..] + b_z), c = u + 1/2 (u >= 0) or
        sigmoid(u) (u < 0), u = proj[:, x_off ..] + b_x; state float [slots, width].  -> S * silu(proj[:, g_off ..]) [T, width]."""
        T = proj.size(0)
        out = torch.empty((T, width), dtype=self.dtype, device=proj.device)
        self._need(b_z, b_x, state)
        assert proj.stride(1) == 1 and proj.dtype == self.dtype and b_z.dtype == b_x.dtype == self.dtype and state.dtype == torch.float32
        assert state.shape[1:] == (width,) and b_z.numel() == b_x.numel() == width and max(z_off, x_off, g_off) + width <= proj.size(1)
        runs = batch.runs()
        self.check(self.L.qsv_min_gru_scan(out.data_ptr(), proj.data_ptr(), proj.stride(0), z_off, x_off, g_off, b_z.data_ptr(),
                                           b_x.data_ptr(), state.data_ptr(), runs.data_ptr(), runs.size(0),
                                           max(n for _, _, n in batch.items), width, self.code, self._s()), "min_gru_scan")
        return out

    # ---- norm after the sum, convolved mixer input, talking-heads attention, retention operands -----------------------------------------
    def embed_rms_norm(self, tokens, table, w, eps):
        """-> float x [T, D] = rms_norm(table[tokens]) * w."""
        T, D = tokens.numel(), table.size(1)
        x = torch.empty((T, D), dtype=torch.float32, device=table.device)
        self._need(tokens, table, w)
        self.check(self.L.qsv_embed_rms_norm(x.data_ptr(), table.data_ptr(), tokens.data_ptr(), w.data_ptr(), float(eps), T, D, self.code,
                                             self._s()), "embed_rms_norm")
        return x

    def residual_conv(self, x, conv_w, hist, batch):
        """-> [T, D] (storage type): x plus its causal convolution over time with per-channel taps conv_w float [taps, D]; hist: two-copy
        state, the last taps - 1 rows of x of every sequence (None with one tap)."""
        T, D = x.shape
        h = torch.empty((T, D), dtype=self.dtype, device=x.device)
        self._need(x, conv_w, hist)
        assert x.dtype == torch.float32 and conv_w.dtype == torch.float32 and conv_w.size(1) == D
        assert conv_w.size(0) == 1 or (hist.dtype == torch.float32 and hist.shape[1:] == (conv_w.size(0) - 1, D))
        self.check(self.L.qsv_residual_conv(h.data_ptr(), x.data_ptr(), conv_w.data_ptr(), conv_w.size(0), 0 if hist is None else hist.data_ptr(),
                                            batch.run_off.data_ptr(), batch.state_rd.data_ptr(), batch.state_wr.data_ptr(), T, D, self.code,
                                            self._s()), "residual_conv")
        return h

    def scaled_add_rms_norm(self, x, y, alpha, w, eps, then_conv=None, batch=None, want_h=True):
        """x <- rms_norm(alpha x + y) * w in place; -> x in the storage type (None without want_h).  then_conv = (conv_w, hist): -> what
        `residual_conv` makes of the new x, in the same launch (steps in which every run is one token)."""
        T, D = x.shape
        h = torch.empty((T, D), dtype=self.dtype, device=x.device) if want_h else None
        self._need(x, y, w)
        assert x.dtype == torch.float32 and y.shape == x.shape and y.dtype == self.dtype and w.dtype == self.dtype and w.numel() == D
        c = [0, 0, 0, 0, 0]
        if then_conv is not None:
            conv_w, hist = then_conv
            self._need(conv_w, hist)
            assert want_h and all(n == 1 for _, _, n in batch.items) and conv_w.dtype == torch.float32 and conv_w.size(1) == D
            assert conv_w.size(0) == 1 or (hist.dtype == torch.float32 and hist.shape[1:] == (conv_w.size(0) - 1, D))
            c = [conv_w.data_ptr(), conv_w.size(0), 0 if hist is None else hist.data_ptr(), batch.state_rd.data_ptr(), batch.state_wr.data_ptr()]
        self.check(self.L.qsv_scaled_add_rms_norm(x.data_ptr(), 0 if h is None else h.data_ptr(), y.data_ptr(), float(alpha), w.data_ptr(),
                                                  float(eps), *c, T, D, self.code, self._s()), "scaled_add_rms_norm")
        return h

    def rotate_qk(self, qkv, heads, dim, vdim, rope, rot_n, batch):
        """qkv [T, >= heads * (2 dim + vdim)] = [q | k | v ..] -> float [T, heads * (2 dim + vdim)] with the first rot_n dimensions of every
        q and k head turned by the position (halves layout)."""
        T = qkv.size(0)
        out = torch.empty((T, heads * (2 * dim + vdim)), dtype=torch.float32, device=qkv.device)
        self._need(rope, batch.pos)
        assert qkv.stride(1) == 1 and qkv.dtype == self.dtype and (rope is None or rope.size(0) > batch.max_pos)
        self.check(self.L.qsv_rotate_qk(out.data_ptr(), qkv.data_ptr(), qkv.stride(0), heads, dim, vdim, 0 if rope is None else rope.data_ptr(),
                                        int(rot_n if rope is not None else 0), batch.pos.data_ptr(), T, self.code, self._s()), "rotate_qk")
        return out

    talking_score_bytes = 1 << 30       # the most memory kept scores may take
    talking_split_targets = (512, 256)  # workgroups the two passes should at least have (few tiles: the keys are cut over several)

    def talking_attention(self, qf, pool, batch, talk, gate, vdim, page, cap=0.0, window=None, variant=0, key_splits=None, decode=None):
        """qf float [T, H, dim] (scaled queries), pool [G, rows, vdim + dim] -> [T, H * vdim]: softmax weights per head (scores soft-capped
        by cap tanh(. / cap) if cap > 0), mixed over the heads by talk [H, H], on each head's own values; head h times sigmoid(gate[t,
        h]) (gate [T, H], a column slice is fine, or None).  variant: 0 = weights mixed before the sum (two passes) where the kernel takes
        the sizes, else 2; 2 = mixed after the sum on the matrix cores where they take the sizes, else 1; 1 = the wave kernel.
        decode: the form for few tokens per sequence (None: chosen): the first of two passes keeps the scores, or (variant 2) a workgroup
        serves the heads of several key pools."""
        T, H, dim = qf.shape
        G, R = pool.size(0), pool.size(2)
        self._need(qf, pool, batch.block_table, batch.seq, batch.pos, talk)
        assert R == vdim + dim and H % G == 0 and qf.dtype == torch.float32 and pool.dtype == self.dtype and talk.shape == (H, H)
        assert talk.dtype == self.dtype and (gate is None or (gate.dtype == self.dtype and gate.stride(1) == 1 and gate.shape == (T, H)))
        out = torch.empty((T, H * vdim), dtype=self.dtype, device=qf.device)
        bt = batch.block_table
        splits, pm = 1, None
        span = min(batch.max_pos + 1, int(window)) if window else batch.max_pos + 1
        if variant == 0 and self.L.qsv_talking_two_pass_ok(H, G, dim, vdim, page, self.code):
            tiles = batch.tiles(self.L.qsv_talking_two_pass_tile_tokens())
            n = tiles.size(0)
            s1, s2 = (max(1, min(t // max(n, 1), span // 128, 32)) for t in self.talking_split_targets) if key_splits is None else (key_splits,) * 2
            pm = torch.empty((s1, T, H, 2), dtype=torch.float32, device=qf.device)
            po = torch.empty((s2, T, H, vdim), dtype=torch.float32, device=qf.device) if s2 > 1 else None
            # few tokens per sequence: keys are read once, their scores kept (a fraction of the cache's bytes) for the second pass
            ctx = (batch.max_pos + 32) // 32 * 32
            keep = T * H * ctx * 4 <= self.talking_score_bytes and (T <= 2 * len(batch.items) if decode is None else decode)
            sc = torch.empty((T, H, ctx), dtype=torch.float32, device=qf.device) if keep else None
            self.check(self.L.qsv_talking_two_pass(out.data_ptr(), 0 if po is None else po.data_ptr(), pm.data_ptr(), qf.data_ptr(), pool.data_ptr(),
                                                   bt.data_ptr(), bt.stride(0), batch.pos.data_ptr(), tiles.data_ptr(), n, int(window or 0), T, H,
                                                   G, dim, page, pool.stride(0), float(cap), talk.data_ptr(), 0 if gate is None else gate.data_ptr(),
                                                   0 if gate is None else gate.stride(0), s1, s2, 0 if sc is None else sc.data_ptr(),
                                                   ctx, self._s()), "talking_two_pass")
            return out
        if variant != 1 and self.L.qsv_talking_attention_mfma_ok(dim, vdim, page, self.code):
            if decode is None:
                decode = T <= 2 * len(batch.items)
            kp = self.L.qsv_talking_attention_key_pools(H, G, dim, int(decode))
            tiles = batch.tiles(self.L.qsv_talking_attention_tile_tokens(H, G, kp))
            groups = tiles.size(0) * (G // kp)
            splits = max(1, min(self.attention_split_target // max(groups, 1), span // 128, 32)) if key_splits is None else key_splits
            po = torch.empty((splits, T, H, G, vdim), dtype=torch.float32, device=qf.device)
            pm = torch.empty((splits, T, H, 2), dtype=torch.float32, device=qf.device)
            self.check(self.L.qsv_talking_attention_mfma(po.data_ptr(), pm.data_ptr(), qf.data_ptr(), pool.data_ptr(), bt.data_ptr(), bt.stride(0),
                                                         batch.pos.data_ptr(), tiles.data_ptr(), tiles.size(0), int(window or 0), T, H, G, dim,
                                                         vdim, page, pool.stride(0), float(cap), kp, splits, self._s()), "talking_attention_mfma")
        else:
            po = torch.empty((1, T, H, G, vdim), dtype=torch.float32, device=qf.device)
            self.check(self.L.qsv_talking_attention(po.data_ptr(), qf.data_ptr(), pool.data_ptr(), bt.data_ptr(), bt.stride(0),
                                                    batch.seq.data_ptr(), batch.pos.data_ptr(), int(window or 0), T, H, G, dim, vdim, page,
                                                    pool.stride(0), float(cap), self.code, self._s()), "talking_attention")
        self.check(self.L.qsv_talking_mix(out.data_ptr(), po.data_ptr(), 0 if pm is None else pm.data_ptr(), talk.data_ptr(),
                                          0 if gate is None else gate.data_ptr(), 0 if gate is None else gate.stride(0), splits, T, H, G, vdim,
                                          self.code, self._s()), "talking_mix")
        return out

    # ---- attention with two key maps over the same values ----------------------------------------------------------------------------
    def conv_heads_cache(self, proj, conv_w, hist, batch, q_channels, kv_heads, key_width, vdim, pool, scale, temperature=None):
        """proj [T, >= C] = [q (q_channels) | k (kv_heads * key_width) | v (kv_heads * vdim) | ..]: a causal convolution over time on each of
        these C channels (conv_w float [taps, C]; hist: two-copy state, the last taps - 1 projected rows, None with one tap).  -> q [T,
        q_channels] (storage type) times scale and, with temperature = (coef, every), times 1 + coef ln(floor((p + 1) / every) + 1); [v | k] go
        into the cache rows of pool [kv_heads, rows, vdim + key_width] (kv_heads 0: queries only)."""
        T, (taps, C) = proj.size(0), conv_w.shape
        q = torch.empty((T, q_channels), dtype=self.dtype, device=proj.device)
        self._need(conv_w, hist, pool, batch.slot, batch.pos, batch.run_off, batch.state_rd, batch.state_wr)
        assert C == q_channels + kv_heads * (key_width + vdim) <= proj.size(1) and proj.stride(1) == 1 and proj.dtype == self.dtype
        assert conv_w.dtype == torch.float32 and (taps == 1 or (hist.dtype == torch.float32 and hist.shape[1:] == (taps - 1, C)))
        assert not kv_heads or (pool.dtype == self.dtype and pool.size(0) == kv_heads and pool.size(2) == vdim + key_width)
        coef, every = temperature if temperature is not None else (0.0, 0.0)
        self.check(self.L.qsv_conv_heads_cache(q.data_ptr(), pool.data_ptr() if kv_heads else 0, pool.size(1) if kv_heads else 0, proj.data_ptr(),
                                               proj.stride(0), conv_w.data_ptr(), taps, 0 if hist is None else hist.data_ptr(),
                                               batch.run_off.data_ptr(), batch.state_rd.data_ptr(), batch.state_wr.data_ptr(),
                                               batch.slot.data_ptr(), batch.pos.data_ptr(), q_channels, kv_heads, key_width, vdim, float(scale),
                                               float(coef), float(every), T, self.code, self._s()), "conv_heads_cache")
        return q

    step_split_target = 256             # workgroups a launch of the step kernel should at least have (one per CU)

    def maps_attention_ok(self, dim, vdim, maps, page):
        """Whether the matrix-core kernels of one or two key maps take these sizes."""
        return bool(self.L.qsv_maps_attention_ok(dim, vdim, maps, page, self.code))

    def single_map_attention(self, q, pool, batch, heads, dim, vdim, page, key_splits=None):
        """q [T, heads * dim] (storage type, scaled), pool [G, rows, vdim + dim] of rows [v | k]: causal softmax attention -> [T, heads * vdim];
        only for sizes that `maps_attention_ok` takes."""
        T = q.size(0)
        self._need(q, pool, batch.block_table, batch.pos)
        assert q.numel() == T * heads * dim and q.dtype == self.dtype == pool.dtype and pool.size(2) == vdim + dim and heads % pool.size(0) == 0
        out = torch.empty((T, heads * vdim), dtype=self.dtype, device=q.device)
        return self._maps_attention(out, q, pool, batch, heads, dim, vdim, 1, page, (0.0, 1.0, 0.0, 0, 0), key_splits)

    def _maps_attention(self, out, q, pool, batch, heads, dim, vdim, maps, page, epilogue, key_splits):
        G, bt = pool.size(0), batch.block_table
        per = heads // G
        prompt, step = batch.split_tiles(self.L.qsv_maps_attention_tile_tokens(per))
        groups, n = G * self.L.qsv_maps_attention_head_groups(per), step.size(0)
        splits, po, pm = 1, None, None
        if n:                                                # few workgroups and long contexts: the keys are cut over several
            splits = max(1, min(self.step_split_target // (n * groups), (batch.max_pos + 1) // 256, 64)) if key_splits is None else key_splits
        if splits > 1:
            po = torch.empty((splits, n, groups, 32, maps, vdim), dtype=torch.float32, device=q.device)
            pm = torch.empty((splits, n, groups, 32, maps, 2), dtype=torch.float32, device=q.device)
        self.check(self.L.qsv_maps_attention(out.data_ptr(), q.data_ptr(), pool.data_ptr(), bt.data_ptr(), bt.stride(0), batch.pos.data_ptr(),
                                             prompt.data_ptr() if prompt.size(0) else 0, prompt.size(0), step.data_ptr() if n else 0, n, heads, G,
                                             dim, vdim, maps, page, pool.stride(0), *epilogue, splits, 0 if po is None else po.data_ptr(),
                                             0 if pm is None else pm.data_ptr(), self._s()), "maps_attention")
        return out

    def diff_attention(self, q, pool, batch, heads, dim, vdim, lam, out_scale, eps, gate, page, variant=0, key_splits=None):
        """q [T, heads * 2 * dim] (storage type, scaled; per head map 1, map 2), pool [G, rows, vdim + 2 dim] of rows [v | k_1 | k_2]: with a_m the
        softmax attention of map m over the keys up to the token, o = a_1 - lam a_2; -> o / sqrt(mean(o^2) + eps) * out_scale * sigmoid(gate) [T,
        heads * vdim] (gate [T, heads * vdim], a column slice is fine, or None).  variant: 0 = the matrix-core kernels where they take the
        sizes, 1 = the wave kernel."""
        T, G = q.size(0), pool.size(0)
        self._need(q, pool, batch.block_table, batch.seq, batch.pos)
        assert q.shape == (T, heads * 2 * dim) and q.dtype == self.dtype == pool.dtype and pool.size(2) == vdim + 2 * dim and heads % G == 0
        assert gate is None or (gate.dtype == self.dtype and gate.stride(1) == 1 and gate.shape == (T, heads * vdim))
        out = torch.empty((T, heads * vdim), dtype=self.dtype, device=q.device)
        bt, ep = batch.block_table, (float(lam), float(out_scale), float(eps), 0 if gate is None else gate.data_ptr(), 0 if gate is None else gate.stride(0))
        if variant == 0 and self.maps_attention_ok(dim, vdim, 2, page) and (gate is None or (gate.stride(0) % 4 == 0 and gate.data_ptr() % 8 == 0)):
            return self._maps_attention(out, q, pool, batch, heads, dim, vdim, 2, page, ep, key_splits)
        self.check(self.L.qsv_diff_attention(out.data_ptr(), q.data_ptr(), pool.data_ptr(), bt.data_ptr(), bt.stride(0), batch.seq.data_ptr(),
                                             batch.pos.data_ptr(), T, heads, G, dim, vdim, page, pool.stride(0), *ep, self.code, self._s()),
                   "diff_attention")
        return out

    # ---- recurrences ----------------------------------------------------------------------------------------------------------
    def decay(self, z, bias, a_log, tau, heads, dim):
        """z [T, heads * dim] (storage type; a column slice is fine) -> float decays: a_log given: exp(-exp(a_log[h]) softplus(z +
        bias)); else sigmoid(z + bias)^(1 / tau)."""
        T = z.size(0)
        out = torch.empty((T, heads * dim), dtype=torch.float32, device=z.device)
        self._need(bias, a_log)
        assert z.stride(1) == 1 and z.size(1) == heads * dim and z.dtype == self.dtype and bias.dtype == self.dtype
        assert a_log is None or (a_log.dtype == torch.float32 and a_log.numel() == heads)
        self.check(self.L.qsv_decay(out.data_ptr(), z.data_ptr(), z.stride(0), bias.data_ptr(), 0 if a_log is None else a_log.data_ptr(),
                                    float(tau), T, heads, dim, self.code, self._s()), "decay")
        return out

    def conv_silu_unit(self, proj, off, conv_w, hist, batch, n_unit, unit_dim, act="silu"):
        """Causal convolution over time of the columns [off, off + C) of proj with per-channel taps conv_w [C, taps], then silu
        (act "none": nothing), then the first n_unit groups of unit_dim channels made unit vectors.  hist: two-copy state, the last
        taps - 1 inputs of every sequence.  -> float [T, C]."""
        T = proj.size(0)
        C, taps = conv_w.shape
        out = torch.empty((T, C), dtype=torch.float32, device=proj.device)
        self._need(conv_w, hist)
        assert proj.is_cuda and proj.stride(1) == 1 and off + C <= proj.size(1)
        assert conv_w.dtype == torch.float32 and hist.dtype == torch.float32 and hist.size(-1) == C and proj.dtype == self.dtype
        assert hist.size(1) == max(taps - 1, 1)
        self.check(self.L.qsv_conv_silu_unit(out.data_ptr(), proj.data_ptr(), proj.stride(0), off, C, taps, conv_w.data_ptr(),
                                             hist.data_ptr(), batch.run_off.data_ptr(), batch.state_rd.data_ptr(),
                                             batch.state_wr.data_ptr(), n_unit, unit_dim, {"none": 0, "silu": 1}[act], T, self.code, self._s()),
                   "conv_silu_unit")
        return out

    def recurrent_scan(self, q, k, v, decay, beta, state, batch, heads, qk_heads, dim, vdim, q_scale, kscale=None, v_cols=None):
        """q, k [T, qk_heads * dim], v [T, heads * vdim] (float or storage type, column slices are fine), decay float [T, heads *
        dim], beta [T, heads] raw (before the sigmoid) or None, state float [slots, heads, dim, vdim] -> o float [T, heads, vdim].
        decay of shape [T, heads]: one factor per head; of shape [heads]: the same for every token.  kscale float [T, heads]: multiplies k where it enters the state.
        v_cols < vdim: v is [T, heads * v_cols] and the state's column v_cols is fed with ones (a normaliser), the rest with zeros."""
        T = q.size(0)
        o = torch.empty((T, heads, vdim), dtype=torch.float32, device=q.device)
        self._need(decay, state, kscale)
        assert q.dtype == k.dtype == v.dtype and q.stride(1) == k.stride(1) == v.stride(1) == 1
        head_decay = 2 if decay.dim() == 1 else int(decay.shape == (T, heads) and dim != 1)
        assert decay.dtype == torch.float32 and (decay.dim() != 1 or decay.numel() == heads)
        assert state.shape[1:] == (heads, dim, vdim) and state.dtype == torch.float32 and (head_decay or decay.shape == (T, heads * dim))
        assert kscale is None or (kscale.dtype == torch.float32 and kscale.shape == (T, heads))
        assert v.size(1) == heads * (v_cols or vdim)
        runs = batch.runs()
        self.check(self.L.qsv_recurrent_scan(o.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
                                             v.stride(0), dtype_code(q.dtype), decay.data_ptr(),
                                             0 if beta is None else beta.data_ptr(), 0 if beta is None else beta.stride(0),
                                             0 if beta is None else dtype_code(beta.dtype), state.data_ptr(), runs.data_ptr(),
                                             runs.size(0), max(n for _, _, n in batch.items), heads, qk_heads, dim, vdim,
                                             float(q_scale), 0 if kscale is None else kscale.data_ptr(), head_decay,
                                             int(v_cols or 0), self._s()), "recurrent_scan")
        return o

    def head_rms_gate(self, o, w, gate, kind, eps, vdim=None, den_m=None):
        """o float [T, H, n] -> [T, H * vdim] (storage type): per head o[..., :vdim] / its root mean square * w * gate_fn(gate).
        w [vdim] (shared by the heads) or [H * vdim].  den_m float [T, H] (then n > vdim): the read-out is first divided by
        max(|o[..., vdim]|, exp(-den_m)) + 1e-6."""
        T, H, n = o.shape
        dv = n if vdim is None else vdim
        out = torch.empty((T, H * dv), dtype=self.dtype, device=o.device)
        self._need(o, w, den_m)
        assert gate.stride(1) == 1 and gate.size(1) == H * dv and gate.dtype == self.dtype and w.dtype == self.dtype
        assert w.numel() in (dv, H * dv) and (den_m is None or (n > dv and den_m.shape == (T, H) and den_m.dtype == torch.float32))
        self.check(self.L.qsv_head_rms_gate(out.data_ptr(), o.data_ptr(), w.data_ptr(), gate.data_ptr(), gate.stride(0),
                                            {"silu": 0, "sigmoid": 1}[kind], eps, T, H, dv, n, int(w.numel() != dv),
                                            0 if den_m is None else den_m.data_ptr(), self.code, self._s()), "head_rms_gate")
        return out

    def moe_route(self, h, router, top_k, groups, keep, bias=None, renorm=False, score="softmax", correction=None, group_top=1,
                  scale=1.0):
        """-> (expert indices int32 [T, top_k], weights float [T, top_k]).  score: softmax over all experts, or sigmoid per expert;
        correction float [E]: added to the scores for the CHOICE only; group_top: a group's score is its largest choice score (1)
        or the sum of its two largest (2); weights = the chosen experts' scores (renorm: divided by their sum) times scale."""
        T, E = h.size(0), router.size(0)
        idx = torch.empty((T, top_k), dtype=torch.int32, device=h.device)
        wt = torch.empty((T, top_k), dtype=torch.float32, device=h.device)
        self._need(h, router, bias, correction)
        assert bias is None or (bias.dtype == self.dtype and bias.numel() == E)
        assert correction is None or (correction.dtype == torch.float32 and correction.numel() == E)
        self.check(self.L.qsv_moe_route(idx.data_ptr(), wt.data_ptr(), h.data_ptr(), router.data_ptr(),
                                        0 if bias is None else bias.data_ptr(), int(bool(renorm)), T, h.size(1), E, top_k,
                                        groups, keep, {"softmax": 0, "sigmoid": 1}[score],
                                        0 if correction is None else correction.data_ptr(), int(group_top), float(scale),
                                        self.code, self._s()), "moe_route")
        return idx, wt

    ACTS = {"none": 0, "relu_sq": 1, "swiglu": 2, "clamped_glu": 3}

    def moe_experts(self, h, up, down, idx, wt, act="relu_sq", limit=0.0, weigh="output"):
        """up [E, rows, D], down [E, D, ff]; y[t] = sum_k wt[t, k] * down[idx[t, k]] a(up[idx[t, k]] h[t]).  act "relu_sq":
        a = relu(.)^2, rows = ff; "swiglu": up's rows come in pairs (2f = gate, 2f + 1 = up), a_f = silu(gate_f) up_f, rows = 2 ff;
        "clamped_glu": the same pairs with g = min(gate_f, limit), u = clamp(up_f, -limit, limit), a_f = g sigmoid(1.702 g) (u + 1).
        Indices at or above E (up.size(0)) name identity experts: their output is h[t] itself.  weigh "input": the weight multiplies the
        expert's input, y[t] = sum_k down[..] a(up[..] (wt[t, k] h[t])) (the products' results are scaled, in float)."""
        T, D = h.shape
        top_k, rows = idx.size(1), up.size(1)
        a = self.ACTS[act]
        ff = rows // 2 if a >= 2 else rows
        if (self.code == BF16 and self.moe_token_slots < T * top_k <= self.moe_expert_major_slots and D % 8 == 0 and ff % 8 == 0
                and D <= 4096 and ff <= 4096):
            return self._moe_experts_expert_major(h, up, down, idx, wt, a, limit, weigh)
        if T * top_k > self.moe_sorted_above:
            return self._moe_experts_sorted(h, up, down, idx, wt, a, limit, weigh)
        act = torch.empty((T, top_k, ff), dtype=self.dtype, device=h.device)
        y = torch.empty((T, D), dtype=self.dtype, device=h.device)
        self._need(h, up, down, idx, wt)
        w_in, w_out = self._weights_at(wt, weigh)
        assert up.shape[2] == D and down.shape == (up.size(0), D, ff)
        self.check(self.L.qsv_moe_up(act.data_ptr(), h.data_ptr(), up.data_ptr(), idx.data_ptr(), T, top_k, D, rows, a, float(limit),
                                     up.size(0), w_in, self.code, self._s()), "moe_up")
        self.check(self.L.qsv_moe_down(y.data_ptr(), act.data_ptr(), down.data_ptr(), idx.data_ptr(), w_out, T, top_k, D,
                                       ff, h.data_ptr(), up.size(0), self.code, self._s()), "moe_down")
        return y

    # More (token, expert) slots than this: sort the slots by expert and run each expert as one matrix product.  Below it the
    # per-token kernels above are used: no host synchronisation, a fixed launch sequence.
    moe_sorted_above = 64
    # the sorted form's products: the grouped matrix-core kernel (bfloat16, widths multiples of its K step) or one vendor product per expert
    moe_grouped_kernel = True

    # (token, expert) slots: up to moe_token_slots the per-token kernels (two launches); up to moe_expert_major_slots the
    # expert-major kernels (bfloat16; every expert weight read once, no host synchronisation); above, the expert-sorted vendor
    # products (compute-bound sizes)
    moe_token_slots = 8
    moe_expert_major_slots = 1024

    @staticmethod
    def _weights_at(wt, weigh):
        """-> addresses of the weights for the up products (on the input) and for the sum over the experts."""
        assert weigh in ("input", "output") and wt.dtype == torch.float32 and wt.is_contiguous()
        return (wt.data_ptr(), 0) if weigh == "input" else (0, wt.data_ptr())

    def _combine(self, h, ys, inv, idx, w_out, E):
        """y[t] = sum_k wt[t, k] * (ys[inv[t K + k]], or h[t] where idx[t, k] names an identity expert)."""
        T, D = h.shape
        y = torch.empty((T, D), dtype=self.dtype, device=h.device)
        self.check(self.L.qsv_moe_combine(y.data_ptr(), ys.data_ptr(), inv.data_ptr(), w_out, T, idx.size(1), D, idx.data_ptr(),
                                          h.data_ptr(), E, self.code, self._s()), "moe_combine")
        return y

    def _moe_experts_expert_major(self, h, up, down, idx, wt, a=1, limit=0.0, weigh="output"):
        T, D = h.shape
        w_in, w_out = self._weights_at(wt, weigh)
        E, rows, K = up.size(0), up.size(1), idx.size(1)
        ff = rows // 2 if a >= 2 else rows
        n = T * K
        expert, order = torch.sort(idx.reshape(-1).long(), stable=True)   # order: sorted slot -> slot (t K + k)
        # first sorted slot of every expert (and the end): a search in the sorted list - no count has to reach the host.  Slots of
        # identity experts (indices from E on) sort behind the last offset and are left to the combine.
        offsets = torch.searchsorted(expert, torch.arange(E + 1, device=h.device))
        inv = torch.empty_like(order)
        inv[order] = torch.arange(n, device=h.device)                  # slot -> sorted slot
        act = torch.empty((n, ff), dtype=self.dtype, device=h.device)
        ys = torch.empty((n, D), dtype=self.dtype, device=h.device)
        self.check(self.L.qsv_expert_rows(act.data_ptr(), h.data_ptr(), order.data_ptr(), K, up.data_ptr(), offsets.data_ptr(),
                                          E, rows, D, a, float(limit), w_in, self._s()), "expert_rows(up)")
        self.check(self.L.qsv_expert_rows(ys.data_ptr(), act.data_ptr(), 0, 1, down.data_ptr(), offsets.data_ptr(), E, D, ff, 0, 0.0,
                                          0, self._s()), "expert_rows(down)")
        return self._combine(h, ys, inv, idx, w_out, E)

    def _moe_experts_sorted(self, h, up, down, idx, wt, code=1, limit=0.0, weigh="output"):
        """code >= 2 (gated units): the grouped kernel folds the two halves of a unit in its epilogue; with vendor products the
        first product leaves both halves ([n, 2 ff]) and `glu` folds them."""
        T, D = h.shape
        w_in, w_out = self._weights_at(wt, weigh)
        E, rows, K = up.size(0), up.size(1), idx.size(1)
        ff = rows // 2 if code >= 2 else rows
        n = T * K
        flat = idx.reshape(-1)
        order = torch.argsort(flat, stable=True)                       # sorted slot -> slot (t K + k)
        counts = torch.bincount(flat, minlength=E).tolist()[:E]        # (host synchronisation: the runs' lengths; identity experts sort last)
        inv = torch.empty_like(order)
        inv[order] = torch.arange(n, device=h.device)                  # slot -> sorted slot
        ks, ts = self.L.qsv_grouped_gemm_k_step(), self.L.qsv_grouped_gemm_tile_slots()
        if self.moe_grouped_kernel and self.code == BF16 and D % ks == 0 and ff % ks == 0:
            # own grouped matrix-core kernel: gather in its loads, the activation in the first product's epilogue
            tiles, a = [], 0
            for e, c in enumerate(counts):
                tiles += [(e, a + o, min(ts, c - o)) for o in range(0, c, ts)]
                a += c
            act = torch.empty((n, ff), dtype=self.dtype, device=h.device)
            ys = torch.empty((n, D), dtype=self.dtype, device=h.device)
            for lo in range(0, len(tiles), 65535):
                tl = torch.tensor(tiles[lo:lo + 65535], dtype=torch.int32).to(h.device)
                self.check(self.L.qsv_grouped_gemm(act.data_ptr(), h.data_ptr(), order.data_ptr(), K, up.data_ptr(), tl.data_ptr(),
                                                   tl.size(0), rows, D, code, float(limit), w_in, self._s()), "grouped_gemm(up)")
                self.check(self.L.qsv_grouped_gemm(ys.data_ptr(), act.data_ptr(), 0, 1, down.data_ptr(), tl.data_ptr(),
                                                   tl.size(0), D, ff, 0, 0.0, 0, self._s()), "grouped_gemm(down)")
            return self._combine(h, ys, inv, idx, w_out, E)
        xs = torch.empty((n, D), dtype=self.dtype, device=h.device)
        self.check(self.L.qsv_gather_rows(xs.data_ptr(), h.data_ptr(), order.data_ptr(), K, n, D, self.code, self._s()),
                   "gather_rows")
        act = torch.empty((n, rows), dtype=self.dtype, device=h.device)
        ys = torch.empty((n, D), dtype=self.dtype, device=h.device)
        at = 0
        for e, c in enumerate(counts):
            if c:
                torch.matmul(xs[at:at + c], up[e].t(), out=act[at:at + c])
            at += c
        if code >= 2:
            act = self.glu(act, "silu" if code == 2 else "clamped", limit, *((wt.view(-1), order) if weigh == "input" else ()))
        else:
            if weigh == "input":
                raise ValueError("weights on the input: gated units only in the expert-sorted form with vendor products")
            self.check(self.L.qsv_relu_sq(act.data_ptr(), act.numel(), self.code, self._s()), "relu_sq")
        at = 0
        for e, c in enumerate(counts):
            if c:
                torch.matmul(act[at:at + c], down[e].t(), out=ys[at:at + c])
            at += c
        return self._combine(h, ys, inv, idx, w_out, E)


def _rotate(v, rope, pos, rot_n):
    """Interleaved-pair rotation of the first rot_n columns of v [..., n] (float); rope [P, 2, rot_n / 2]."""
    if not rot_n:
        return v
    cs = rope[pos.long()]                       # [T, 2, half]
    c, s = cs[:, 0], cs[:, 1]
    while c.dim() < v.dim():
        c, s = c.unsqueeze(1), s.unsqueeze(1)
    a, b = v[..., 0:rot_n:2], v[..., 1:rot_n:2]
    out = v.clone()
    out[..., 0:rot_n:2] = a * c - b * s
    out[..., 1:rot_n:2] = b * c + a * s
    return out


class TorchOps:
    """Unfused tensor-op form of HipOps (see the module docstring).  Same storage roundings at the same places."""
    name = "unfused"

    def __init__(self, dtype):
        self.dtype = dtype
        dtype_code(dtype)

    def embed(self, tokens, table):
        h = table[tokens.long()]
        return h.float(), h.to(self.dtype)

    @staticmethod
    def _ln(y, w, eps):
        y = y.float()
        mu = y.mean(-1, keepdim=True)
        var = ((y - mu) ** 2).mean(-1, keepdim=True)
        return (y - mu) / torch.sqrt(var + eps) * w.float()

    def add_layer_norm(self, x, y, w, eps):
        x += self._ln(y, w, eps)
        return x.to(self.dtype)

    def layer_norm_rows(self, x, rows, w, eps):
        return self._ln(x if rows is None else x[rows.long()], w, eps).to(self.dtype)

    @staticmethod
    def _rms(v, w, eps):
        v = v.float()
        return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps) * w.float()

    def latent_prep(self, down, q_off, q_rank, q_w, kv_off, kv_rank, kv_w, rot_dim, rot_n, rope, pool, slot, pos, eps):
        cq = self._rms(down[:, q_off:q_off + q_rank], q_w, eps).to(self.dtype)
        c = self._rms(down[:, kv_off:kv_off + kv_rank], kv_w, eps)
        kr = _rotate(down[:, kv_off + kv_rank:kv_off + kv_rank + rot_dim].float(), rope, pos, rot_n)
        pool[slot] = torch.cat([c, kr], dim=-1).to(self.dtype)
        return cq

    def latent_query(self, q, q_abs, rope, pos, scale, heads, dim, rot_dim, rot_n, rank):
        T = q.size(0)
        qr = _rotate(q.view(T, heads, dim + rot_dim)[..., dim:].float(), rope, pos, rot_n)
        return (torch.cat([q_abs.transpose(0, 1).float(), qr], dim=-1) * scale).contiguous()

    def latent_attention(self, qf, pool, batch, window, rank, page, variant=0, key_splits=None, q_first=0, chunk=None, bias=None,
                         keep_first=0, sink=None, pooled=None, pool_block=0, slopes=None):
        T, H, R = qf.shape
        block_table, seq, pos = batch.block_table, batch.seq, batch.pos
        out = torch.empty((T, H, rank), dtype=self.dtype, device=qf.device)
        bt = block_table.long()
        pools = [pool] if pool.dim() == 2 else list(pool)
        extra = None if pooled is None else ([pooled] if pooled.dim() == 2 else list(pooled))
        per = H // len(pools)
        per_page = (page + pool_block - 1) // pool_block if pooled is not None else 0
        for t in range(T):
            p = int(pos[t])
            lo = max(0, p - window + 1) if window else 0
            if chunk:
                lo = max(lo, p - p % chunk)
            j = torch.arange(lo, p + 1, device=qf.device)
            if keep_first:
                j = torch.cat([torch.arange(0, min(int(keep_first), lo), device=qf.device), j])
            at = bt[int(seq[t]), j // page] * page + j % page
            for g, pl in enumerate(pools):
                hs = slice(g * per, (g + 1) * per)
                rows = pl[at].float()                                                # [n, R]
                s = qf[t, hs] @ rows.t()                                             # [per, n]
                if bias is not None:
                    s = s + bias[hs][:, (p - j).clamp(max=bias.size(1) - 1)]
                if slopes is not None:
                    s = s - slopes[hs, None] * (p - j).float()
                if extra is not None:                                                # blocks wholly before the window
                    first = torch.arange(max(0, p - window + 1) // pool_block, device=qf.device) * pool_block
                    more = extra[g][bt[int(seq[t]), first // page] * per_page + (first % page) // pool_block].float()
                    s, rows = torch.cat([qf[t, hs] @ more.t(), s], dim=-1), torch.cat([more, rows])
                if sink is not None:
                    pr = torch.softmax(torch.cat([s, sink[hs, None]], dim=-1), dim=-1)[:, :-1]
                else:
                    pr = torch.softmax(s, dim=-1)
                out[t, hs] = (pr @ rows[:, :rank]).to(self.dtype)
        return out

    def sigmoid_gate(self, o, g):
        o.copy_((o.float() * torch.sigmoid(g.float())).to(self.dtype))
        return o

    # ---- streams, position-free norm, token shift -----------------------------------------------------------------------------
    def embed_streams(self, tokens, table, scale, streams):
        x = table[tokens.long()].float() * scale
        return x[:, None, :].repeat(1, streams, 1).contiguous()

    def hc_read(self, x, w_in, norm, shift=None, batch=None, prev=None):
        w, b, alpha = norm
        n = torch.tanh(alpha * torch.einsum("s,tsd->td", w_in, x)) * w.float() + b.float()
        if shift is None:
            return n.to(self.dtype)
        before = torch.zeros_like(n)
        before[1:] = n[:-1]
        for slot, first, cnt in batch.items:
            rd, wr = int(batch.state_rd[first]), int(batch.state_wr[first + cnt - 1])
            before[first] = prev[rd] if rd >= 0 else 0.0
            prev[wr] = n[first + cnt - 1]
        return (n + (before - n) * shift.float()).to(self.dtype)

    def hc_write(self, x, y, w_mix, w_out, then_read=None):
        x.copy_(torch.einsum("sr,tsd->trd", w_mix, x) + w_out[None, :, None] * y.float()[:, None, :])
        return None if then_read is None else self.hc_read(x, then_read[0], then_read[1])

    def dyt_sum_rows(self, x, rows, norm):
        w, b, alpha = norm
        u = (x if rows is None else x[rows.long()]).sum(1)
        return (torch.tanh(alpha * u) * w.float() + b.float()).to(self.dtype)

    # ---- rotations in the halves layout (pair i = dimensions i, i + n / 2) ------------------------------------------------------
    @staticmethod
    def _rotate_halves(v, rope, pos, n, sign=1.0):
        cs = rope[pos.long()]
        c, s = cs[:, 0, None, :], cs[:, 1, None, :] * sign
        a, b = v[..., :n // 2], v[..., n // 2:n]
        return torch.cat([a * c - b * s, b * c + a * s, v[..., n:]], dim=-1)

    def attention_prep(self, proj, q_off, k_off, v_off, heads, kv_heads, dim, vdim, rot_n, rope_k, rope_v, scale, pool, batch):
        T = proj.size(0)
        q = proj[:, q_off:q_off + heads * dim].float().view(T, heads, dim)
        k = proj[:, k_off:k_off + kv_heads * dim].float().view(T, kv_heads, dim)
        v = proj[:, v_off:v_off + kv_heads * vdim].float().view(T, kv_heads, vdim)
        q = self._rotate_halves(q, rope_k, batch.pos, rot_n) * scale
        k = self._rotate_halves(k, rope_k, batch.pos, rot_n)
        v = self._rotate_halves(v, rope_v, batch.pos, vdim)
        pool[:, batch.slot] = torch.cat([v, k], dim=-1).transpose(0, 1).to(self.dtype)
        return torch.cat([torch.zeros(T, heads, vdim, device=proj.device), q], dim=-1).contiguous()

    def rotate_heads(self, o, rope, pos, sign):
        o.copy_(self._rotate_halves(o.float(), rope, pos, o.size(-1), sign).to(self.dtype))
        return o


    # ---- sandwich norms, sink / kept-first / pooled-block attention, element-wise gated recurrence -----------------------------------
    def add_normed_rms_norm(self, x, y, w_post, w_next, eps):
        if y is not None:
            x += self._rms(y, w_post, eps)
        return None if w_next is None else self._rms(x, w_next, eps).to(self.dtype)

    def relu_sq(self, a):
        a.copy_((torch.relu(a.float()) ** 2).to(a.dtype))
        return a

    def qk_norm_rope_prep(self, q, k, v, heads, kv_heads, dim, vdim, q_w, k_w, per_head, eps, rope, rot_n, scale, pool, batch,
                          q_b=None, k_b=None, v_b=None, halves=False, head_scale=None, q_pad=None, rot_gain=0.0, q_store=False):
        T = q.size(0)

        def biased(u, b):
            return u.float() if b is None else u.float() + b.float()

        def prep(u, w, n):
            def turn(u):
                if rope is None:
                    return u
                return self._rotate_halves(u, rope, batch.pos, rot_n) if halves else _rotate(u, rope, batch.pos, rot_n)

            one = torch.ones(dim, device=u.device) if w is None else w
            if rot_gain > 0:
                return self._rms(turn(u.reshape(T, n, dim)), one, eps)
            return turn(self._rms(u.reshape(T, n, dim), one, eps) if per_head else self._rms(u, w, eps).view(T, n, dim))

        if k is not None:
            rows = torch.cat([biased(v, v_b).reshape(T, kv_heads, vdim), prep(biased(k, k_b), k_w, kv_heads)], dim=-1)
            pool[:, batch.slot] = rows.transpose(0, 1).to(self.dtype)
        out = prep(biased(q, q_b), q_w, heads) * scale
        if head_scale is not None:
            out = out * head_scale[:, None]
        out = torch.cat([torch.zeros(T, heads, vdim if q_pad is None else q_pad, device=q.device), out], dim=-1).contiguous()
        return out.to(self.dtype) if q_store else out

    def pool_blocks(self, pool, pooled, batch, block, page):
        per_page = (page + block - 1) // block
        bt = batch.block_table.long()
        for t in range(batch.n_tokens):
            p, s = int(batch.pos[t]), int(batch.seq[t])
            if (p + 1) % block:
                continue
            j = torch.arange(p + 1 - block, p + 1, device=pool.device)
            first = p + 1 - block
            dst = bt[s, first // page] * per_page + (first % page) // block
            pooled[:, dst] = (pool[:, bt[s, j // page] * page + j % page].float().sum(1) / block).to(self.dtype)

    def min_gru_scan(self, proj, z_off, x_off, g_off, b_z, b_x, state, batch, width):
        z = torch.sigmoid(proj[:, z_off:z_off + width].float() + b_z.float())
        u = proj[:, x_off:x_off + width].float() + b_x.float()
        c = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
        g = proj[:, g_off:g_off + width].float()
        out = torch.empty_like(z)
        for slot, first, cnt in batch.items:
            S = state[slot].clone() if int(batch.pos[first]) else torch.zeros_like(state[slot])
            for t in range(first, first + cnt):
                S = (1.0 - z[t]) * S + z[t] * c[t]
                out[t] = S
            state[slot] = S
        return (out * g * torch.sigmoid(g)).to(self.dtype)

    # ---- norm after the sum, convolved mixer input, talking-heads attention, retention operands -----------------------------------------
    def embed_rms_norm(self, tokens, table, w, eps):
        return self._rms(table[tokens.long()], w, eps)

    def residual_conv(self, x, conv_w, hist, batch):
        taps = conv_w.size(0)
        out = torch.empty_like(x)
        for slot, first, cnt in batch.items:
            rd, wr = int(batch.state_rd[first]), int(batch.state_wr[first + cnt - 1])
            past = hist[rd] if rd >= 0 and taps > 1 else torch.zeros((taps - 1, x.size(1)), device=x.device)
            seq = torch.cat([past, x[first:first + cnt]])
            out[first:first + cnt] = x[first:first + cnt] + sum(seq[j:j + cnt] * conv_w[j] for j in range(taps))
            if taps > 1:
                hist[wr] = seq[cnt:]
        return out.to(self.dtype)

    def scaled_add_rms_norm(self, x, y, alpha, w, eps, then_conv=None, batch=None, want_h=True):
        x.copy_(self._rms(alpha * x + y.float(), w, eps))
        if then_conv is not None:
            return self.residual_conv(x, then_conv[0], then_conv[1], batch)
        return x.to(self.dtype) if want_h else None

    def rotate_qk(self, qkv, heads, dim, vdim, rope, rot_n, batch):
        T = qkv.size(0)
        qk, v = qkv[:, :2 * heads * dim].float().reshape(T, 2 * heads, dim), qkv[:, 2 * heads * dim:heads * (2 * dim + vdim)].float()
        if rope is not None:
            qk = self._rotate_halves(qk, rope, batch.pos, rot_n)
        return torch.cat([qk.reshape(T, 2 * heads * dim), v], dim=-1)

    def talking_attention(self, qf, pool, batch, talk, gate, vdim, page, cap=0.0, window=None, variant=0, key_splits=None, decode=None):
        T, H, dim = qf.shape
        G = pool.size(0)
        per, bt = H // G, batch.block_table.long()
        out = torch.empty((T, H, vdim), dtype=torch.float32, device=qf.device)
        for t in range(T):
            p = int(batch.pos[t])
            j = torch.arange(max(0, p - int(window) + 1) if window else 0, p + 1, device=qf.device)
            rows = pool[:, bt[int(batch.seq[t]), j // page] * page + j % page].float()                # [G, n, R]
            s = torch.cat([qf[t, g * per:(g + 1) * per] @ rows[g, :, vdim:].t() for g in range(G)])       # [H, n]
            w = talk.float() @ torch.softmax(cap * torch.tanh(s / cap) if cap > 0 else s, dim=-1)
            out[t] = torch.cat([w[g * per:(g + 1) * per] @ rows[g, :, :vdim] for g in range(G)])
        if gate is not None:
            out = out * torch.sigmoid(gate.float())[:, :, None]
        return out.reshape(T, H * vdim).to(self.dtype)

    # ---- recurrences ----------------------------------------------------------------------------------------------------------
    def decay(self, z, bias, a_log, tau, heads, dim):
        z = z.float() + bias.float()
        if a_log is None:
            return torch.exp(-torch.nn.functional.softplus(-z) / tau).contiguous()          # sigmoid(z) ^ (1 / tau)
        rate = torch.exp(a_log.float()).repeat_interleave(dim)
        return torch.exp(-rate * torch.nn.functional.softplus(z)).contiguous()

    def conv_silu_unit(self, proj, off, conv_w, hist, batch, n_unit, unit_dim, act="silu"):
        C, taps = conv_w.shape
        xin = proj[:, off:off + C].to(self.dtype).float()
        out = torch.empty_like(xin)
        w = conv_w.float()
        for slot, first, cnt in batch.items:
            rd, wr = int(batch.state_rd[first]), int(batch.state_wr[first + cnt - 1])
            past = hist[rd][:taps - 1] if rd >= 0 else torch.zeros((taps - 1, C), device=xin.device)
            seq = torch.cat([past, xin[first:first + cnt]])
            y = sum(seq[j:j + cnt] * w[:, j] for j in range(taps))
            out[first:first + cnt] = y * torch.sigmoid(y) if act == "silu" else y
            if taps > 1:
                hist[wr] = seq[cnt:]
        if not n_unit:
            return out
        u = out[:, :n_unit * unit_dim].view(-1, n_unit, unit_dim)
        out[:, :n_unit * unit_dim] = (u / torch.sqrt((u * u).sum(-1, keepdim=True) + 1e-6)).view(-1, n_unit * unit_dim)
        return out

    def recurrent_scan(self, q, k, v, decay, beta, state, batch, heads, qk_heads, dim, vdim, q_scale, kscale=None, v_cols=None):
        T = q.size(0)
        rep = heads // qk_heads
        qf = q.float().reshape(T, qk_heads, dim).repeat_interleave(rep, 1) * q_scale
        kf = k.float().reshape(T, qk_heads, dim).repeat_interleave(rep, 1)
        if kscale is not None:
            kf = kf * kscale[:, :, None]
        vf = v.float().reshape(T, heads, v_cols or vdim)
        if v_cols and v_cols < vdim:
            ones = torch.zeros((T, heads, vdim - v_cols), device=q.device)
            ones[..., 0] = 1.0
            vf = torch.cat([vf, ones], dim=-1)
        if decay.dim() == 1:
            decay = decay.expand(T, heads)
        g = decay[:, :, None].expand(T, heads, dim) if decay.shape == (T, heads) and dim != 1 else decay.reshape(T, heads, dim)
        bt = None if beta is None else torch.sigmoid(beta.float())
        o = torch.empty((T, heads, vdim), dtype=torch.float32, device=q.device)
        for slot, first, cnt in batch.items:
            S = state[slot].clone() if int(batch.pos[first]) else torch.zeros_like(state[slot])
            for t in range(first, first + cnt):
                S = g[t][:, :, None] * S
                if bt is None:
                    S = S + kf[t][:, :, None] * vf[t][:, None, :]
                else:
                    u = bt[t][:, None] * (vf[t] - torch.einsum("hdv,hd->hv", S, kf[t]))
                    S = S + kf[t][:, :, None] * u[:, None, :]
                o[t] = torch.einsum("hdv,hd->hv", S, qf[t])
            state[slot] = S
        return o

    def head_rms_gate(self, o, w, gate, kind, eps, vdim=None, den_m=None):
        T, H, n_cols = o.shape
        dv = n_cols if vdim is None else vdim
        if den_m is not None:
            o = o[..., :dv] / (torch.maximum(o[..., dv].abs(), torch.exp(-den_m)) + 1e-6)[..., None]
        o = o[..., :dv]
        w = w.float().view(H, dv) if w.numel() == H * dv else w.float()
        n = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps) * w
        g = gate.float().reshape(T, H, dv)
        g = g * torch.sigmoid(g) if kind == "silu" else torch.sigmoid(g)
        return (n * g).reshape(T, H * dv).to(self.dtype)

    def rms_pair_mean(self, a, wa, b, wb, eps):
        return (0.5 * (self._rms(a, wa, eps) + self._rms(b, wb, eps))).to(self.dtype)

    def glu(self, a, act="silu", limit=0.0, row_scale=None, scale_index=None):
        a = a.float()
        if row_scale is not None:
            a = a * (row_scale if scale_index is None else row_scale[scale_index])[:, None]
        g, u = a[..., 0::2], a[..., 1::2]
        if act == "clamped":
            g, u = g.clamp(max=limit), u.clamp(-limit, limit)
            return (g * torch.sigmoid(1.702 * g) * (u + 1.0)).to(self.dtype)
        ag = g * torch.sigmoid(g) if act == "silu" else torch.nn.functional.gelu(g, approximate="tanh")
        return (ag * u).to(self.dtype)

    def moe_route(self, h, router, top_k, groups, keep, bias=None, renorm=False, score="softmax", correction=None, group_top=1,
                  scale=1.0):
        z = h.float() @ router.float().t()
        if bias is not None:
            z = z + bias.float()
        if renorm and score == "softmax" and correction is None and groups == 1:   # weights = softmax over the chosen logits only
            top = z.topk(top_k, dim=-1)
            return top.indices.int(), torch.softmax(top.values, dim=-1) * scale
        s = torch.softmax(z, dim=-1) if score == "softmax" else torch.sigmoid(z)
        c = s if correction is None else s + correction.float()
        T, E = s.shape
        per = E // groups
        gs = c.view(T, groups, per).topk(min(group_top, per), dim=-1).values.sum(-1)
        kept = torch.zeros_like(gs, dtype=torch.bool).scatter_(1, gs.topk(keep, dim=-1).indices, True)
        ok = kept[:, :, None].expand(T, groups, per).reshape(T, E)
        idx = c.masked_fill(~ok, float("-inf")).topk(top_k, dim=-1).indices
        wt = s.gather(1, idx)
        if renorm:
            wt = wt / wt.sum(-1, keepdim=True)
        return idx.int(), wt * scale

    # ---- sinusoidal positions, RMS-normed residual, whole-projection query / key norms ----------------------------------------------
    def embed_sinusoid(self, tokens, pos, table, freq, scale):
        a = pos.float()[:, None] * freq[None, :]                                    # float angles
        sc = torch.stack([torch.sin(a), torch.cos(a)], dim=-1).reshape(a.size(0), -1)[:, :table.size(1)]
        return table[tokens.long()].float() * scale + sc

    def add_rms_norm(self, x, ys, w, eps):
        ys = [y.float() for y in ys if y is not None]
        if ys:
            y = ys[0]
            if len(ys) > 1:
                y = y + (ys[1] + ys[2] if len(ys) > 2 else ys[1])
            x += y
        return None if w is None else self._rms(x, w, eps).to(self.dtype)

    def rms_norm_rows(self, x, rows, w, eps):
        return self._rms(x if rows is None else x[rows.long()], w, eps).to(self.dtype)

    def scaled_sum_rms_norms(self, x, parts, gains, eps, tokens=None, table=None):
        if tokens is not None:
            start = table[tokens.long()].float()
            x = start if x is None else x.copy_(start)
        if parts:
            x += sum((1.0 if s is None else s.float()) * y.float() for y, s in parts)
        return x, [self._rms(x, g, eps).to(self.dtype) for g in gains]

    # ---- attention with two key maps over the same values ----------------------------------------------------------------------------
    def conv_heads_cache(self, proj, conv_w, hist, batch, q_channels, kv_heads, key_width, vdim, pool, scale, temperature=None):
        taps, C = conv_w.shape
        u, y = proj[:, :C].float(), torch.empty((proj.size(0), C), device=proj.device)
        for slot, first, cnt in batch.items:
            rd, wr = int(batch.state_rd[first]), int(batch.state_wr[first + cnt - 1])
            past = hist[rd] if rd >= 0 and taps > 1 else torch.zeros((taps - 1, C), device=proj.device)
            seq = torch.cat([past, u[first:first + cnt]])
            y[first:first + cnt] = sum(seq[j:j + cnt] * conv_w[j] for j in range(taps))
            if taps > 1:
                hist[wr] = seq[cnt:]
        if kv_heads:
            T, n = proj.size(0), q_channels + kv_heads * key_width
            rows = torch.cat([y[:, n:].reshape(T, kv_heads, vdim), y[:, q_channels:n].reshape(T, kv_heads, key_width)], dim=-1)
            pool[:, batch.slot] = rows.transpose(0, 1).to(self.dtype)
        q = y[:, :q_channels] * scale
        if temperature is not None:
            coef, every = temperature
            q = q * (1.0 + coef * torch.log(torch.floor((batch.pos.double() + 1.0) / every).float() + 1.0))[:, None]
        return q.to(self.dtype)

    def maps_attention_ok(self, dim, vdim, maps, page):
        return False

    def diff_attention(self, q, pool, batch, heads, dim, vdim, lam, out_scale, eps, gate, page, variant=0, key_splits=None):
        T, G = q.size(0), pool.size(0)
        q, per, bt = q.view(T, heads, 2, dim).float(), heads // G, batch.block_table.long()
        o = torch.empty((T, heads, vdim), device=q.device)
        for t in range(T):
            j = torch.arange(int(batch.pos[t]) + 1, device=q.device)
            rows = pool[:, bt[int(batch.seq[t]), j // page] * page + j % page].float()                 # [G, n, R]
            for g in range(G):
                hs, v = slice(g * per, (g + 1) * per), rows[g, :, :vdim]
                a1, a2 = (torch.softmax(q[t, hs, m] @ rows[g, :, vdim + m * dim:vdim + (m + 1) * dim].t(), dim=-1) @ v for m in (0, 1))
                o[t, hs] = a1 - lam * a2
        o = (o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps) * out_scale).reshape(T, heads * vdim)
        if gate is not None:
            o = o * torch.sigmoid(gate.float())
        return o.to(self.dtype)

    def normed_attention_prep(self, proj, q_off, k_off, v_off, heads, kv_heads, dim, vdim, q_w, k_w, eps, scale, v_first, mix, pool,
                              batch):
        T = proj.size(0)
        q = self._rms(proj[:, q_off:q_off + heads * dim], q_w, eps).view(T, heads, dim) * scale
        k = self._rms(proj[:, k_off:k_off + kv_heads * dim], k_w, eps).view(T, kv_heads, dim)
        v = proj[:, v_off:v_off + kv_heads * vdim].float()
        if v_first is not None:
            v = (1.0 - mix) * v + mix * v_first.float()
        pool[:, batch.slot] = torch.cat([v.view(T, kv_heads, vdim), k], dim=-1).transpose(0, 1).to(self.dtype)
        return torch.cat([torch.zeros(T, heads, vdim, device=proj.device), q], dim=-1).contiguous()

    def max_gates(self, proj, i_off, f_off, bias_i, bias_f, cap, m_state, batch, heads):
        li = cap * torch.tanh((proj[:, i_off:i_off + heads].float() + bias_i) / cap)
        lf = torch.nn.functional.logsigmoid(cap * torch.tanh((proj[:, f_off:f_off + heads].float() + bias_f) / cap))
        a, b, m = torch.empty_like(li), torch.empty_like(li), torch.empty_like(li)
        for slot, first, cnt in batch.items:
            prev = m_state[slot].clone() if int(batch.pos[first]) else torch.zeros_like(m_state[slot])
            for t in range(first, first + cnt):
                m[t] = torch.maximum(lf[t] + prev, li[t])
                a[t], b[t] = torch.exp(lf[t] + (prev - m[t])), torch.exp(li[t] - m[t])
                prev = m[t]
            m_state[slot] = prev
        return a, b, m

    def moe_experts(self, h, up, down, idx, wt, act="relu_sq", limit=0.0, weigh="output"):
        T, D = h.shape
        E = up.size(0)
        y = torch.zeros((T, D), dtype=torch.float32, device=h.device)
        for k in range(idx.size(1)):
            e = idx[:, k].long()
            real = e < E
            e = e.clamp(max=E - 1)
            a = torch.einsum("tfd,td->tf", up[e].float(), h.float())
            if weigh == "input":
                a = a * wt[:, k, None]
            if act == "relu_sq":
                a = torch.relu(a) ** 2
            else:
                a = self.glu(a.to(self.dtype), "silu" if act == "swiglu" else "clamped", limit).float()
            a = a.to(self.dtype).float()
            o = torch.einsum("tdf,tf->td", down[e].float(), a)
            y += (wt[:, k, None] if weigh == "output" else 1.0) * torch.where(real[:, None], o, h.float())
        return y.to(self.dtype)


def make_ops(backend, dtype, device):
    """backend: "hip" (the only one a served model uses) or "unfused" (bring-up and host-logic tests)."""
    if backend == "hip":
        if torch.device(device).type != "cuda":
            raise RuntimeError("the hip backend needs a GPU device; there is no CPU path for served models")
        return HipOps(dtype)
    if backend == "unfused":
        return TorchOps(dtype)
    raise ValueError(f"unknown backend {backend!r}")
