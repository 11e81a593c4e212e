"""Host-side handle of the resident decoder behind ``fa_decoder_*``: a Llama-style stack of W8A8 linears,
RMSNorm, RoPE and paged GQA attention whose weights, KV pools, block tables and generator state stay on the
device; a decode step or a prompt pass only queues kernels."""
import ctypes as C

import numpy as np

from . import capi
from .backend import check

lib = capi.lib


class Decoder:
    state_slots = 0                                       # recurrent states the decoder holds; 0: it has none
    takes_portions = False                                # whether ``forward`` is there

    def __init__(self, ops, n_layers, d_model, n_heads, n_kv_heads, d_ffn, vocab, max_blocks_per_seq, num_blocks,
                 max_batch, head_dim=128, block_size=16, rms_eps=1e-5, rope_theta=500000.0):
        self._ops = ops
        self.cfg = capi.DecoderConfig(n_layers, d_model, n_heads, n_kv_heads, head_dim, d_ffn, vocab, block_size,
                                      max_blocks_per_seq, num_blocks, max_batch, rms_eps, rope_theta)
        self._h = C.c_void_p()
        check(lib.fa_decoder_create(ops._ctx, C.byref(self.cfg), C.byref(self._h)))
        self._keep = []                                   # weights must outlive the decoder that points at them
        self.batch = 0

    @classmethod
    def from_handle(cls, ops, handle, cfg):
        """Wraps an fa_decoder created elsewhere (not destroyed by ``close``)."""
        d = cls.__new__(cls)
        d._ops, d._h, d.cfg, d._keep, d.batch, d._borrowed = ops, handle, cfg, [], 0, True
        return d

    def close(self):
        if getattr(self, "_borrowed", False):
            self._h = None
            return
        h, self._h = getattr(self, "_h", None), None
        if h and self._ops._ctx:
            lib.fa_decoder_destroy(self._ops._ctx, h)
        for w in self._keep:
            w.free()
        self._keep = []

    def set_layer(self, layer, attn_norm, ffn_norm, wqkv, wo, wgu, wdown):
        """attn_norm / ffn_norm: device buffers [d_model] f32; the others QuantizedWeight (int8, per channel):
        wqkv [d_model, (heads + 2 kv_heads) head_dim], wo [heads head_dim, d_model], wgu [d_model, 2 d_ffn]
        (gate columns first), wdown [d_ffn, d_model]."""
        check(lib.fa_decoder_set_layer(self._h, layer, attn_norm._h, ffn_norm._h, wqkv._h, wo._h, wgu._h, wdown._h))
        self._keep += [attn_norm, ffn_norm, wqkv, wo, wgu, wdown]

    def set_head(self, embed, final_norm, lm_head):
        check(lib.fa_decoder_set_head(self._h, embed._h, final_norm._h, lm_head._h))
        self._keep += [embed, final_norm, lm_head]

    def set_sequences(self, block_tables, seq_lens):
        t = np.ascontiguousarray(block_tables, dtype=np.uint32)
        s = np.ascontiguousarray(seq_lens, dtype=np.uint32)
        check(lib.fa_decoder_set_sequences(self._ops._ctx, self._h, s.size, t.ctypes.data_as(capi.u32p),
                                           s.ctypes.data_as(capi.u32p)))
        self.batch = int(s.size)

    def set_tokens(self, tokens):
        t = np.ascontiguousarray(tokens, dtype=np.int32)
        check(lib.fa_decoder_set_tokens(self._ops._ctx, self._h, t.ctypes.data_as(capi.i32p)))

    def set_sampling(self, strategy, temperature=1.0, top_k=0, seed=0):
        check(lib.fa_decoder_set_sampling(self._ops._ctx, self._h, strategy, temperature, top_k, seed))

    def set_row_sampling(self, rows):
        """rows: a ctypes array of ``capi.RowSampling``, one per installed sequence."""
        if len(rows) != self.batch:
            raise ValueError("one sampling record per installed sequence")
        check(lib.fa_decoder_set_row_sampling(self._ops._ctx, self._h, rows))

    def read_row_sampling(self):
        rows = (capi.RowSampling * self.batch)()
        check(lib.fa_decoder_read_row_sampling(self._ops._ctx, self._h, rows))
        return rows

    def prefill(self, prompt):
        """prompt: int32 [batch, l_new]; leaves the next tokens resident like a step."""
        p = np.ascontiguousarray(prompt, dtype=np.int32)
        if p.ndim != 2 or p.shape[0] != self.batch:
            raise ValueError("prompt must be [batch, l_new]")
        check(lib.fa_decoder_prefill(self._ops._ctx, self._h, p.ctypes.data_as(capi.i32p), p.shape[1]))

    def prefill_padded(self, prompts):
        """prompts: one int32 sequence per installed row, of any lengths >= 1; they are padded to the longest
        and ingested in one pass (batch * longest <= 4096).  Every row ends as after its own ``prefill``."""
        if len(prompts) != self.batch:
            raise ValueError("one prompt per installed sequence")
        lens = np.array([len(p) for p in prompts], dtype=np.uint32)
        padded = np.zeros((self.batch, int(lens.max()) if len(prompts) else 0), dtype=np.int32)
        for b, p in enumerate(prompts):
            padded[b, :len(p)] = p
        check(lib.fa_decoder_prefill_padded(self._ops._ctx, self._h, padded.ctypes.data_as(capi.i32p), padded.shape[1],
                                            lens.ctypes.data_as(capi.u32p)))

    def verify(self, tokens, want_logits=False):
        """Speculative verification: feeds tokens [batch, l_new] like ``prefill`` and returns the greedy token
        after every one of them, int32 [batch, l_new] (and the logits [batch, l_new, vocab] if asked)."""
        p = np.ascontiguousarray(tokens, dtype=np.int32)
        if p.ndim != 2 or p.shape[0] != self.batch:
            raise ValueError("tokens must be [batch, l_new]")
        picked = np.empty(p.shape, dtype=np.int32)
        logits = np.empty(p.shape + (self.cfg.vocab,), dtype=np.float32) if want_logits else None
        check(lib.fa_decoder_verify(self._ops._ctx, self._h, p.ctypes.data_as(capi.i32p), p.shape[1],
                                    picked.ctypes.data_as(capi.i32p),
                                    logits.ctypes.data_as(capi.f32p) if want_logits else None))
        return (picked, logits) if want_logits else picked

    def rewind(self, seq_lens):
        """Shortens the installed sequences (no row may grow); the pages are kept."""
        s = np.ascontiguousarray(seq_lens, dtype=np.uint32)
        if s.size != self.batch:
            raise ValueError("one length per installed sequence")
        check(lib.fa_decoder_rewind(self._ops._ctx, self._h, s.ctypes.data_as(capi.u32p)))

    def step(self, use_graph=True):
        check(lib.fa_decoder_step(self._ops._ctx, self._h, 1 if use_graph else 0))

    def tokens(self):
        out = np.empty(self.batch, dtype=np.int32)
        check(lib.fa_decoder_read_tokens(self._ops._ctx, self._h, out.ctypes.data_as(capi.i32p)))
        return out

    def logits(self):
        out = np.empty((self.batch, self.cfg.vocab), dtype=np.float32)
        check(lib.fa_decoder_read_logits(self._ops._ctx, self._h, out.ctypes.data_as(capi.f32p)))
        return out

    def logits_buffer(self):
        """Raw handle of the resident logits [max_batch, vocab] (owned by the decoder)."""
        h = capi.buf_p()
        check(lib.fa_decoder_logits_buffer(self._h, C.byref(h)))
        return h

    def seq_lens(self):
        out = np.empty(self.batch, dtype=np.uint32)
        check(lib.fa_decoder_read_seq_lens(self._ops._ctx, self._h, out.ctypes.data_as(capi.u32p)))
        return out


class LayeredDecoder(Decoder):
    """A decoder whose layers are described one by one (``fa_decoder_create_layered``): unquantized weights in bf16 or
    f32, per layer one mixer or two side by side (gated delta rule, lightning attention or a minimal gated recurrence with a
    recurrent state, attention, latent or grouped-query, over the paged cache), and an optional feed-forward, dense or of sparse experts.  Sequences,
    steps, prompt passes and sampling are ``Decoder``'s."""

    takes_portions = True

    def __init__(self, ops, d_model, vocab, layers, norm_eps, logit_softcap, max_blocks_per_seq, num_blocks, max_batch,
                 state_slots=None, dtype=capi.BF16, block_size=16, norm=capi.NORM_INPUT, embed_scale=1.0, position_base=0.0,
                 logit_scale=1.0):
        """layers: one dict of ``capi.LayerConfig`` fields per layer (``right``: such a dict, ``decay``: a list)."""
        self._ops = ops
        rows = (capi.LayerConfig * len(layers))(*[self._layer(l) for l in layers])
        recurrent = any(m["mixer"] in (capi.MIXER_DELTA, capi.MIXER_LIGHTNING, capi.MIXER_MINGRU) for l in layers for m in (l, l.get("right") or l))
        slots = max_batch if state_slots is None else state_slots
        self.cfg = capi.LayeredConfig(len(layers), d_model, vocab, block_size, max_blocks_per_seq, num_blocks, max_batch,
                                      slots, norm_eps, logit_softcap, dtype, rows, norm, embed_scale, position_base, logit_scale)
        self.state_slots = slots if recurrent else 0
        self._h = C.c_void_p()
        check(lib.fa_decoder_create_layered(ops._ctx, C.byref(self.cfg), C.byref(self._h)))
        self._keep = []
        self.batch = 0

    @classmethod
    def _layer(cls, fields):
        f = dict(fields)
        if f.get("decay") is not None:
            f["decay"] = (C.c_float * len(f["decay"]))(*f["decay"])
        if f.get("right") is not None:
            f["right"] = C.pointer(cls._layer(f["right"]))
        return capi.LayerConfig(**f)

    def tensors(self):
        """name -> shape of every weight tensor the decoder takes."""
        n, name, rows, cols = C.c_uint32(), C.c_char_p(), capi.u64(), capi.u64()
        check(lib.fa_decoder_tensor_count(self._h, C.byref(n)))
        out = {}
        for i in range(n.value):
            check(lib.fa_decoder_tensor_info(self._h, i, C.byref(name), C.byref(rows), C.byref(cols)))
            out[name.value.decode()] = (rows.value, cols.value) if cols.value else (rows.value,)
        return out

    def set_tensor(self, name, array, bf16=False):
        """array: float32 values, or bf16 bit patterns in uint16 (bf16=True), as the checkpoint stores them."""
        a = np.ascontiguousarray(array, dtype=np.uint16 if bf16 else np.float32)
        rows, cols = (a.shape[0], a.shape[1]) if a.ndim == 2 else (a.size, 0)
        check(lib.fa_decoder_set_tensor(self._ops._ctx, self._h, name.encode(), capi.BF16 if bf16 else capi.F32,
                                        a.ctypes.data_as(C.c_void_p), rows, cols))

    def set_state_slots(self, slots):
        s = np.ascontiguousarray(slots, dtype=np.uint32)
        if s.size != self.batch:
            raise ValueError("one state slot per installed sequence")
        check(lib.fa_decoder_set_state_slots(self._ops._ctx, self._h, s.ctypes.data_as(capi.u32p)))

    def forward(self, portions, want=None, residuals=False):
        """One pass over all installed sequences: portions[b] are row b's next tokens (any number, none included).
        want[b]: places in portions[b] whose logits are asked for.  Returns the logits [wanted, vocab] in row order (and,
        with residuals, the residual stream after every layer, [layers, tokens, d_model])."""
        if len(portions) != self.batch:
            raise ValueError("one portion per installed sequence")
        counts = np.array([len(p) for p in portions], dtype=np.uint32)
        flat = np.array([t for p in portions for t in p], dtype=np.int32)
        starts = np.concatenate([[0], np.cumsum(counts)]).astype(np.int64)
        places = np.array([starts[b] + k for b, ks in enumerate(want or []) for k in ks], dtype=np.uint32)
        logits = np.empty((places.size, self.cfg.vocab), dtype=np.float32)
        trace = np.empty((self.cfg.n_layers, flat.size, self.cfg.d_model), dtype=np.float32) if residuals else None
        if residuals:
            check(lib.fa_decoder_debug_residuals(self._h, trace.ctypes.data_as(capi.f32p), flat.size))
        check(lib.fa_decoder_forward(self._ops._ctx, self._h, counts.ctypes.data_as(capi.u32p), flat.ctypes.data_as(capi.i32p),
                                     places.size, places.ctypes.data_as(capi.u32p) if places.size else None,
                                     logits.ctypes.data_as(capi.f32p) if places.size else None))
        return (logits, trace) if residuals else logits
