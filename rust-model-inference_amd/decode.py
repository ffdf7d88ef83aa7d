"""Decoder sessions over the device-resident entry points of the C ABI: weights go to HBM once, then whole
generations run on the GPU with one synchronisation at the end.  ``Qwen3Session`` mirrors the reference's
(src/models/qwen3.rs:581-1158); the ``FolderSession`` classes run model folders; ``models`` picks the class.
"""
import ctypes as C

import numpy as np

from . import hip

_MATMULS = (("wq", "attn_q"), ("wk", "attn_k"), ("wv", "attn_v"), ("wo", "attn_output"), ("w_gate", "ffn_gate"),
            ("w_up", "ffn_up"), ("w_down", "ffn_down"))
_NORMS = (("attn_norm", "attn_norm"), ("ffn_norm", "ffn_norm"), ("q_norm", "attn_q_norm"), ("k_norm", "attn_k_norm"))


class _Session:
    """What the sessions share: `_abi` names the C functions, `_h` is the handle, `vocab` the logits' width."""

    _abi = None
    _h = None

    def _fn(self, name):
        return getattr(hip.lib, f"rmi_hip_{self._abi}_{name}")

    def set_stop_ids(self, ids):
        """The tokenizer's EOS / `im_end` ids (src/models/qwen3.rs:1123-1130): generation ends before the first."""
        ids = np.ascontiguousarray(ids, np.uint32)
        hip.check(self._fn("set_stop_ids")(self._h, hip.ptr(ids, hip._u32p), ids.size))

    def set_prompt_passes(self, enabled):
        """Prompt positions as many to a pass as the session takes (True, the default), every position its own step
        (False), or that many to a pass (an int above 1); same results either way (bit for bit for Qwen3, within
        rounding for model folders)."""
        hip.check(self._fn("set_prompt_passes")(self._h, int(enabled)))

    def generate(self, prompt, max_new, dump_steps=()):
        prompt = np.ascontiguousarray(prompt, np.uint32)
        steps = prompt.size + max_new - 1
        gen = np.zeros(max(max_new, 1), np.uint32)
        argmax = np.zeros(steps, np.uint32)
        top2 = np.zeros((steps, 2), np.float32)
        dump_steps = np.ascontiguousarray(dump_steps, np.uint32)
        dump = np.zeros((max(dump_steps.size, 1), self.vocab), np.float32)
        seconds = C.c_double()
        n = self._fn("generate")(self._h, hip.ptr(prompt, hip._u32p), prompt.size, max_new, hip.ptr(gen, hip._u32p),
                                 hip.ptr(argmax, hip._u32p), hip.ptr(top2, hip._f32p), hip.ptr(dump_steps, hip._u32p),
                                 dump_steps.size, hip.ptr(dump, hip._f32p), C.byref(seconds))
        if n < 0:
            raise hip.RmiHipError(n, hip.last_error())
        return dict(tokens=gen[:n], argmax=argmax, top2=top2, dump=dump[:dump_steps.size], seconds=seconds.value,
                    steps=steps)

    def close(self):
        if self._h:
            self._fn("destroy")(self._h)
            self._h = None

    def __del__(self):
        self.close()


class Qwen3Session(_Session):
    """`metadata` and `tensors` as a GGUF file gives them (keys of src/core/loader.rs:379-461, tensor
    names of src/models/qwen3.rs:269-349); every 2-D weight must be Q8_0 bytes, norms f32."""

    _abi = "qwen3"
    vocab = property(lambda self: self.config.vocab)

    def __init__(self, metadata, tensors, capacity, rounding=hip.ROUND_TIES_EVEN):
        g = lambda k: int(metadata[f"qwen3.{k}"])  # noqa: E731
        c = hip.Qwen3Config()
        c.n_embd, c.n_layer, c.n_head, c.n_head_kv = (g("embedding_length"), g("block_count"),
                                                      g("attention.head_count"), g("attention.head_count_kv"))
        c.head_dim_k = int(metadata.get("qwen3.attention.key_length", c.n_embd // c.n_head))
        c.head_dim_v = int(metadata.get("qwen3.attention.value_length", c.n_embd // c.n_head))
        c.n_ff, c.vocab, c.capacity = g("feed_forward_length"), int(metadata["qwen3.vocab_size"]), int(capacity)
        c.eps = float(metadata["qwen3.attention.layer_norm_rms_epsilon"])
        c.freq_base = float(metadata.get("qwen3.rope.freq_base", 1e6))
        c.has_qk_norm = 1 if "blk.0.attn_q_norm.weight" in tensors else 0
        c.rounding = rounding
        keep = []

        def raw(name):
            a = hip.as_u8(tensors[name])
            keep.append(a)
            return hip.ptr(a, hip._u8p)

        def f32(name):
            a = np.ascontiguousarray(np.asarray(tensors[name]).view(np.float32))
            keep.append(a)
            return hip.ptr(a, hip._f32p)

        w = hip.Qwen3Weights()
        w.token_embd = raw("token_embd.weight")
        w.output = raw("output.weight") if "output.weight" in tensors else None
        w.output_norm = f32("output_norm.weight")
        for field, name in _NORMS:
            if not c.has_qk_norm and field in ("q_norm", "k_norm"):
                continue
            arr = (hip._f32p * c.n_layer)(*[f32(f"blk.{layer}.{name}.weight") for layer in range(c.n_layer)])
            keep.append(arr)
            setattr(w, field, arr)
        for field, name in _MATMULS:
            arr = (hip._u8p * c.n_layer)(*[raw(f"blk.{layer}.{name}.weight") for layer in range(c.n_layer)])
            keep.append(arr)
            setattr(w, field, arr)
        self.config = c
        self._h = hip.lib.rmi_hip_qwen3_create(C.byref(c), C.byref(w))
        if not self._h:
            raise hip.RmiHipError(-1, hip.last_error())

    @classmethod
    def from_gguf(cls, loader, capacity, rounding=hip.ROUND_TIES_EVEN):
        """Qwen3Model::from_source + Qwen3Session::new over an open ``loader.GGUFLoader``: tensor bytes go from
        the file's mapping to HBM inside the library (src/models/qwen3.rs:262-349)."""
        self = cls.__new__(cls)
        self._h = None
        self.config = loader.qwen3_config(capacity, rounding)
        self._h = hip.lib.rmi_hip_qwen3_create_from_gguf(loader._h, int(capacity), rounding)
        if not self._h:
            raise hip.RmiHipError(-1, hip.last_error())
        return self


class FolderSession(_Session):
    """A model folder (config.json, model.safetensors) of any design the library knows.  dtype: hip.DTYPE_BF16 or
    hip.DTYPE_F32 (everything true f32); capacity: most tokens of a sequence.  One sequence at a time."""

    _abi = "folder"
    architecture = None  # the one that config.json has to name

    def __init__(self, folder, capacity, dtype=hip.DTYPE_BF16):
        arch = self.architecture.encode() if self.architecture else None
        self._h = hip.lib.rmi_hip_folder_open(str(folder).encode(), arch, dtype, int(capacity))
        if not self._h:
            raise hip.RmiHipError(-1, hip.last_error())
        v = [C.c_uint32() for _ in range(4)]
        hip.check(hip.lib.rmi_hip_folder_sizes(self._h, *[C.byref(x) for x in v]))
        self.vocab, self.width, self.n_layer, self.capacity = (x.value for x in v)

    position = property(lambda self: hip.lib.rmi_hip_folder_position(self._h))

    def step(self, tokens, want=(), layers=False):
        """The sequence's next tokens; logits [len(want), vocab] of the places `want` among them.  With `layers` also
        the residual stream behind every layer, [n_layer, tokens, width] (a looped layer counts each time)."""
        tokens = np.ascontiguousarray(tokens, np.uint32)
        want = np.ascontiguousarray(want, np.uint32)
        logits = np.zeros((want.size, self.vocab), np.float32)
        dump = np.zeros((self.n_layer, tokens.size, self.width), np.float32) if layers else None
        hip.check(hip.lib.rmi_hip_folder_step(self._h, hip.ptr(tokens, hip._u32p), tokens.size, hip.ptr(want, hip._u32p), want.size,
                                               hip.ptr(logits, hip._f32p), hip.ptr(dump, hip._f32p) if layers else None))
        return (logits, dump) if layers else logits

    def reset(self):
        """The sequence is over; the next step begins a new one."""
        hip.check(hip.lib.rmi_hip_folder_reset(self._h))


class RuvenexSession(FolderSession):
    """Parallel layers of softmax attention, an HGRN2 recurrence and a gelu feed-forward."""

    architecture = "Ruvenex"


class VogizenSession(FolderSession):
    """Layers of sliding-window latent attention or the gated delta rule, a token-side input, a looped run of layers."""

    architecture = "Vogizen"
