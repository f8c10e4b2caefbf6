"""MI355X-native multi-LoRA decode/prefill hot path: HIP kernels behind a C ABI, Python host on top.

Submodules: `ops` and `decoder_ops` (operator surface over the C ABI), `registry` (models by config.json, folder loading),
`model_base`, `llama` (LlamaForCausalLM with the reference's entry points), `safolorn` and `dinasun` with their mechanisms
`latent_attention`, `tied_attention`, `time_mix`, `feed_forward`, `rotary`, `lora` (LoraConfig, GatherMMLinear), `kv_cache`
(PagedKVCache, PagedLatentCache, PagedStateCache), `seq_info`, `exec_graph`, `llama_exec_graph`, `auto_batcher` (the auto-batching front end), `trace`
(replays token ids), `synth` (seeded synthetic inputs), `build` (compiles the libraries).  Importing the package does not
load a library; the first operator call does, and fails loudly if it has not been built.
"""
__all__ = ["ops", "decoder_ops", "registry", "model_base", "lora", "kv_cache", "llama", "safolorn", "dinasun", "latent_attention",
           "tied_attention", "time_mix", "feed_forward", "rotary", "seq_info", "exec_graph", "llama_exec_graph", "auto_batcher", "trace", "synth", "build"]
