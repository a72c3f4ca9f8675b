// The attention of attention_mfma.hip (prompts, portions of prompts and decoded tokens) with every head's result multiplied
// by the sigmoid of one number per token and head, as a library of its own: the same kernels, under names of their own.
// Entry point: llms_attention_mfma_gated.
#define LLMS_ATTENTION_HEAD_GATED 1
#define attn_mfma_kernel attn_mfma_gated_kernel
#define attn_prompt_kernel attn_prompt_gated_kernel
#define attn_merge_kernel attn_merge_gated_kernel
#include "attention_mfma.hip"
