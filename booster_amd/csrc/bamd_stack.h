// bamd_stack.h — configured layer stacks: decoder-only models whose config.json lists its layers (a mixer and an optional feed-forward each).
// A design is a bamd_stack_design: the mechanisms it fixes, by name.  Sizes and constants come from config.json, shapes from the tensors.
#pragma once
enum {
    STACK_NORM_OUTPUT_SCALAR = 1,                  // x + norm(sublayer(x)); RMS norm with one number as gain
    STACK_NORM_SANDWICH = 2                        // x + scale * norm_b(sublayer(norm(x))); layer norms with a gain per element, a scale per element behind them
};
enum { STACK_ACT_POLYNORM = 1, STACK_ACT_CLAMPED_GLU = 2 };
struct bamd_stack_design {
    bool scaled_embedding;                         // embedding times a constant
    bool learned_positions;                        // pos[p] added to the embedding
    bool token_shift;                              // mixers read h + (h_prev - h) * shift
    int norm, mlp_act;
    bool tied_head;                                // logits = embedding table x * logit_scale
    const char * mixers;                           // the mixers its layers may name, blank-separated
    bool latent_sink, latent_gate;                 // latent attention: sink in the softmax, gate per head
    bool kv_unit, kv_cap, kv_bias, kv_gate;        // attention over keys and values: unit-RMS queries and keys, capped scores, bias per distance, gate per head
    bool gla_gate;                                 // gated linear attention: silu gate behind the norm of a head's output
};
