// Softmax attention on the matrix cores (attention_mfma.h): the instantiations with value heads of a size of their own (half or
// twice the keys'), with several key/value heads on one head of values, with a table of distance terms added to the scores
// (ATT_REL), and with a sequence's first keys kept in sight beside a window (ATT_KEEP).
#include "attention_mfma.h"

bool attn_masked_sizes(int d, int dv) {
    if (d % 32 || dv % 32 || d > 128 || dv > 128) return false;
    return d == dv || 2 * d == dv || d == 2 * dv;
}

template <int NDB, int VDB>
static int run_sizes(const AttnArgs& a, const AttnCut& c) {
    if (a.rel) return c.prompt ? launch_prompt<NDB, ATT_REL, VDB>(a, c) : launch_step<NDB, ATT_REL, VDB, false>(a, c);
    return c.prompt ? launch_prompt<NDB, ATT_KEEP, VDB>(a, c) : launch_step<NDB, ATT_KEEP, VDB, false>(a, c);
}

int attn_masked_run(const AttnArgs& a, const AttnCut& c) {
    const int dv = a.v_head_dim > 0 ? a.v_head_dim : a.head_dim;
    switch (a.head_dim / 32 * 10 + dv / 32) {
        case 11: return run_sizes<1, 1>(a, c);
        case 22: return run_sizes<2, 2>(a, c);
        case 33: return run_sizes<3, 3>(a, c);
        case 44: return run_sizes<4, 4>(a, c);
        case 12: return run_sizes<1, 2>(a, c);
        case 24: return run_sizes<2, 4>(a, c);
        case 21: return run_sizes<2, 1>(a, c);
        case 42: return run_sizes<4, 2>(a, c);
    }
    hfa_set_error("paged_attention: heads of %d and %d are not built", a.head_dim, dv);
    return 1;
}
