// The attention variants behind hfa_paged_attention.
#pragma once
#include <hip/hip_runtime.h>

struct AttnArgs {
    const void* q; int ldq;
    const void* k_cache; const void* v_cache; int kv_width;
    const int* block_table; int max_blocks;
    const int* token_slot; const int* positions; const int* q_start;
    int n_seqs, max_q_len, max_seq_len;
    void* out; int ldo;
    int n_tokens, n_heads, n_kv_heads, head_dim, page_tokens, window;
    float scale;
    void* workspace; size_t workspace_bytes;
    hipStream_t stream;
    // decoded tokens whose queries, new key and new value still lie in 32-bit rows [q | k | v] (see attn_mfma_kernel,
    // FUSED): raw is null otherwise
    const float* raw; int ld_raw;
    const float* cos_sin;          // [token][head_dim / 2 cosines, head_dim / 2 sines], null: no rotation
    const int* slot_map;           // the cache row of each token's key and value
    int mask_chunk;                // > 0: a query sees only the keys of its own run of mask_chunk positions, counted from 0
    int sink;                      // 1: the softmax's denominator holds one more term of score 0 that has no value
    int v_rot;                     // the weights of a head of group c are applied to the values of group (c + v_rot) mod G (0: its own)
    float softcap;                 // > 0: score <- softcap tanh(score / softcap)
    int weights;                   // 0: softmax; 1: sigmoid(score + head_bias[head]), not normalised over the keys
    const float* head_bias;        // one number a query head, or null
    const float* sink_w;           // with sink: the extra term's score per query head (null: 0)
    const float* dist_scale;       // per query head, or null: a softmax's score is lowered by dist_scale[h] ln(1 + dist_rate[h] (i - j))
    const float* dist_rate;
    int v_head_dim, v_width;       // a value head's size and the value rows' width (0: the keys')
    int v_share;                   // that many neighbouring key heads read one value head (0: one)
    int keep_first;                // > 0: under a window the keys 0 .. keep_first - 1 stay in sight
    const float* rel; int rel_n;   // [query head][rel_n]: a number by distance (beyond rel_n - 1: the last) added to a softmax's score, or null
    const void* gate; int gate_bf16, ldg;      // [token][query head]: a head's result is multiplied by sigmoid(gate), or null
    float out_mul;                 // and by this number
    int out_f32;                   // results leave in 32 bits
};

// How a call is cut: tiles of columns, chunks of keys, and for the kernel of prompt portions the pairing of long and short tiles.
struct AttnCut {
    int prompt, tiles, tpt, cpt, chunk_keys, n_chunks, prompt_tiles, pair_from;
};

// Whether a softmax's scores are more than a scaled product (a soft cap, a term of the distance): the matrix-core kernels
// then run an instantiation of their own.
inline bool attn_shaped_scores(const AttnArgs& a) { return a.weights == 0 && (a.softcap > 0.f || a.dist_scale != nullptr); }

// Whether a query sees a bounded run of keys only: cuts of the keys are then counted from the first key block of a tile.
__host__ __device__ __forceinline__ bool attn_bounded(int window, int mask_chunk) { return window > 0 || mask_chunk > 0; }

// The first key that the query at `pos` sees: a window of the last `window` positions (0: none) and/or the start
// of the query's own masking chunk (0: none). It never falls as pos grows.
__host__ __device__ __forceinline__ int first_visible(int pos, int window, int mask_chunk) {
    int lo = window > 0 && pos - window + 1 > 0 ? pos - window + 1 : 0;
    if (mask_chunk > 0) {
        const int c = pos - pos % mask_chunk;
        lo = c > lo ? c : lo;
    }
    return lo;
}

// The plain kernel: any of what AttnArgs can ask for (with v_head_dim and v_width given).
int attn_generic_launch(const AttnArgs& a, int dtype, const float* slopes, int cross);

// Single tokens of a mixer that mixes its heads' weights after the softmax: every head's weights on the values of every
// group in one pass over the cache, written in rounds of groups (see attention_cross.hip). `supports` leaves the cut
// of the keys that `launch` takes.
bool attn_cross_supports(const AttnArgs& a, int* chunk_keys, int* n_chunks);
int attn_cross_launch(const AttnArgs& a, int chunk_keys, int n_chunks);

// Many query heads on one key/value head with wide key rows and value rows of another size (attention through latents), bf16 on
// the matrix cores; see attention_shared.hip for what it needs.
bool attn_shared_supports(const AttnArgs& a, int v_head_dim, int v_width);
int attn_shared_launch(const AttnArgs& a, int v_head_dim);

// Calls that take an instantiation of attention_masked.hip (whose sizes `attn_masked_sizes` names).
inline bool attn_masked_mode(const AttnArgs& a) {
    return a.rel != nullptr || a.keep_first > 0 || a.v_share > 1 || (a.v_head_dim > 0 && a.v_head_dim != a.head_dim) ||
           (a.v_width > 0 && a.v_width != a.kv_width);
}
bool attn_masked_sizes(int head_dim, int v_head_dim);
int attn_masked_run(const AttnArgs& a, const AttnCut& c);

// bf16 on the matrix cores; see attention_mfma.hip for what it needs.
bool attn_mfma_supports(const AttnArgs& a);
int attn_mfma_launch(const AttnArgs& a);
