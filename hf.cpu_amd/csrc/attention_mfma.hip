// Softmax attention on the matrix cores: which kernel takes a call, how its keys are cut, the merge of chunks, and the
// instantiations of the kernels (attention_mfma.h) with heads of one size.
#include "attention_mfma.h"

// out[t, h, :] = sum_c o_c 2^(m_c - M) / sum_c l_c 2^(m_c - M), chunks in ascending order.
// One wave per (token, head). The kernel is a chain of memory round trips and little else, so it
// is written to have few of them: the first MERGE_GROUP chunks' outputs are asked for before
// anything else, a lane reads maximum and sum of "its" chunk as one pair, and the rest of the
// outputs come MERGE_GROUP loads at a time. A lane owns two neighbouring dimensions (D <= 128).
#define MERGE_GROUP 16
__global__ __launch_bounds__(WAVE) void attn_merge_kernel(const float* __restrict__ partial, uint16_t* __restrict__ out,
                                                          int ldo, int H, int D, int n_chunks, int sink,
                                                          const float* __restrict__ sink_w, AttnExtra ex) {
    __shared__ float w_s[MERGE_MAX_CHUNKS];
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const size_t row = D + 2;
    const float* src = partial + (size_t)(t * H + h) * n_chunks * row;
    const bool has = 2 * lane < D;
    const float* mine = src + 2 + 2 * lane;
    float2 pre[MERGE_GROUP];
#pragma unroll
    for (int i = 0; i < MERGE_GROUP; i++)
        pre[i] = has && i < n_chunks ? *reinterpret_cast<const float2*>(mine + i * row) : make_float2(0.f, 0.f);
    const float2 ml0 = lane < n_chunks ? *reinterpret_cast<const float2*>(src + lane * row) : make_float2(NEG_BIG, 0.f);
    float M = ml0.x;
    for (int c = lane + WAVE; c < n_chunks; c += WAVE) M = fmaxf(M, src[c * row]);
    M = wave_max(M);
    float L = 0.f;
    if (lane < n_chunks) {
        const float w = exp2f(ml0.x - M);
        w_s[lane] = w;
        L = ml0.y * w;
    }
    for (int c = lane + WAVE; c < n_chunks; c += WAVE) {
        const float2 ml = *reinterpret_cast<const float2*>(src + c * row);
        const float w = exp2f(ml.x - M);
        w_s[c] = w;
        L += ml.y * w;
    }
    L = wave_sum(L);
    if (sink) L += exp2f((sink_w ? sink_w[h] * LOG2E : 0.f) - M);       // once for all chunks: the term that has no value
    __syncthreads();
    if (!has) return;
    float ax = 0.f, ay = 0.f;
#pragma unroll
    for (int i = 0; i < MERGE_GROUP; i++)
        if (i < n_chunks) {
            ax = fmaf(pre[i].x, w_s[i], ax);
            ay = fmaf(pre[i].y, w_s[i], ay);
        }
    for (int c0 = MERGE_GROUP; c0 < n_chunks; c0 += MERGE_GROUP) {
        float2 v[MERGE_GROUP];
#pragma unroll
        for (int i = 0; i < MERGE_GROUP; i++)
            v[i] = c0 + i < n_chunks ? *reinterpret_cast<const float2*>(mine + (c0 + i) * row) : make_float2(0.f, 0.f);
#pragma unroll
        for (int i = 0; i < MERGE_GROUP; i++)
            if (c0 + i < n_chunks) {
                ax = fmaf(v[i].x, w_s[c0 + i], ax);
                ay = fmaf(v[i].y, w_s[c0 + i], ay);
            }
    }
    const float inv = head_factor(ex, t, h) / L;
    if (ex.out_f32) {
        *reinterpret_cast<float2*>(reinterpret_cast<float*>(out) + (size_t)t * ldo + h * D + 2 * lane) = make_float2(ax * inv, ay * inv);
        return;
    }
    *reinterpret_cast<uint32_t*>(out + (size_t)t * ldo + h * D + 2 * lane) =
        (uint32_t)bf16_bits(ax * inv) | ((uint32_t)bf16_bits(ay * inv) << 16);
}

bool attn_mfma_supports(const AttnArgs& a) {
    const int group = a.n_heads / a.n_kv_heads;
    // a scale that is not positive goes to the plain kernel: the prompt kernel takes the maximum before scaling
    const int dv = a.v_head_dim > 0 ? a.v_head_dim : a.head_dim, vw = a.v_width > 0 ? a.v_width : a.kv_width;
    const bool masked = attn_masked_mode(a);
    // what the instantiations of attention_masked.hip take: one kind of extra at a time, a head's own values, no fused prologue
    if (masked && (a.raw != nullptr || a.v_rot != 0 || a.weights != 0 || attn_shaped_scores(a) || (a.rel && a.keep_first > 0) ||
                   !attn_masked_sizes(a.head_dim, dv) || vw % 8 != 0 || vw * a.page_tokens >= (1 << 20)))
        return false;
    return a.scale > 0.f && a.head_dim % 32 == 0 && a.head_dim <= 128 && a.page_tokens >= 4 && page_shift(a.page_tokens) >= 0 && group <= 32 && a.q_start != nullptr &&
           a.ldq % 8 == 0 && a.ldo % 4 == 0 && a.kv_width % 8 == 0 && a.kv_width * a.page_tokens < (1 << 20) &&
           ((uintptr_t)a.q & 15) == 0 &&
           ((uintptr_t)a.out & (a.out_f32 ? 15 : 7)) == 0 && ((uintptr_t)a.k_cache & 15) == 0 && ((uintptr_t)a.v_cache & 15) == 0;
}

// The instantiation that a call needs; heads of one size here, everything else in attention_masked.hip.
template <int NDB>
static int step_ndb(const AttnArgs& a, const AttnCut& c) {
    const bool shaped = attn_shaped_scores(a);
    if (a.weights == 1) return launch_step<NDB, ATT_SIGMOID, NDB, false>(a, c);
    if (a.raw && shaped) return launch_step<NDB, ATT_SHAPED, NDB, true>(a, c);
    if (a.raw) return launch_step<NDB, ATT_PLAIN, NDB, true>(a, c);
    if (shaped) return launch_step<NDB, ATT_SHAPED, NDB, false>(a, c);
    return launch_step<NDB, ATT_PLAIN, NDB, false>(a, c);
}
template <int NDB>
static int prompt_ndb(const AttnArgs& a, const AttnCut& c) {
    if (a.weights == 1) return launch_prompt<NDB, ATT_SIGMOID, NDB>(a, c);
    if (attn_shaped_scores(a)) return launch_prompt<NDB, ATT_SHAPED, NDB>(a, c);
    return launch_prompt<NDB, ATT_PLAIN, NDB>(a, c);
}
static int run_cut(const AttnArgs& a, const AttnCut& c) {
    if (attn_masked_mode(a)) return attn_masked_run(a, c);
    switch (a.head_dim / 32) {
        case 1: return c.prompt ? prompt_ndb<1>(a, c) : step_ndb<1>(a, c);
        case 2: return c.prompt ? prompt_ndb<2>(a, c) : step_ndb<2>(a, c);
        case 3: return c.prompt ? prompt_ndb<3>(a, c) : step_ndb<3>(a, c);
        default: return c.prompt ? prompt_ndb<4>(a, c) : step_ndb<4>(a, c);
    }
}
static int merge_chunks(const AttnArgs& a, int n_chunks) {
    attn_merge_kernel<<<dim3(a.n_tokens, a.n_heads), WAVE, 0, a.stream>>>((const float*)a.workspace, (uint16_t*)a.out, a.ldo, a.n_heads,
                                                                        a.v_head_dim > 0 ? a.v_head_dim : a.head_dim, n_chunks, a.sink,
                                                                        a.sink_w, attn_extra(a));
    HFA_LAUNCH_CHECK("attn_merge");
    return 0;
}

static int attn_cu_count() {
    static int n = 0;
    if (n == 0) {
        int dev = 0;
        if (hipGetDevice(&dev) != hipSuccess || hipDeviceGetAttribute(&n, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || n <= 0)
            n = 256;
    }
    return n;
}

static int launch_prefill(const AttnArgs& a, int tpt, int cpt) {
    const int tile_tokens = 4 * tpt, kept = a.keep_first > 0 ? 1 : 0;        // kept keys are a chunk of their own
    const int dv = a.v_head_dim > 0 ? a.v_head_dim : a.head_dim;
    // One request: the number of tiles is known here, and with it whether all blocks are resident at once.
    const int n_tiles = a.n_seqs == 1 ? (a.n_tokens + tile_tokens - 1) / tile_tokens : 0;
    const int cus = attn_cu_count();
    int pair_from = n_tiles * a.n_kv_heads > cus && n_tiles * a.n_kv_heads <= 2 * cus ? cus : 0;
    // Fewer blocks than two a CU, each with a long walk over its request's keys: the keys are cut into
    // chunks of 256 or more over blockIdx.z until the machine is full, and attn_merge_kernel puts the
    // chunks' results together (portions of a few hundred tokens far into a long prompt).
    int n_chunks = 1, chunk_keys = a.max_seq_len;
    const long blocks = (long)a.n_kv_heads * ((a.n_tokens + tile_tokens - 1) / tile_tokens);
    // the keys that one tile can see: all of the sequence, or a window or masking chunk and the tile's own tokens (and the key
    // block that the cuts are aligned to); the cuts are made over these
    int reach = a.max_seq_len;
    if (a.mask_chunk > 0 && a.mask_chunk + tile_tokens + KB < reach) reach = a.mask_chunk + tile_tokens + KB;
    if (a.window > 0 && a.window + tile_tokens + KB < reach) reach = a.window + tile_tokens + KB;
    if (blocks < 2 * cus && reach >= 512 && a.workspace != nullptr) {
        long want = (2 * cus + blocks - 1) / blocks;
        if (want > reach / 256) want = reach / 256;
        if (want > MERGE_MAX_CHUNKS) want = MERGE_MAX_CHUNKS;
        const size_t per_chunk = (size_t)a.n_tokens * a.n_heads * (dv + 2) * sizeof(float);
        if ((size_t)(want + kept) * per_chunk > a.workspace_bytes) want = (long)(a.workspace_bytes / per_chunk) - kept;
        if (want > 1) {
            chunk_keys = (int)((reach + want - 1) / want + 63) / 64 * 64;
            n_chunks = (reach + chunk_keys - 1) / chunk_keys;
        }
    }
    if (n_chunks > 1) {
        pair_from = 0;
        n_chunks += kept;
    }
    AttnCut c = {};
    c.prompt = 1;
    c.tiles = (a.n_tokens + tile_tokens - 1) / tile_tokens + a.n_seqs;
    c.tpt = tpt;
    c.cpt = cpt;
    c.prompt_tiles = n_tiles;
    c.pair_from = pair_from;
    c.chunk_keys = chunk_keys;
    c.n_chunks = n_chunks;
    const int rc = run_cut(a, c);
    return rc || n_chunks == 1 ? rc : merge_chunks(a, n_chunks);
}

// A call in which some request brings this many tokens or more goes to the kernel for prompt portions,
// whole: it walks each request's keys in one piece. A caller that has requests with single tokens and
// long contexts beside prompt portions does better to make two calls, one below and one from this number up.
#define PROMPT_ROWS 16
extern "C" int hfa_attention_prompt_rows(void) { return PROMPT_ROWS; }

int attn_mfma_launch(const AttnArgs& a) {
    const int cpt = a.n_heads / a.n_kv_heads;              // columns per token: the heads of a group
    const int tpt = 32 / cpt;                              // tokens per tile
    // Steps with prompt portions: the kernel that shares keys and values between four waves.
    // That kernel has one block per 4 x tpt tokens and key/value head (and chunk of keys, when it has
    // few blocks). Very few tokens with long contexts (a token budget of 64 far into a long prompt)
    // fill its tiles badly: those go to the kernel below, one wave per tile, which also cuts the keys.
    const long prompt_blocks = ((long)(a.n_tokens + 4 * tpt - 1) / (4 * tpt)) * a.n_kv_heads;
    const bool few_long = 8 * prompt_blocks < attn_cu_count() && a.max_seq_len >= 1024 && a.workspace != nullptr;
    if (a.raw == nullptr && a.max_q_len >= PROMPT_ROWS && !few_long && a.page_tokens % 8 == 0 &&
        (a.n_tokens + 4 * tpt - 1) / (4 * tpt) + a.n_seqs <= 65535) {
        return launch_prefill(a, tpt, cpt);
    }
    const int tiles = a.max_q_len <= tpt ? a.n_seqs : (a.n_tokens + tpt - 1) / tpt + a.n_seqs;
    // Few waves and long contexts: cut the keys into chunks so that the machine is full.
    const long waves = (long)(a.max_q_len <= tpt ? a.n_seqs : (a.n_tokens + tpt - 1) / tpt) * a.n_kv_heads;
    int span = a.window > 0 && a.window + a.max_q_len < a.max_seq_len ? a.window + a.max_q_len : a.max_seq_len;
    if (a.mask_chunk > 0 && a.mask_chunk + a.max_q_len < span) span = a.mask_chunk + a.max_q_len;      // a masking chunk bounds the keys as a window does
    int n_chunks = 1, chunk_keys = a.max_seq_len;
    // How many waves in all is a measured choice. Head size 128 (7B shape): 512; with 1,024 a step took 1.3 % longer
    // at 64 sequences and 4.5 % longer at 8 sequences of 16,384 tokens, with 256 more than that. Head size 64 (0.5B
    // shape), where a wave has half the work per key: 1,024; with 512 a step of 64 sequences took 4.5 % longer; but no
    // chunk of fewer than 128 keys for either head size (with chunks of 64 keys a step of 8 sequences of the 0.5B shape at
    // 2,048 took 5 % longer, one of 16 2 %; one of 2 sequences of the 7B shape 2 % longer).
    const int fill = a.head_dim > 64 ? 512 : 1024;
    if (waves < fill && span > 128 && a.workspace) {
        int want = (int)((fill + waves - 1) / waves);
        const int most = (span + 127) / 128;
        if (want > most) want = most;
        // under a window or a mask by chunks the cuts are counted from the tile's first key block: they cover what a tile can see
        const int reach = attn_bounded(a.window, a.mask_chunk) && span + KB < a.max_seq_len ? span + KB : a.max_seq_len;
        chunk_keys = ((reach + want - 1) / want + KB - 1) / KB * KB;
        if (chunk_keys < 64) chunk_keys = 64;
        n_chunks = (reach + chunk_keys - 1) / chunk_keys;
        const int kept = a.keep_first > 0 ? 1 : 0, dv = a.v_head_dim > 0 ? a.v_head_dim : a.head_dim;
        if (n_chunks >= 2) n_chunks += kept;                // (the kept keys are a chunk of their own)
        const size_t need = (size_t)a.n_tokens * a.n_heads * n_chunks * (dv + 2) * sizeof(float);
        if (n_chunks < 2 || n_chunks > MERGE_MAX_CHUNKS || need > a.workspace_bytes) {
            n_chunks = 1;
            chunk_keys = a.max_seq_len;
        }
    }
    AttnCut c = {};
    c.tiles = tiles;
    c.tpt = tpt;
    c.cpt = cpt;
    c.chunk_keys = chunk_keys;
    c.n_chunks = n_chunks;
    const int rc = run_cut(a, c);
    return rc || n_chunks == 1 ? rc : merge_chunks(a, n_chunks);
}
