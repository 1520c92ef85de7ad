// Paged softmax attention, plain form: one wave per (token, query head), for any mix of
// prompt portions and decoded tokens, any head count and grouping, head_dim up to 256,
// with or without a window, fp32 or bf16 cache. Scores, softmax and the weighted sum are
// fp32; keys are visited in tiles of 64 aligned to absolute positions, in ascending order,
// so a token's result depends on its request's cache alone, never on the rest of the batch.
#include "api.h"
#include "common.h"
#include "attention_internal.h"

#define ATT_MAX_D 256
#define ATT_MAX_D_WIDE 640       // heads that hold a latent and a rotated part side by side

__device__ __forceinline__ float dot_row(const float* __restrict__ q_s, const bf16* __restrict__ kp, int D) {
    float dot = 0.f;
    if ((D & 7) == 0) {
        for (int d = 0; d < D; d += 8) {
            const uint4 u = *reinterpret_cast<const uint4*>(kp + d);
            const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
            for (int i = 0; i < 4; i++) {
                dot = fmaf(q_s[d + 2 * i], __uint_as_float(w[i] << 16), dot);
                dot = fmaf(q_s[d + 2 * i + 1], __uint_as_float(w[i] & 0xffff0000u), dot);
            }
        }
    } else {
        for (int d = 0; d < D; d++) dot = fmaf(q_s[d], to_f32(kp[d]), dot);
    }
    return dot;
}
__device__ __forceinline__ float dot_row(const float* __restrict__ q_s, const float* __restrict__ kp, int D) {
    float dot = 0.f;
    if ((D & 3) == 0) {
        for (int d = 0; d < D; d += 4) {
            const float4 u = *reinterpret_cast<const float4*>(kp + d);
            dot = fmaf(q_s[d], u.x, dot);
            dot = fmaf(q_s[d + 1], u.y, dot);
            dot = fmaf(q_s[d + 2], u.z, dot);
            dot = fmaf(q_s[d + 3], u.w, dot);
        }
    } else {
        for (int d = 0; d < D; d++) dot = fmaf(q_s[d], kp[d], dot);
    }
    return dot;
}

// CROSS: every query head's weights are applied to the values of EVERY key/value group (the whole value row, up to
// ATT_MAX_CROSS columns), and out is [token][G rounds][H heads][Dv]: round r of head h holds its weights on the values of
// group (h's group + r) mod G. A design that mixes the heads' weights after the softmax sums these (hfa_talk_mix).
#define ATT_MAX_CROSS 1024
// softcap > 0: score <- softcap tanh(score / softcap). weights 1: no softmax; a visible key weighs sigmoid(score + head_bias[h])
// (head_bias null: 0), and the weights are not normalised over the keys. dist_scale (null: none): the score is lowered by
// dist_scale[h] ln(1 + dist_rate[h] (i - j)) after the cap. sink with sink_w: the extra term's score is sink_w[h] instead of 0.
// rel (null: none): a number by distance, [head][rel_n], is added to the score. keep > 0: keys 0 .. keep - 1 are seen beside the
// window's. v_share key/value heads of keys read one head of values. A head's result is multiplied by out_mul sigmoid(gate[t, h])
// (gate null: by out_mul).
template <typename T, typename TO, bool CROSS, int MAXD>
__global__ __launch_bounds__(WAVE) void attn_generic_kernel(
    const T* __restrict__ q, int ldq, const T* __restrict__ kc, const T* __restrict__ vc, int kvw, int vw,
    const int* __restrict__ block_table, int max_blocks, const int* __restrict__ token_slot,
    const int* __restrict__ positions, TO* __restrict__ out, int ldo, int H, int G, int D, int Dv, int page_tokens,
    int window, int mask_chunk, float scale, const float* __restrict__ slopes, int sink, float softcap, int weights,
    const float* __restrict__ head_bias, const float* __restrict__ sink_w, const float* __restrict__ dist_scale,
    const float* __restrict__ dist_rate, int keep, int v_share, const float* __restrict__ rel, int rel_n, const void* __restrict__ gate,
    int gate_bf16, int ldg, float out_mul) {
    __shared__ float q_s[MAXD];
    __shared__ float p_s[WAVE];
    __shared__ int row_s[WAVE];
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const int kvh = h / (H / G);
    const int pos = positions[t];
    const int* bt = block_table + (size_t)token_slot[t] * max_blocks;
    for (int d = lane; d < D; d += WAVE) q_s[d] = to_f32(q[(size_t)t * ldq + h * D + d]);
    __syncthreads();
    const int lo = first_visible(pos, window, mask_chunk);
    const float slope = slopes ? slopes[h] : 0.f;           // a position encoding that enters the scores
    float m = -INFINITY, l = 0.f;
    constexpr int NACC = (CROSS ? ATT_MAX_CROSS : MAXD) / WAVE;
    const float inv_cap = softcap > 0.f ? 1.0f / softcap : 0.f;
    const float hb = (weights == 1 && head_bias) ? head_bias[h] : 0.f;
    const float r1 = dist_scale ? dist_scale[h] : 0.f, r2 = dist_scale ? dist_rate[h] : 0.f;
    const int v_first = CROSS ? 0 : kvh / v_share * Dv, v_cols = CROSS ? G * Dv : Dv;      // the columns of a value row that this head reads
    float acc[NACC];
#pragma unroll
    for (int i = 0; i < NACC; i++) acc[i] = 0.f;

    const int window_tile = (lo / WAVE) * WAVE;
    for (int j0 = keep > 0 ? 0 : window_tile; j0 <= pos; j0 += WAVE) {
        if (j0 < window_tile && j0 >= keep) j0 = window_tile;           // from the kept keys to the window's
        const int j = j0 + lane;
        const bool valid = (j >= lo || j < keep) && j <= pos;
        float s = -INFINITY;
        int row = 0;
        if (valid) {
            row = bt[j / page_tokens] * page_tokens + j % page_tokens;
            s = dot_row(q_s, kc + (size_t)row * kvw + kvh * D, D) * scale;
            if (slopes) s += slope * (float)(j - pos);
            if (softcap > 0.f) s = softcap * tanhf(s * inv_cap);
            if (dist_scale) s -= r1 * log1pf(r2 * (float)(pos - j));
            if (rel) s += rel[(size_t)h * rel_n + (pos - j < rel_n ? pos - j : rel_n - 1)];
        }
        float corr = 1.f, p;
        if (weights == 1) {
            p = valid ? 1.0f / (1.0f + expf(-(s + hb))) : 0.f;
        } else {
            // every tile holds at least one visible key, so the maximum is finite
            const float mn = fmaxf(m, wave_max(s));
            corr = expf(m - mn);
            p = valid ? expf(s - mn) : 0.f;
            l = l * corr + wave_sum(p);
            m = mn;
        }
        p_s[lane] = p;
        row_s[lane] = row;
        __syncthreads();
        const int first = lo > j0 && j0 >= keep ? lo - j0 : 0;
        const int last = pos - j0 < WAVE - 1 ? pos - j0 : WAVE - 1;
#pragma unroll
        for (int i = 0; i < NACC; i++) acc[i] *= corr;
        for (int jj = first; jj <= last; jj++) {
            if (j0 + jj < lo && j0 + jj >= keep) continue;               // (a kept tile's end; uniform)
            const float pj = p_s[jj];
            // values lie transposed inside their page: [page][column][token]
            const int vr = row_s[jj];
            const T* vp = vc + (size_t)(vr / page_tokens) * page_tokens * vw + (size_t)v_first * page_tokens +
                          vr % page_tokens;
#pragma unroll
            for (int i = 0; i < NACC; i++) {
                const int d = lane + WAVE * i;
                if (d < v_cols) acc[i] = fmaf(pj, to_f32(vp[(size_t)d * page_tokens]), acc[i]);
            }
        }
        __syncthreads();
    }
    // the term that has no value: its score is the head's number, or 0
    float factor = out_mul;
    if (gate) {
        const size_t gi = (size_t)t * ldg + h;
        factor /= 1.0f + expf(-(gate_bf16 ? to_f32(((const bf16*)gate)[gi]) : ((const float*)gate)[gi]));
    }
    const float inv = weights == 1 ? factor : factor / (sink ? l + expf((sink_w ? sink_w[h] : 0.f) - m) : l);
#pragma unroll
    for (int i = 0; i < NACC; i++) {
        const int d = lane + WAVE * i;
        if (d >= v_cols) continue;
        if (CROSS) {
            const int vh = d / Dv, r = (vh - kvh + G) % G;
            out[(size_t)t * ldo + ((size_t)r * H + h) * Dv + d % Dv] = from_f32<TO>(acc[i] * inv);
        } else {
            out[(size_t)t * ldo + h * Dv + d] = from_f32<TO>(acc[i] * inv);
        }
    }
}

int attn_generic_launch(const AttnArgs& a, int dtype, const float* slopes, int cross) {
    const int D = a.head_dim, Dv = a.v_head_dim;
    HFA_REQUIRE(!cross || a.n_kv_heads * Dv <= ATT_MAX_CROSS, "paged_attention: a value row of %d columns exceeds what one wave "
                "applies its weights to (%d)", a.n_kv_heads * Dv, ATT_MAX_CROSS);
    const bool wide = D > ATT_MAX_D || Dv > ATT_MAX_D;
    HFA_REQUIRE(D <= ATT_MAX_D_WIDE && Dv <= ATT_MAX_D_WIDE && !(wide && cross),
                "paged_attention: head_dim %d (values: %d) exceeds the kernel's limit %d", D, Dv, ATT_MAX_D_WIDE);
    HFA_REQUIRE(a.weights == 0 || (a.weights == 1 && !a.sink), "paged_attention: weights are a softmax (0) or sigmoids without a sink term (1)");
    HFA_REQUIRE(a.n_heads <= 65535, "paged_attention: %d heads exceed the grid", a.n_heads);
    dim3 grid(a.n_tokens, a.n_heads);
#define ATT_GO(T, TO, CROSS, MAXD)                                                                                                \
    attn_generic_kernel<T, TO, CROSS, MAXD><<<grid, WAVE, 0, a.stream>>>(                                                         \
        (const T*)a.q, a.ldq, (const T*)a.k_cache, (const T*)a.v_cache, a.kv_width, a.v_width, a.block_table, a.max_blocks, a.token_slot, \
        a.positions, (TO*)a.out, a.ldo, a.n_heads, a.n_kv_heads, D, Dv, a.page_tokens, a.window, a.mask_chunk, a.scale, slopes,    \
        a.sink, a.softcap, a.weights, a.head_bias, a.sink_w, a.dist_scale, a.dist_rate, a.keep_first, a.v_share, a.rel, a.rel_n, a.gate, \
        a.gate_bf16, a.ldg, a.out_mul)
#define ATT_SIZES(T, TO) \
    do { if (cross) ATT_GO(T, TO, true, ATT_MAX_D); else if (wide) ATT_GO(T, TO, false, ATT_MAX_D_WIDE); else ATT_GO(T, TO, false, ATT_MAX_D); } while (0)
    if (dtype == HFA_F32) ATT_SIZES(float, float);
    else if (!a.out_f32) ATT_SIZES(bf16, bf16);
    else if (wide) ATT_GO(bf16, float, false, ATT_MAX_D_WIDE);
    else ATT_GO(bf16, float, false, ATT_MAX_D);
#undef ATT_SIZES
#undef ATT_GO
    HFA_LAUNCH_CHECK("paged_attention");
    return 0;
}

// cos_sin[t][0 .. half) = cos(positions[t] * inv_freq[i]), [half .. 2 half) the sines: the angles of src/model.c:472-476
// as rope_store forms them, once for all the layers of a step.
__global__ void rope_table_kernel(const int* __restrict__ positions, const float* __restrict__ inv_freq, int half,
                                  float* __restrict__ out) {
    const int t = blockIdx.x;
    const float pos = (float)positions[t];
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
        float sn, cs;
        sincosf(pos * inv_freq[i], &sn, &cs);
        out[(size_t)t * 2 * half + i] = cs;
        out[(size_t)t * 2 * half + half + i] = sn;
    }
}

extern "C" int hfa_rope_table(const int* positions, const float* inv_freq, int half, float* out, int n_tokens, hipStream_t stream) {
    HFA_REQUIRE(positions && inv_freq && out && half > 0 && n_tokens > 0, "rope_table: bad arguments");
    rope_table_kernel<<<n_tokens, half < 256 ? (half + 63) / 64 * 64 : 256, 0, stream>>>(positions, inv_freq, half, out);
    HFA_LAUNCH_CHECK("rope_table");
    return 0;
}

// Whether hfa_decode_attention takes a step: bf16 on the matrix cores, one head size of 32 to 128 in steps of 32
// for keys and values, rotation of whole heads (rot_dim == head_dim) or none.
extern "C" int hfa_decode_attention_supports(int n_heads, int n_kv_heads, int head_dim, int rot_dim, int page_tokens,
                                             int kv_width, int ld_raw, int ldo) {
    if (n_kv_heads <= 0 || n_heads % n_kv_heads != 0 || !(rot_dim == head_dim || rot_dim == 0) || ld_raw % 4 != 0) return 0;
    AttnArgs a = {};
    a.scale = 1.f; a.head_dim = head_dim; a.page_tokens = page_tokens; a.n_heads = n_heads; a.n_kv_heads = n_kv_heads;
    a.q_start = (const int*)16; a.ldq = 8; a.ldo = ldo; a.kv_width = kv_width;
    return attn_mfma_supports(a) ? 1 : 0;
}

// Attention of decoded tokens (one token a request) whose queries, new keys and new values are still the 32-bit rows
// [q | k | v] that the product left (`raw`, row stride ld_raw, bias added): rotation of queries and keys, the store
// of the new key and value into the cache rows slot_map[t], and attention over the cache in one kernel (and the merge
// of the key chunks). cos_sin: hfa_rope_table's output for these tokens, or null for no rotation. slot_map null: the
// rows hold queries only ([q], a layer that reads the keys and values another layer has stored). Everything else as
// in hfa_paged_attention, whose result with hfa_rope_store before it this equals.
extern "C" int hfa_decode_attention(const float* raw, int ld_raw, const float* cos_sin, void* k_cache, void* v_cache,
                                    int kv_width, const int* slot_map, const int* block_table, int max_blocks,
                                    const int* token_slot, const int* positions, const int* q_start, int n_seqs,
                                    int max_seq_len, void* out, int ldo, int n_heads, int n_kv_heads, int head_dim,
                                    int page_tokens, int window, int mask_chunk, float scale, float softcap,
                                    const float* dist_scale, const float* dist_rate, void* workspace,
                                    size_t workspace_bytes, hipStream_t stream) {
    HFA_REQUIRE(softcap >= 0.f && (!dist_scale) == (!dist_rate), "decode_attention: a negative soft cap, or half of a distance term");
    HFA_REQUIRE(raw && k_cache && v_cache && block_table && token_slot && positions && q_start && out,
                "decode_attention: a null argument");
    HFA_REQUIRE(n_seqs > 0 && max_seq_len > 0 && max_blocks > 0 && window >= 0 && mask_chunk >= 0, "decode_attention: bad sizes");
    HFA_REQUIRE(ld_raw >= (n_heads + (slot_map ? 2 * n_kv_heads : 0)) * head_dim && ldo >= n_heads * head_dim && kv_width >= n_kv_heads * head_dim,
                "decode_attention: a row stride is smaller than its row");
    AttnArgs a = {nullptr, 8, k_cache, v_cache, kv_width, block_table, max_blocks, token_slot, positions, q_start,
                  n_seqs, 1, max_seq_len, out, ldo, n_seqs, n_heads, n_kv_heads, head_dim, page_tokens,
                  window, scale, workspace, workspace_bytes, stream, raw, ld_raw, cos_sin, slot_map, mask_chunk, 0, 0,
                  softcap, 0, nullptr, nullptr, dist_scale, dist_rate};
    a.out_mul = 1.f;
    HFA_REQUIRE(((uintptr_t)raw & 15) == 0 && (cos_sin == nullptr || ((uintptr_t)cos_sin & 15) == 0) && attn_mfma_supports(a),
                "decode_attention: this shape is not taken (see hfa_decode_attention_supports)");
    return attn_mfma_launch(a);
}

extern "C" int hfa_paged_attention(const void* q, int dtype, int ldq, const void* k_cache, const void* v_cache,
                                   int kv_width, int v_width, const int* block_table, int max_blocks, const int* token_slot,
                                   const int* positions, const int* q_start, int n_seqs, int max_q_len,
                                   int max_seq_len, void* out, int ldo, int n_tokens, int n_heads, int n_kv_heads,
                                   int head_dim, int v_head_dim, int page_tokens, int window, int mask_chunk, float scale,
                                   const float* slopes, int sink, int cross_values, float softcap, int weights,
                                   const float* head_bias, const float* sink_w, const float* dist_scale, const float* dist_rate,
                                   int v_share, int keep_first, const float* rel, int rel_n, const void* gate, int gate_dtype, int ldg,
                                   float out_mul, int out_dtype, void* workspace, size_t workspace_bytes,
                                   int force_plain, hipStream_t stream) {
    HFA_REQUIRE(n_tokens > 0 && n_heads > 0 && n_kv_heads > 0 && head_dim > 0 && v_head_dim > 0 && page_tokens > 0 && max_blocks > 0,
                "paged_attention: bad sizes");
    HFA_REQUIRE(n_heads % n_kv_heads == 0, "paged_attention: %d heads are not a multiple of %d key/value heads",
                n_heads, n_kv_heads);
    HFA_REQUIRE(v_share > 0 && n_kv_heads % v_share == 0 && keep_first >= 0 && (!rel || rel_n > 0) && (out_dtype == dtype || out_dtype == HFA_F32) &&
                    (!gate || (ldg >= n_heads && (gate_dtype == HFA_F32 || gate_dtype == HFA_BF16))),
                "paged_attention: bad value heads, kept keys, distance table, gate or output type");
    HFA_REQUIRE(!cross_values || (v_share == 1 && !keep_first && !rel && !gate && out_mul == 1.f && out_dtype == dtype),
                "paged_attention: mixed heads go without kept keys, a distance table, gates and shared values");
    HFA_REQUIRE(kv_width >= n_kv_heads * head_dim && v_width >= n_kv_heads / v_share * v_head_dim && ldq >= n_heads * head_dim &&
                    ldo >= n_heads * v_head_dim * (cross_values ? n_kv_heads : 1),
                "paged_attention: a row stride is smaller than its row");
    HFA_REQUIRE(window >= 0 && mask_chunk >= 0, "paged_attention: negative window or masking chunk");
    HFA_REQUIRE(dtype == HFA_F32 || dtype == HFA_BF16, "paged_attention: unknown dtype %d", dtype);
    AttnArgs a = {q, ldq, k_cache, v_cache, kv_width, block_table, max_blocks, token_slot, positions, q_start,
                  n_seqs, max_q_len, max_seq_len, out, ldo, n_tokens, n_heads, n_kv_heads, head_dim, page_tokens,
                  window, scale, workspace, workspace_bytes, stream, nullptr, 0, nullptr, nullptr, mask_chunk, sink ? 1 : 0, 0,
                  softcap, weights, head_bias, sink ? sink_w : nullptr, dist_scale, dist_rate};
    a.v_head_dim = v_head_dim;
    a.v_width = v_width;
    a.v_share = v_share;
    a.keep_first = window > 0 || mask_chunk > 0 ? keep_first : 0;           // (otherwise everything is in sight)
    a.rel = rel;
    a.rel_n = rel ? rel_n : 0;
    a.gate = gate;
    a.gate_bf16 = gate && gate_dtype == HFA_BF16;
    a.ldg = ldg;
    a.out_mul = out_mul;
    a.out_f32 = dtype == HFA_BF16 && out_dtype == HFA_F32;
    // the matrix-core kernels take no slopes: scores with a linear position term go the plain way
    HFA_REQUIRE(softcap >= 0.f && (weights == 0 || weights == 1), "paged_attention: a negative soft cap or an unknown kind of weights");
    HFA_REQUIRE((!dist_scale) == (!dist_rate) && (!dist_scale || (weights == 0 && !slopes && !cross_values)) && (!sink_w || (sink && !cross_values)),
                "paged_attention: a distance term has two numbers a head and goes with a softmax over a head's own values, a sink's scores with a sink");
    // sigmoid weights and shaped scores (a soft cap, a distance term) they take for a head's own values
    if (!force_plain && !slopes && (weights == 1 ? !cross_values && !sink : !cross_values || (softcap == 0.f && v_head_dim == head_dim && v_width == kv_width)) && dtype == HFA_BF16 &&
        !(v_head_dim != head_dim && attn_shared_supports(a, v_head_dim, v_width)) && attn_mfma_supports(a)) {
        if (!cross_values) return attn_mfma_launch(a);
        // single tokens: one pass over the cache for all rounds
        int chunk_keys = 0, n_chunks = 0;
        if (attn_cross_supports(a, &chunk_keys, &n_chunks)) return attn_cross_launch(a, chunk_keys, n_chunks);
        // The weights on every group's values, on the matrix cores: one pass a round, the scores taken again each time (a
        // round's output lies n_heads * head_dim further on in the token's row, whose stride ldo spans all rounds). The
        // passes share the workspace; they run one after the other on the stream.
        for (int r = 0; r < n_kv_heads; r++) {
            AttnArgs b = a;
            b.v_rot = r;
            b.out = (char*)out + (size_t)r * n_heads * head_dim * 2;
            const int rc = attn_mfma_launch(b);
            if (rc) return rc;
        }
        return 0;
    }
    // one key/value head with wide keys and values of a size of their own, read by every query head
    if (!force_plain && !slopes && !cross_values && dtype == HFA_BF16 && attn_shared_supports(a, v_head_dim, v_width))
        return attn_shared_launch(a, v_head_dim);
    return attn_generic_launch(a, dtype, slopes, cross_values ? 1 : 0);
}
