// Paged softmax attention on the matrix cores (bf16 cache, fp32 scores, softmax and sums).
//
// One wave owns up to 32 "columns": the query heads of one key/value head for a few
// consecutive tokens of one request (a prompt portion: several tokens; a decoded token: one).
// The columns share every key and value they read, so grouped heads cost one pass over the
// cache. Keys are walked in blocks of 32, aligned to absolute positions:
//
//   S^T[key, col] = K[key, :] . Q[col, :]        v_mfma_f32_32x32x16_bf16, A = 32 keys x 16 dims
//                                                straight from the cache, B = queries in registers
//   online softmax per column: a column is one lane pair (l, l ^ 32), so maximum and sum need
//   one cross-lane step; the probabilities a lane holds are exactly the B operand of
//   O^T[dim, col] += V^T[dim, key] . P^T[key, col]   A = values, which the cache keeps transposed
//                                                inside a page, so 4 consecutive keys of one
//                                                dimension are one 8-byte load.
// The order of keys inside a 16-key product is permuted the same way in both operands of the
// second product, so the probabilities never leave their registers.
//
// When a step has few columns (decode) the key range is cut into chunks over blockIdx.z; each
// wave writes (max, sum, unnormalised output) for its chunk and a second kernel merges them in
// chunk order. Keys and values come from global memory in operand layout, without a barrier.
//
// The kernels are templates: attention_mfma.hip holds the instantiations with heads of one size, attention_masked.hip those
// with value heads of a size of their own, with a table of distance terms or with a sequence's first keys kept in sight.
#pragma once
#include "attention_internal.h"
#include "common.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float floatx16 __attribute__((ext_vector_type(16)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

#define KB 32
#define PG_MAX 512
#define NEG_BIG (-1.0e30f)

// The running maximum of a column follows the scores only when they pass it by more than this (in
// powers of two): probabilities then reach 2^MAX_SLACK at most, which bf16 and the fp32 sums hold
// as exactly as values up to 1, and the accumulators are rescaled in few blocks instead of in most.
#define MAX_SLACK 8.0f

// 2^x by the hardware instruction (arguments here are at most MAX_SLACK or the -1e30 sentinel's
// difference, never subnormal results that matter).
__device__ __forceinline__ float fast_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
// A column's scores lie in lanes c and c + 32. v_permlane32_swap exchanges the upper half of one
// register with the lower half of another; with the same value in both, every lane then holds
// the lower lane's value in the first and the upper lane's in the second: maximum and sum of the
// pair without a trip through LDS, and the same bits in both lanes.
__device__ __forceinline__ float pair_max(float x) {
    const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    return fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
}
__device__ __forceinline__ float pair_sum(float x) {
    const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    return __uint_as_float(r[0]) + __uint_as_float(r[1]);
}

// Two probabilities as a pair of bf16, round to nearest even: one v_cvt_pk_bf16_f32 on gfx950.
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
typedef float floatx2 __attribute__((ext_vector_type(2)));
__device__ __forceinline__ uint32_t prob_pair(float lo, float hi) {
    const floatx2 f = {lo, hi};
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(f, bf16x2));
}

union Frag {
    uint4 u;
    uint2 h[2];
    bf16x8 v;
};

// FUSED (decoded tokens only, one token a tile): queries, the new key and the new value are not in `q` and in the
// cache yet but in `raw`, fp32 rows [q | k | v] as the product left them (bias added). The wave rotates its queries
// while it loads them (cosines and sines of the token's angles come from `cs`, [token][D / 2 cosines, D / 2 sines];
// rot_dim = D, or no rotation when cs is null); the wave whose keys include the token's own position rotates the
// new key, stores it and the new value into the cache (rows slot_map[token]) for the steps to come, and uses them
// from LDS itself, since what the cache row held before is not the token's. What rope_store would have done in a
// kernel and a pass over memory of its own.
// MODE ATT_SIGMOID: the weights are no softmax but sigmoid(capped score + head_bias[head]) (see hfa_paged_attention); records of key
// chunks then carry maximum 0 and sum 1 in the first chunk and 0 in the others, so that the merge adds the chunks up.
// MODE ATT_SHAPED: a softmax whose scores are soft-capped and/or lowered by a term of the distance first.
#define ATT_PLAIN 0
#define ATT_SIGMOID 1
#define ATT_SHAPED 2
// MODE ATT_REL: a softmax whose scores get a number of a table by (head, distance) added.
// MODE ATT_KEEP: a softmax under a window beside which the first `keep` keys of the sequence stay in sight.
#define ATT_REL 3
#define ATT_KEEP 4
#define LOG2E 1.4426950408889634f

// A score in powers of two from the product `dot`: dot * scale (natural; sc = the scale), capped by c tanh(s / c) = c (1 - 2 / (1 +
// exp(2 s / c))) where c > 0 (cap2 = 2 log2(e) / c), lowered by r1 ln(1 + r2 d).
__device__ __forceinline__ float shaped_score(float dot, float sc, float softcap, float cap2, bool dist, float r1, float r2, float d) {
    float sv = dot * sc;
    if (softcap > 0.f) sv = softcap * (1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + fast_exp2(sv * cap2)));
    sv *= LOG2E;
    if (dist) sv = fmaf(-r1, __builtin_amdgcn_logf(fmaf(r2, d, 1.0f)), sv);       // r1 ln(x) log2(e) = r1 log2(x)
    return sv;
}

// What the modes above and a result's destination need beside the arguments that every instantiation reads.
struct AttnExtra {
    const float* rel; int rel_n, rel_lds;   // ATT_REL: [query head][rel_n] by distance (beyond: the last); staged in LDS or not
    int keep;                               // ATT_KEEP: keys 0 .. keep - 1 are seen by every later query
    int v_share;                            // key/value heads of keys that share one head of values
    int vw;                                 // the value rows' width
    const void* gate; int gate_bf16, ldg;   // [token][query head]: a head's result is multiplied by sigmoid(gate); null: none
    float out_mul;                          // and by this
    int out_f32;                            // results leave in 32 bits
};

__device__ __forceinline__ float head_factor(const AttnExtra& ex, int tok, int head) {
    if (!ex.gate) return ex.out_mul;
    const size_t i = (size_t)tok * ex.ldg + head;
    const float z = ex.gate_bf16 ? __uint_as_float((uint32_t)((const uint16_t*)ex.gate)[i] << 16) : ((const float*)ex.gate)[i];
    return ex.out_mul / (1.0f + expf(-z));
}

// A group's rows of the table into LDS (dynamic, cpt * rel_n values), in powers of two.
__device__ __forceinline__ void stage_rel(const AttnExtra& ex, float* rel_s, int first_head, int n_heads, int tid, int threads) {
    const float* src = ex.rel + (size_t)first_head * ex.rel_n;
    for (int i = tid; i < n_heads * ex.rel_n; i += threads) rel_s[i] = src[i] * LOG2E;
}
// The terms of this lane's sixteen keys of a block (see the kernels for their order), in powers of two.
__device__ __forceinline__ void rel_terms(const AttnExtra& ex, const float* rel_s, int row_in_group, int head, int pos, int key0, int half,
                                          float (&b)[16]) {
    const int last = ex.rel_n - 1;
    if (ex.rel_lds) {
        const float* t = rel_s + row_in_group * ex.rel_n;
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int d = pos - (key0 + 8 * (r / 4) + 4 * half + (r % 4));
            b[r] = t[d < 0 ? 0 : d > last ? last : d];
        }
    } else {
        const float* t = ex.rel + (size_t)head * ex.rel_n;
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int d = pos - (key0 + 8 * (r / 4) + 4 * half + (r % 4));
            b[r] = t[d < 0 ? 0 : d > last ? last : d] * LOG2E;
        }
    }
}

// ATT_KEEP: the kept keys that lie in whole blocks before the first block of the window (first_block its first key, a
// multiple of KB): 0 .. kept_before(...) - 1; the others are seen on the window's own walk.
__device__ __forceinline__ int kept_before(int keep, int first_block) { return keep < first_block ? keep : first_block; }

template <int NDB, bool SPLIT, bool FUSED, int MODE = ATT_PLAIN, int VDB = NDB>
__global__ __launch_bounds__(WAVE) void attn_mfma_kernel(
    const uint16_t* __restrict__ q, int ldq, const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc, int kvw,
    const int* __restrict__ block_table, int max_blocks, const int* __restrict__ token_slot,
    const int* __restrict__ positions, const int* __restrict__ q_start, int n_seqs, uint16_t* __restrict__ out,
    int ldo, float* __restrict__ partial, int H, int psh, int window, int mask_chunk, float scale_log2e, int tpt, int cpt,
    int chunk_keys, int n_chunks, int one_tile_each, const float* __restrict__ raw, int ld_raw,
    const float* __restrict__ cs, const int* __restrict__ slot_map, int G, int sink, int v_rot, float softcap,
    const float* __restrict__ head_bias, const float* __restrict__ sink_w,
    const float* __restrict__ dist_scale, const float* __restrict__ dist_rate, AttnExtra ex) {
    constexpr int D = NDB * 32, KS = D / 16, DV = VDB * 32;
    constexpr bool SIG = MODE == ATT_SIGMOID, REL = MODE == ATT_REL, KEEP = MODE == ATT_KEEP;
    static_assert(!FUSED || NDB == VDB, "the fused prologue knows one head size");
    const int P = 1 << psh;                                // tokens per page, a power of two
    const int lane = threadIdx.x, col = lane & 31, half = lane >> 5;
    const int g = blockIdx.y, chunk = blockIdx.z;
    // The group whose values the weights are applied to: the heads' own, or (v_rot > 0, never with FUSED) the group
    // v_rot further on, for designs that mix the heads' weights after the softmax (see hfa_talk_mix).
    const int gv = VDB != NDB || KEEP || REL ? g / ex.v_share : g + v_rot < G ? g + v_rot : g + v_rot - G;
    const int vvw = VDB != NDB || KEEP || REL ? ex.vw : kvw;
    const int keep = KEEP ? ex.keep : 0;

    // ---- the tile's request and tokens: tiles are numbered request by request ----
    int tile = blockIdx.x, t0 = -1, t_end = 0;
    if (one_tile_each) {                                   // no request has more tokens than a tile: tile s is request s
        if (tile < n_seqs) {
            t0 = q_start[tile];
            t_end = q_start[tile + 1];
        }
    } else
    for (int s = 0; s < n_seqs; s++) {
        const int a = q_start[s], b = q_start[s + 1];
        const int nt = (b - a + tpt - 1) / tpt;
        if (tile < nt) {
            t0 = a + tile * tpt;
            t_end = t0 + tpt < b ? t0 + tpt : b;
            break;
        }
        tile -= nt;
    }
    if (t0 < 0) return;                                    // the grid is an upper bound on the tiles

    const int n_cols = (t_end - t0) * cpt;
    const bool col_ok = col < n_cols;
    const int my_tok = col_ok ? t0 + col / cpt : t0;
    const int my_head = g * cpt + (col_ok ? col % cpt : 0);
    const float hb = (SIG && head_bias) ? head_bias[my_head] : 0.f;
    const bool dist = MODE == ATT_SHAPED && dist_scale != nullptr;
    const float r1 = dist ? dist_scale[my_head] : 0.f, r2 = dist ? dist_rate[my_head] : 0.f;
    const int pos = positions[my_tok];
    const int pos_first = positions[t0], hi = positions[t_end - 1];
    int k_begin = first_visible(pos_first, window, mask_chunk);
    int k_end = hi;
    // ATT_KEEP: the keys kept in sight before the window's first block are a walk of their own (of the first chunk, if the keys
    // are cut: the others then count from the second)
    const int n_kept = KEEP ? kept_before(keep, k_begin / KB * KB) : 0, kept_chunk = keep > 0 ? 1 : 0;
    if (SPLIT && kept_chunk && chunk == 0) {
        k_end = n_kept - 1 < hi ? n_kept - 1 : hi;
    } else if (SPLIT) {
        // Under a window or a mask by chunks the tile's keys begin far into the sequence: the cuts are then counted from the
        // first key block that the tile sees, not from key 0 (whose chunks would mostly hold nothing).
        const int c_lo = (attn_bounded(window, mask_chunk) ? k_begin / KB * KB : 0) + (chunk - kept_chunk) * chunk_keys;
        k_begin = k_begin > c_lo ? k_begin : c_lo;
        k_end = k_end < c_lo + chunk_keys - 1 ? k_end : c_lo + chunk_keys - 1;
    }
    // visible keys of this lane's column: [vlo, vhi]
    int vlo = first_visible(pos, window, mask_chunk) > k_begin ? first_visible(pos, window, mask_chunk) : k_begin;
    int vhi = col_ok ? (pos < k_end ? pos : k_end) : -1;
    const int* bt = block_table + (size_t)token_slot[t0] * max_blocks;

    // The query fragments stay in registers: read from LDS one by one before each product, they
    // cost an LDS round trip a product that a single wave on its SIMD has nothing to hide behind.
    Frag qf[KS];
    __shared__ __attribute__((aligned(16))) uint16_t new_s[FUSED ? 2 * D : 8];     // the token's own key (rotated) and value
    bool owns_new = false;                                 // this wave's keys include the token's own position
    if (!FUSED) {
        const uint16_t* qp = q + (size_t)my_tok * ldq + my_head * D + half * 8;
#pragma unroll
        for (int ks = 0; ks < KS; ks++)
            qf[ks].u = col_ok ? *reinterpret_cast<const uint4*>(qp + ks * 16) : make_uint4(0, 0, 0, 0);
    }
    // FUSED: called once the first blocks of keys and values are on their way, so that the trip for the 32-bit rows
    // is not a trip of its own at the head of the kernel
    auto fused_prologue = [&]() {
        // A head's fragments ks and ks + KS / 2 hold the two halves of its rotated pairs (i, i + D / 2), i = 16 ks + 8 half + e.
        // Everything a pass needs from memory is asked for before anything is computed (left alone, the compiler asks,
        // waits and computes fragment by fragment: eight trips to L2 one after the other), in two passes over the
        // fragments so that the registers suffice.
        const float* row = raw + (size_t)my_tok * ld_raw;
        const float* qsrc = row + my_head * D + half * 8;
        const float* ksrc = row + (H + g) * D + half * 8;
        const float* cp = cs ? cs + (size_t)my_tok * D + half * 8 : nullptr;
        // uniform: hi is the token's own position. Without slot_map the rows hold queries only (a layer that reads another
        // layer's keys and values, which that layer has stored already): nothing is new.
        owns_new = slot_map != nullptr && k_begin <= hi && hi <= k_end;
        const int slot = owns_new ? slot_map[my_tok] : 0;
        float vraw[NDB];
        if (owns_new && half == 0) {
#pragma unroll
            for (int db = 0; db < NDB; db++) vraw[db] = row[(H + G) * D + g * D + 32 * db + col];
        }
        // (x0, x1) -> (x0 c - x1 s, x0 s + x1 c), src/model.c:488-490; without rotation the values pass as they are
        auto lo_of = [&](float x0, float x1, float c, float s) { return cp ? x0 * c - x1 * s : x0; };
        auto hi_of = [&](float x0, float x1, float c, float s) { return cp ? x0 * s + x1 * c : x1; };
        auto two = [](float a, float b) { return (uint32_t)bf16_bits(a) | ((uint32_t)bf16_bits(b) << 16); };
        auto turn = [&](const float4 (&lo)[2], const float4 (&hh)[2], const float4 (&c)[2], const float4 (&sn)[2], Frag& fl, Frag& fh) {
            fl.u = make_uint4(two(lo_of(lo[0].x, hh[0].x, c[0].x, sn[0].x), lo_of(lo[0].y, hh[0].y, c[0].y, sn[0].y)),
                              two(lo_of(lo[0].z, hh[0].z, c[0].z, sn[0].z), lo_of(lo[0].w, hh[0].w, c[0].w, sn[0].w)),
                              two(lo_of(lo[1].x, hh[1].x, c[1].x, sn[1].x), lo_of(lo[1].y, hh[1].y, c[1].y, sn[1].y)),
                              two(lo_of(lo[1].z, hh[1].z, c[1].z, sn[1].z), lo_of(lo[1].w, hh[1].w, c[1].w, sn[1].w)));
            fh.u = make_uint4(two(hi_of(lo[0].x, hh[0].x, c[0].x, sn[0].x), hi_of(lo[0].y, hh[0].y, c[0].y, sn[0].y)),
                              two(hi_of(lo[0].z, hh[0].z, c[0].z, sn[0].z), hi_of(lo[0].w, hh[0].w, c[0].w, sn[0].w)),
                              two(hi_of(lo[1].x, hh[1].x, c[1].x, sn[1].x), hi_of(lo[1].y, hh[1].y, c[1].y, sn[1].y)),
                              two(hi_of(lo[1].z, hh[1].z, c[1].z, sn[1].z), hi_of(lo[1].w, hh[1].w, c[1].w, sn[1].w)));
        };
        constexpr int HALF_KS = KS / 2, PASS = HALF_KS > 2 ? 2 : HALF_KS;         // fragments of a half head per pass
        Frag kn[KS];
#pragma unroll
        for (int k0 = 0; k0 < HALF_KS; k0 += PASS) {
            float4 c[PASS][2], sn[PASS][2], ql[PASS][2], qh[PASS][2], kl[PASS][2], kh[PASS][2];
#pragma unroll
            for (int j = 0; j < PASS; j++) {
                const int ks = k0 + j;
                if (ks < HALF_KS) {
#pragma unroll
                    for (int u = 0; u < 2; u++) {
                        c[j][u] = make_float4(1.f, 1.f, 1.f, 1.f);
                        sn[j][u] = make_float4(0.f, 0.f, 0.f, 0.f);
                        if (cp) {
                            c[j][u] = *reinterpret_cast<const float4*>(cp + ks * 16 + 4 * u);
                            sn[j][u] = *reinterpret_cast<const float4*>(cp + D / 2 + ks * 16 + 4 * u);
                        }
                        ql[j][u] = *reinterpret_cast<const float4*>(qsrc + ks * 16 + 4 * u);
                        qh[j][u] = *reinterpret_cast<const float4*>(qsrc + (ks + HALF_KS) * 16 + 4 * u);
                        if (owns_new) {
                            kl[j][u] = *reinterpret_cast<const float4*>(ksrc + ks * 16 + 4 * u);
                            kh[j][u] = *reinterpret_cast<const float4*>(ksrc + (ks + HALF_KS) * 16 + 4 * u);
                        }
                    }
                }
            }
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int j = 0; j < PASS; j++) {
                const int ks = k0 + j;
                if (ks < HALF_KS) {
                    turn(ql[j], qh[j], c[j], sn[j], qf[ks], qf[ks + HALF_KS]);
                    if (owns_new) turn(kl[j], kh[j], c[j], sn[j], kn[ks], kn[ks + HALF_KS]);
                }
            }
        }
        if (!col_ok) {
#pragma unroll
            for (int ks = 0; ks < KS; ks++) qf[ks].u = make_uint4(0, 0, 0, 0);
        }
        if (owns_new) {
            const int P_ = 1 << psh;
            if (col == 0) {                                  // every lane of a half computed the same key: one lane of each stores
                uint16_t* dst = const_cast<uint16_t*>(kc) + (size_t)slot * kvw + g * D + half * 8;
#pragma unroll
                for (int ks = 0; ks < KS; ks++) {
                    *reinterpret_cast<uint4*>(dst + ks * 16) = kn[ks].u;
                    *reinterpret_cast<uint4*>(&new_s[ks * 16 + half * 8]) = kn[ks].u;
                }
            }
            if (half == 0) {                                 // the value: dimension 32 db + col, transposed inside its page
                uint16_t* vdst = const_cast<uint16_t*>(vc) + (size_t)(slot >> psh) * P_ * kvw + (slot & (P_ - 1));
#pragma unroll
                for (int db = 0; db < NDB; db++) {
                    const uint16_t v = bf16_bits(vraw[db]);
                    vdst[(size_t)(g * D + 32 * db + col) * P_] = v;
                    new_s[D + 32 * db + col] = v;
                }
            }
        }
    };
    floatx16 o[VDB];
#pragma unroll
    for (int db = 0; db < VDB; db++)
#pragma unroll
        for (int r = 0; r < 16; r++) o[db][r] = 0.f;
    float m = NEG_BIG, l = 0.f;
    extern __shared__ float rel_s[];
    if constexpr (REL) {
        if (ex.rel_lds) stage_rel(ex, rel_s, g * cpt, cpt, lane, WAVE);       // (the walk's first barrier stands before its first use)
    }

    // Page ids come from LDS, never from the block table inside the loop: a block-table load
    // whose result feeds an address would have to be waited for, and since loads return in order
    // that wait would drain every key and value load issued before it. The ids of a window of
    // PG_MAX pages are fetched at once (pw0 = first page of the window), outside the steady loop.
    __shared__ int pg_s[PG_MAX];
    int pw0 = 0;
    auto page_of = [&](int key) { return pg_s[(key >> psh) - pw0]; };

    auto load_k = [&](int key0, Frag (&kf)[KS]) {
        int key = key0 + col;                              // this lane's row of the key block
        key = key < hi ? key : hi;                         // rows past the end repeat the last key; they are masked
        const int page = page_of(key);
        const unsigned off = __umul24((unsigned)((page << psh) + (key & (P - 1))), (unsigned)kvw) + (unsigned)(g * D + half * 8);
#pragma unroll
        for (int ks = 0; ks < KS; ks++) kf[ks].u = *reinterpret_cast<const uint4*>(kc + (off + (unsigned)(ks * 16)));
    };

    // values of a block: for product step kk the lane needs keys key0 + 16 kk + 4 half + {0..3}
    // and the same + 8, for dimension 32 db + col
    auto load_v = [&](int key0, Frag (&vf)[VDB][2]) {
#pragma unroll
        for (int kk = 0; kk < 2; kk++) {
#pragma unroll
            for (int run = 0; run < 2; run++) {
                int ka = key0 + 16 * kk + 8 * run + 4 * half;
                ka = ka < (hi & ~3) ? ka : (hi & ~3);       // runs past the end are masked; read a valid one
                const int page = page_of(ka);
                // element offsets fit 32 bits (checked on the host), so one base serves every load
                const unsigned off = __umul24((unsigned)(page << psh), (unsigned)vvw) + (unsigned)(((gv * DV + col) << psh) + (ka & (P - 1)));
#pragma unroll
                for (int db = 0; db < VDB; db++)
                    vf[db][kk].h[run] = *reinterpret_cast<const uint2*>(vc + (off + (unsigned)((db * 32) << psh)));
            }
        }
    };

    // One block of 32 keys in two halves, so that the registers of its keys can be refilled as
    // soon as the scores are formed: scores + online softmax, then weighted values.
    Frag pf[2];
    auto scores = [&](int key0, Frag (&kf)[KS]) {
        if (FUSED && owns_new && key0 <= hi && hi < key0 + KB) {       // the block of the token's own key (uniform)
            if (key0 + col == hi) {
#pragma unroll
                for (int ks = 0; ks < KS; ks++) kf[ks].u = *reinterpret_cast<const uint4*>(&new_s[ks * 16 + half * 8]);
            }
        }
        floatx16 st;
#pragma unroll
        for (int r = 0; r < 16; r++) st[r] = 0.f;
#pragma unroll
        for (int ks = 0; ks < KS; ks++)
            st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[ks].v, qf[ks].v, st, 0, 0, 0);
        // element r of the lane: key key0 + 8 (r / 4) + 4 half + r % 4, this lane's column.
        // Most blocks lie wholly inside what every column of the wave may see (unused columns
        // aside, whose results are dropped): no key of them needs the visibility test, and the
        // scale (positive) moves into the exponent's fma.
        if constexpr (SIG) {
            // no softmax: a visible key weighs sigmoid(score + the head's number), the score capped by c tanh(score / c) =
            // c (1 - 2 / (1 + exp(2 score / c))) first if a cap is given; no maximum, no sum, nothing to rescale
            const float sc = scale_log2e * 0.6931471805599453f, cap2 = softcap > 0.f ? 2.885390081777927f / softcap : 0.f;
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int kr = key0 + 8 * (r / 4) + 4 * half + (r % 4);
                float sv = st[r] * sc;
                if (softcap > 0.f) sv = softcap * (1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + fast_exp2(sv * cap2)));
                st[r] = (kr >= vlo && kr <= vhi) ? __builtin_amdgcn_rcpf(1.0f + fast_exp2(-1.4426950408889634f * (sv + hb))) : 0.f;
            }
        } else {
            const bool inside = (MODE == ATT_PLAIN || KEEP) &&
                                __all(!col_ok || ((key0 >= vlo || (KEEP && key0 + KB <= keep)) && key0 + KB - 1 <= vhi)) != 0;
            float mx = NEG_BIG, mn, corr, psum = 0.f;
            if (inside) {
#pragma unroll
                for (int r = 0; r < 16; r++) mx = fmaxf(mx, st[r]);
                mx = pair_max(mx) * scale_log2e;
                mn = mx > m + MAX_SLACK ? mx : m;
                corr = fast_exp2(m - mn);
#pragma unroll
                for (int r = 0; r < 16; r++) {
                    st[r] = fast_exp2(fmaf(st[r], scale_log2e, -mn));
                    psum += st[r];
                }
            } else {
                const float cap2 = MODE == ATT_SHAPED && softcap > 0.f ? 2.0f * LOG2E / softcap : 0.f;
                float rel_b[16];
                if constexpr (REL) rel_terms(ex, rel_s, my_head - g * cpt, my_head, pos, key0, half, rel_b);
#pragma unroll
                for (int r = 0; r < 16; r++) {
                    const int kr = key0 + 8 * (r / 4) + 4 * half + (r % 4);
                    const bool vis = (kr >= vlo || (KEEP && kr < keep)) && kr <= vhi;
                    const float sv = MODE == ATT_SHAPED ? shaped_score(st[r], scale_log2e * 0.6931471805599453f, softcap, cap2, dist, r1, r2, (float)(pos - kr))
                                     : REL ? fmaf(st[r], scale_log2e, rel_b[r]) : st[r] * scale_log2e;
                    st[r] = vis ? sv : NEG_BIG;
                    mx = fmaxf(mx, st[r]);
                }
                mx = pair_max(mx);
                mn = mx > m + MAX_SLACK ? mx : m;
                corr = fast_exp2(m - mn);
#pragma unroll
                for (int r = 0; r < 16; r++) {
                    const float p = st[r] > 0.5f * NEG_BIG ? fast_exp2(st[r] - mn) : 0.f;
                    st[r] = p;
                    psum += p;
                }
            }
            psum = pair_sum(psum);
            l = l * corr + psum;
            m = mn;
            // the running maxima settle after a few blocks; the accumulators are rescaled only when
            // some column's maximum moved (decided by the whole wave together)
            if (__any(corr != 1.0f)) {
#pragma unroll
                for (int db = 0; db < VDB; db++)
#pragma unroll
                    for (int r = 0; r < 16; r++) o[db][r] *= corr;
            }
        }
#pragma unroll
        for (int kk = 0; kk < 2; kk++) {
            uint32_t w[4];
#pragma unroll
            for (int e = 0; e < 4; e++)
                w[e] = prob_pair(st[8 * kk + 2 * e], st[8 * kk + 2 * e + 1]);
            pf[kk].u = make_uint4(w[0], w[1], w[2], w[3]);
        }
    };
    // Keys of a block that lie outside [k_begin, k_end] (before the first key any column sees, past the
    // last one) have probability zero in every column, but what the cache holds there is not this
    // request's: rows of a page it has not written yet, or of a page the window gave back, with
    // whatever their last owner left, Inf and NaN included, and 0 x Inf is NaN. Their values are
    // replaced by zeros; only the first and the last block of a walk have such keys.
    auto values = [&](int key0, Frag (&vf)[VDB][2]) {
        if constexpr (FUSED) if (owns_new && key0 <= hi && hi < key0 + KB) {       // the token's own value, in the run of four keys that holds it
#pragma unroll
            for (int kk = 0; kk < 2; kk++)
#pragma unroll
                for (int run = 0; run < 2; run++) {
                    const int ka = key0 + 16 * kk + 8 * run + 4 * half;
                    if (ka <= hi && hi < ka + 4) {
                        const int e = hi - ka;
#pragma unroll
                        for (int db = 0; db < NDB; db++) {
                            const uint32_t v = new_s[D + 32 * db + col];
                            const uint32_t x = vf[db][kk].h[run].x, y = vf[db][kk].h[run].y;
                            vf[db][kk].h[run].x = e == 0 ? (x & 0xffff0000u) | v : e == 1 ? (x & 0x0000ffffu) | (v << 16) : x;
                            vf[db][kk].h[run].y = e == 2 ? (y & 0xffff0000u) | v : e == 3 ? (y & 0x0000ffffu) | (v << 16) : y;
                        }
                    }
                }
        }
        if (key0 < k_begin || key0 + KB - 1 > k_end) {         // uniform over the wave
#pragma unroll
            for (int kk = 0; kk < 2; kk++)
#pragma unroll
                for (int run = 0; run < 2; run++) {
                    const int kb = key0 + 16 * kk + 8 * run + 4 * half;
                    uint32_t mk[2];
#pragma unroll
                    for (int e = 0; e < 2; e++) {
                        const bool lo_ok = (kb + 2 * e >= k_begin || (KEEP && kb + 2 * e < keep)) && kb + 2 * e <= k_end;
                        const bool hi_ok = (kb + 2 * e + 1 >= k_begin || (KEEP && kb + 2 * e + 1 < keep)) && kb + 2 * e + 1 <= k_end;
                        mk[e] = (lo_ok ? 0x0000ffffu : 0u) | (hi_ok ? 0xffff0000u : 0u);
                    }
#pragma unroll
                    for (int db = 0; db < VDB; db++) {
                        vf[db][kk].h[run].x &= mk[0];
                        vf[db][kk].h[run].y &= mk[1];
                    }
                }
        }
#pragma unroll
        for (int kk = 0; kk < 2; kk++)
#pragma unroll
            for (int db = 0; db < VDB; db++)
                o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[db][kk].v, pf[kk].v, o[db], 0, 0, 0);
    };

    // Two register sets in rotation. The keys of block b + 2 are requested as soon as the scores
    // of block b are formed, its values as soon as block b's values are used, so between one and
    // two blocks (16 to 32 KB a wave at head_dim 128) are always on their way. Inside a window
    // every load is issued unconditionally (past the window's end its last block is fetched again
    // and not used) and there is no branch around a load: the compiler then knows how many loads
    // are outstanding at each use and waits for exactly those instead of draining all of them.
    for (int seg = KEEP ? 0 : 1; seg < 2; seg++) {                                // the kept keys, then the window's
    if (SPLIT && kept_chunk && (seg == 0) != (chunk == 0)) continue;                    // (uniform)
    const int first = seg == 0 ? 0 : (k_begin / KB) * KB;
    const int seg_end = seg == 0 && n_kept - 1 < k_end ? n_kept - 1 : k_end;
    const int nb = first <= seg_end ? (seg_end - first) / KB + 1 : 0;
    const int k_top = first + nb * KB - 1 < hi ? first + nb * KB - 1 : hi;       // last key any load touches
    // key blocks a window of pages covers; a walk starts at a multiple of 32 keys, which with pages of more
    // than 32 tokens may lie inside a page: the window's keys then touch one page more than they fill
    const int win_blocks = ((P > KB ? PG_MAX - 1 : PG_MAX) << psh) / KB;
    for (int wb = 0; wb < nb; wb += win_blocks) {
        const int we = wb + win_blocks < nb ? wb + win_blocks : nb;               // blocks [wb, we)
        __syncthreads();                                                          // the old window is no longer read
        pw0 = (first + wb * KB) >> psh;
        {
            const int top = first + we * KB - 1 < k_top ? first + we * KB - 1 : k_top;
            const int n_pg = (top >> psh) - pw0 + 1;
            for (int i = lane; i < n_pg; i += WAVE) pg_s[i] = bt[pw0 + i];
        }
        __syncthreads();
        const int last = first + (we - 1) * KB;
        auto at = [&](int b) { const int k = first + b * KB; return k < last ? k : last; };
        Frag k0f[KS], k1f[KS], v0f[VDB][2], v1f[VDB][2];
        load_k(at(wb), k0f);
        load_v(at(wb), v0f);
        load_k(at(wb + 1), k1f);
        load_v(at(wb + 1), v1f);
        if (FUSED && wb == 0) fused_prologue();
        for (int b = wb; b < we; b += 2) {
            scores(first + b * KB, k0f);
            load_k(at(b + 2), k0f);
            values(first + b * KB, v0f);
            load_v(at(b + 2), v0f);
            if (b + 1 >= we) break;
            scores(first + (b + 1) * KB, k1f);
            load_k(at(b + 3), k1f);
            values(first + (b + 1) * KB, v1f);
            load_v(at(b + 3), v1f);
        }
    }
    }

    if (!col_ok) return;
    if (SIG) {
        m = 0.f;
        l = (!SPLIT || chunk == 0) ? 1.f : 0.f;
    }
    // element r of o[db]: dimension 32 db + 8 (r / 4) + 4 half + r % 4 of this lane's column
    if (SPLIT) {
        float* dst = partial + ((size_t)(my_tok * H + my_head) * n_chunks + chunk) * (DV + 2);
        if (half == 0) {
            dst[0] = m;
            dst[1] = l;
        }
#pragma unroll
        for (int db = 0; db < VDB; db++)
#pragma unroll
            for (int rg = 0; rg < 4; rg++) {
                float4 v = make_float4(o[db][4 * rg], o[db][4 * rg + 1], o[db][4 * rg + 2], o[db][4 * rg + 3]);
                *reinterpret_cast<float4*>(dst + 2 + 32 * db + 8 * rg + 4 * half) = v;
            }
    } else {
        const float inv = head_factor(ex, my_tok, my_head) / (sink ? l + exp2f((sink_w ? sink_w[my_head] * LOG2E : 0.f) - m) : l);      // the term that has no value
        if (ex.out_f32) {
            float* dst32 = reinterpret_cast<float*>(out) + (size_t)my_tok * ldo + my_head * DV;
#pragma unroll
            for (int db = 0; db < VDB; db++)
#pragma unroll
                for (int rg = 0; rg < 4; rg++)
                    *reinterpret_cast<float4*>(dst32 + 32 * db + 8 * rg + 4 * half) =
                        make_float4(o[db][4 * rg] * inv, o[db][4 * rg + 1] * inv, o[db][4 * rg + 2] * inv, o[db][4 * rg + 3] * inv);
            return;
        }
        uint16_t* dst = out + (size_t)my_tok * ldo + my_head * DV;
#pragma unroll
        for (int db = 0; db < VDB; db++)
#pragma unroll
            for (int rg = 0; rg < 4; rg++) {
                uint2 v;
                v.x = (uint32_t)bf16_bits(o[db][4 * rg] * inv) | ((uint32_t)bf16_bits(o[db][4 * rg + 1] * inv) << 16);
                v.y = (uint32_t)bf16_bits(o[db][4 * rg + 2] * inv) |
                      ((uint32_t)bf16_bits(o[db][4 * rg + 3] * inv) << 16);
                *reinterpret_cast<uint2*>(dst + 32 * db + 8 * rg + 4 * half) = v;
            }
    }
}

// ---- prompt portions: four waves share the keys and values of a block through LDS ---------------
// A block of four waves owns 4 x (tokens per wave) consecutive tokens of one request and one
// key/value head; wave w takes its own 32 columns as above. Every block of 32 keys is fetched
// once by the 256 threads (keys as rows of K, values as rows of V^T), stored in LDS with padded
// rows (272 and 72 bytes: the fragment reads of a wave are conflict-free) and read by all four
// waves, so L2-to-CU traffic drops fourfold against the kernel above and several waves per SIMD
// overlap their matrix products and softmax. Two LDS stages, one barrier per key block. Tiles
// are numbered from the end of each request backwards, so the longest ones start first.
#define MERGE_MAX_CHUNKS 512     // chunks of keys that the merge takes
#define PVS 36       // LDS row of a value dimension: 32 keys + 4 pad (elements)

template <int NDB, bool SMALL_PAGES, int MODE = ATT_PLAIN, int VDB = NDB>
__global__ __launch_bounds__(4 * WAVE) __attribute__((amdgpu_waves_per_eu(2))) void attn_prefill_kernel(
    const uint16_t* __restrict__ q, int ldq, const uint16_t* __restrict__ kc, const uint16_t* __restrict__ vc, int kvw,
    const int* __restrict__ block_table, int max_blocks, const int* __restrict__ token_slot,
    const int* __restrict__ positions, const int* __restrict__ q_start, int n_seqs, uint16_t* __restrict__ out,
    int ldo, int psh, int window, int mask_chunk, float scale_log2e, int tpt, int cpt, int n_tiles, int pair_from,
    float* __restrict__ partial, int H, int chunk_keys, int n_chunks, int sink, int v_rot, float softcap,
    const float* __restrict__ head_bias, const float* __restrict__ sink_w,
    const float* __restrict__ dist_scale, const float* __restrict__ dist_rate, AttnExtra ex) {
    constexpr int D = NDB * 32, KS = D / 16, KROW = D + 8, DV = VDB * 32;
    constexpr bool SIG = MODE == ATT_SIGMOID, REL = MODE == ATT_REL, KEEP = MODE == ATT_KEEP;
    const int keep = KEEP ? ex.keep : 0;
    const int P = 1 << psh;                                // tokens per page, a power of two
    __shared__ __attribute__((aligned(16))) uint16_t k_s[2][KB * KROW];
    __shared__ __attribute__((aligned(16))) uint16_t v_s[2][DV * PVS];
    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wave = tid / WAVE;
    const int col = lane & 31, half = lane >> 5;
    int g = blockIdx.x, tile = blockIdx.y;
    const int tile_tokens = 4 * tpt;

    // Tiles late in a prompt see many keys, early ones few. Blocks are numbered with the key/value
    // head fastest and the tiles from the longest down, so that the long tiles of all heads start
    // first and the short ones fill in beside them (with the head slowest, a CU got two blocks of
    // the same length, and the CUs with the longest tiles set the kernel's time).
    //
    // When all blocks are resident at once, two to a CU, the second block of a CU (id pair_from + j,
    // beside block j) takes the tiles from the shortest up, so that every CU has the same sum of keys.
    if (pair_from > 0) {
        const int id = blockIdx.y * gridDim.x + blockIdx.x;
        if (id >= pair_from) {
            const int j = id - pair_from;
            if (j >= n_tiles * (int)gridDim.x - pair_from) return;
            tile = n_tiles - 1 - j / (int)gridDim.x;
            g = j % (int)gridDim.x;
        }
    }
    // the group whose values the weights are applied to (see attn_mfma_kernel)
    const int gv = VDB != NDB || KEEP || REL ? g / ex.v_share : g + v_rot < (int)gridDim.x ? g + v_rot : g + v_rot - (int)gridDim.x;
    const int vvw = VDB != NDB || KEEP || REL ? ex.vw : kvw;
    int t0 = -1, t_end = 0;
    for (int s = 0; s < n_seqs; s++) {
        const int a = q_start[s], b = q_start[s + 1];
        const int nt = (b - a + tile_tokens - 1) / tile_tokens;
        if (tile < nt) {
            const int rt = nt - 1 - tile;                   // last tile of the request first
            t0 = a + rt * tile_tokens;
            t_end = t0 + tile_tokens < b ? t0 + tile_tokens : b;
            break;
        }
        tile -= nt;
    }
    if (t0 < 0) return;                                    // uniform over the block: no barrier is skipped

    // this wave's tokens and columns
    const int w0 = t0 + wave * tpt;
    const int w_end = w0 + tpt < t_end ? w0 + tpt : t_end;
    const int n_cols = w_end > w0 ? (w_end - w0) * cpt : 0;
    const bool col_ok = col < n_cols;
    const int my_tok = col_ok ? w0 + col / cpt : t0;
    const int my_head = g * cpt + (col_ok ? col % cpt : 0);
    const float hb = (SIG && head_bias) ? head_bias[my_head] : 0.f;
    const bool dist = MODE == ATT_SHAPED && dist_scale != nullptr;
    const float r1 = dist ? dist_scale[my_head] : 0.f, r2 = dist ? dist_rate[my_head] : 0.f;
    const int pos = positions[my_tok];
    const int pos_first = positions[t0];
    int hi = positions[t_end - 1];
    int k_begin = first_visible(pos_first, window, mask_chunk);
    // With n_chunks > 1 the block takes the keys of chunk blockIdx.z only (chunk_keys is a multiple
    // of the key block) and leaves maximum, sum and unscaled output for attn_merge_kernel; a chunk
    // that holds none of the tile's keys leaves an empty record.
    const int n_kept = KEEP ? kept_before(keep, k_begin / KB * KB) : 0, kept_chunk = keep > 0 ? 1 : 0;         // (see attn_mfma_kernel)
    if (kept_chunk && n_chunks > 1 && blockIdx.z == 0) {
        hi = n_kept - 1 < hi ? n_kept - 1 : hi;
    } else if (n_chunks > 1) {
        // (under a window or a mask by chunks, counted from the first key block that the tile sees: see attn_mfma_kernel)
        const int c_lo = (attn_bounded(window, mask_chunk) ? k_begin / KB * KB : 0) + ((int)blockIdx.z - kept_chunk) * chunk_keys, c_hi = c_lo + chunk_keys - 1;
        k_begin = k_begin > c_lo ? k_begin : c_lo;
        hi = hi < c_hi ? hi : c_hi;
    }
    const int vlo = first_visible(pos, window, mask_chunk) > k_begin ? first_visible(pos, window, mask_chunk) : k_begin;
    const int vhi = col_ok ? (pos < hi ? pos : hi) : -1;
    const int* bt = block_table + (size_t)token_slot[t0] * max_blocks;

    // query fragments stay in registers for the whole tile
    Frag qf[KS];
    {
        const uint16_t* qp = q + (size_t)my_tok * ldq + my_head * D + half * 8;
#pragma unroll
        for (int ks = 0; ks < KS; ks++)
            qf[ks].u = col_ok ? *reinterpret_cast<const uint4*>(qp + ks * 16) : make_uint4(0, 0, 0, 0);
    }
    floatx16 o[VDB];
#pragma unroll
    for (int db = 0; db < VDB; db++)
#pragma unroll
        for (int r = 0; r < 16; r++) o[db][r] = 0.f;
    float m = NEG_BIG, l = 0.f;
    extern __shared__ float rel_s[];
    if constexpr (REL) {
        if (ex.rel_lds) stage_rel(ex, rel_s, g * cpt, cpt, tid, 4 * WAVE);
    }

    // page ids in LDS, a window of PG_MAX pages at a time (see the kernel above)
    __shared__ int pg_s[PG_MAX];
    int pw0 = 0;
    auto page_of = [&](int key) { return pg_s[(key >> psh) - pw0]; };

    // global -> registers -> LDS. Keys: 32 rows of D elements = 4 D chunks of 16 bytes.
    // Values: D rows of 32 keys = 4 D chunks of 8 keys. Each thread takes up to NCH of both.
    // With a whole number of chunks per thread (head_dim 64 and 128) no load or store stands under a
    // condition: only then does the compiler count the loads in flight and wait for the older set alone.
    constexpr int TOT = 4 * D, NCH = (TOT + 255) / 256, TOTV = 4 * DV, NCV = (TOTV + 255) / 256;
    constexpr bool EVEN = TOT % 256 == 0, EVENV = TOTV % 256 == 0;
    u32x4 rk0[NCH], rk1[NCH];
    uint2 rv0[NCV][2], rv1[NCV][2];
    // Pages of up to 32 tokens divide a block of keys, whose first key is a multiple of 32: a
    // thread's row then lies at the same place of the same page of every block, and its addresses
    // are a page id times the page's size plus a constant. No key is clamped on this path: the
    // window of page ids repeats the last valid page for pages past the end (see below), so what is
    // read there is memory of that page, and it is masked like any key past a column's position.
    constexpr bool small_pages = SMALL_PAGES;                  // the launcher's choice: pages of up to 32 tokens
    const unsigned page_elems = (unsigned)kvw << psh, v_page_elems = (unsigned)vvw << psh;
    int k_pg[NCH], v_pg[NCV];
    unsigned k_at[NCH], v_at[NCV];
#pragma unroll
    for (int i = 0; i < NCH; i++) {
        const int c = tid + i * 256, row = c / (D / 8);
        k_pg[i] = row >> psh;
        k_at[i] = (unsigned)((row & (P - 1)) * kvw + g * D + (c % (D / 8)) * 8);
    }
#pragma unroll
    for (int i = 0; i < NCV; i++) {
        const int c = tid + i * 256, k8 = 8 * (c % 4);
        v_pg[i] = k8 >> psh;
        v_at[i] = (unsigned)(((gv * DV + c / 4) << psh) + (k8 & (P - 1)));
    }
    auto gload = [&](int key0, u32x4 (&rk)[NCH], uint2 (&rv)[NCV][2]) {
        if constexpr (small_pages) {
            const int pb = (key0 >> psh) - pw0;
#pragma unroll
            for (int i = 0; i < (NCH > NCV ? NCH : NCV); i++) {
                if (i < NCH) {
                    if (EVEN || tid + i * 256 < TOT)
                        rk[i < NCH ? i : 0] = *reinterpret_cast<const u32x4*>(kc + (__umul24((unsigned)pg_s[pb + k_pg[i < NCH ? i : 0]], page_elems) + k_at[i < NCH ? i : 0]));
                }
                if (i < NCV) {
                    if (EVENV || tid + i * 256 < TOTV) {
                        const int j = i < NCV ? i : 0;
                        const uint4 v = *reinterpret_cast<const uint4*>(vc + (__umul24((unsigned)pg_s[pb + v_pg[j]], v_page_elems) + v_at[j]));
                        rv[j][0] = make_uint2(v.x, v.y);
                        rv[j][1] = make_uint2(v.z, v.w);
                    }
                }
            }
            return;
        }
#pragma unroll
        for (int i = 0; i < NCH; i++) {
            const int c = tid + i * 256;
            if (!EVEN && c >= TOT) break;
            {   // key chunk: row c / (D / 8), 16-byte piece c % (D / 8)
                int key = key0 + c / (D / 8);
                key = key < hi ? key : hi;
                const int page = page_of(key);
                const unsigned off = __umul24((unsigned)((page << psh) + (key & (P - 1))), (unsigned)kvw) + (unsigned)(g * D + (c % (D / 8)) * 8);
                rk[i] = *reinterpret_cast<const u32x4*>(kc + off);
            }
        }
#pragma unroll
        for (int i = 0; i < NCV; i++) {
            const int c = tid + i * 256;
            if (!EVENV && c >= TOTV) break;
            {   // value chunk: dimension c / 4, keys key0 + 8 (c % 4) .. + 7
                int ka = key0 + 8 * (c % 4);
                ka = ka < (hi & ~7) ? ka : (hi & ~7);
                const int page = page_of(ka);
                const unsigned off = __umul24((unsigned)(page << psh), (unsigned)vvw) + (unsigned)(((gv * DV + c / 4) << psh) + (ka & (P - 1)));
                const uint4 v = *reinterpret_cast<const uint4*>(vc + off);
                rv[i][0] = make_uint2(v.x, v.y);
                rv[i][1] = make_uint2(v.z, v.w);
            }
        }
    };
    // Values of keys outside [k_begin, hi] are stored as zeros (see the kernel above: their probabilities
    // are zero, what the cache holds there may be anything); only a walk's first and last block have such.
    auto sstore = [&](int stage, int key0, const u32x4 (&rk)[NCH], const uint2 (&rv)[NCV][2]) {
        const bool edge = key0 < k_begin || key0 + KB - 1 > hi;           // uniform over the block
#pragma unroll
        for (int i = 0; i < NCH; i++) {
            const int c = tid + i * 256;
            if (!EVEN && c >= TOT) break;
            *reinterpret_cast<u32x4*>(&k_s[stage][(c / (D / 8)) * KROW + (c % (D / 8)) * 8]) = rk[i];
        }
#pragma unroll
        for (int i = 0; i < NCV; i++) {
            const int c = tid + i * 256;
            if (!EVENV && c >= TOTV) break;
            uint2* dst = reinterpret_cast<uint2*>(&v_s[stage][(c / 4) * PVS + 8 * (c % 4)]);
            uint2 v0 = rv[i][0], v1 = rv[i][1];
            if (edge) {
                const int kb = key0 + 8 * (c % 4);
                auto kept = [&](int k) { return (k >= k_begin || (KEEP && k < keep)) && k <= hi; };
                v0.x &= (kept(kb) ? 0x0000ffffu : 0u) | (kept(kb + 1) ? 0xffff0000u : 0u);
                v0.y &= (kept(kb + 2) ? 0x0000ffffu : 0u) | (kept(kb + 3) ? 0xffff0000u : 0u);
                v1.x &= (kept(kb + 4) ? 0x0000ffffu : 0u) | (kept(kb + 5) ? 0xffff0000u : 0u);
                v1.y &= (kept(kb + 6) ? 0x0000ffffu : 0u) | (kept(kb + 7) ? 0xffff0000u : 0u);
            }
            dst[0] = v0;
            dst[1] = v1;
        }
    };

    for (int seg = KEEP ? 0 : 1; seg < 2; seg++) {                                // the kept keys, then the window's
    if (kept_chunk && n_chunks > 1 && (seg == 0) != (blockIdx.z == 0)) continue;        // (uniform)
    const int first = seg == 0 ? 0 : (k_begin / KB) * KB;
    const int seg_hi = seg == 0 && n_kept - 1 < hi ? n_kept - 1 : hi;
    const int nb = seg_hi >= (seg == 0 ? 0 : k_begin) ? (seg_hi - first) / KB + 1 : 0;
    const int win_blocks = ((P > KB ? PG_MAX - 1 : PG_MAX) << psh) / KB;     // see the kernel above
    for (int wb = 0; wb < nb; wb += win_blocks) {
        const int we = wb + win_blocks < nb ? wb + win_blocks : nb;               // blocks [wb, we)
        __syncthreads();                                                          // old window and stages are no longer read
        pw0 = (first + wb * KB) >> psh;
        {
            const int top = first + we * KB - 1 < hi ? first + we * KB - 1 : hi;
            const int n_pg = (top >> psh) - pw0 + 1;
            // pages past the last one that holds keys (the window's last block is loaded whole): its id again
            const int n_all = small_pages ? ((first + we * KB - 1) >> psh) - pw0 + 1 : n_pg;
            for (int i = tid; i < n_all; i += 4 * WAVE) pg_s[i] = bt[pw0 + (i < n_pg ? i : n_pg - 1)];
        }
        __syncthreads();
        const int last = first + (we - 1) * KB;
        auto at = [&](int b) { const int k = first + b * KB; return k < last ? k : last; };
        gload(at(wb), rk0, rv0);
        sstore(wb & 1, at(wb), rk0, rv0);
        gload(at(wb + 1), rk0, rv0);                          // unconditional: past the end the last block is fetched again
        gload(at(wb + 2), rk1, rv1);
        __syncthreads();
        // Two register sets in rotation: the block after the next one is on its way while the next one
        // goes into LDS, so a load has two blocks' worth of products and softmax to arrive.
        auto one_block = [&](int b) {
            const int key0 = first + b * KB, stage = b & 1;
            // A wave whose columns all end before this block skips the math. The test is made by all
            // lanes together: the matrix products need every lane, also those of unused columns.
            const bool wave_sees = __any(key0 <= vhi) != 0;
            if (wave_sees) {
                const uint16_t* ks_ = &k_s[stage][col * KROW + half * 8];
                floatx16 st;
#pragma unroll
                for (int r = 0; r < 16; r++) st[r] = 0.f;
                // All fragment reads of the block are asked for before the first product: left to itself
                // the compiler reads one fragment, waits for it and multiplies, sixteen LDS round trips
                // a block. The values' first half arrives while the softmax is computed.
                Frag kf[KS], vf[2][VDB];
#pragma unroll
                for (int ks = 0; ks < KS; ks++) kf[ks].u = *reinterpret_cast<const uint4*>(ks_ + ks * 16);
                auto vread = [&](int kk) {
#pragma unroll
                    for (int db = 0; db < VDB; db++) {
                        const uint16_t* vs_ = &v_s[stage][(32 * db + col) * PVS + 16 * kk + 4 * half];
                        vf[kk][db].h[0] = *reinterpret_cast<const uint2*>(vs_);
                        vf[kk][db].h[1] = *reinterpret_cast<const uint2*>(vs_ + 8);
                    }
                };
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int ks = 0; ks < KS; ks++)
                    st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[ks].v, qf[ks].v, st, 0, 0, 0);
                vread(0);
                __builtin_amdgcn_sched_barrier(0);
                // Most blocks lie wholly inside what every column of the wave may see (unused columns
                // aside, whose results are dropped): no key of them needs the visibility test.
                if constexpr (SIG) {
                    // no softmax: a visible key weighs sigmoid(score + the head's number), the score capped by c tanh(score / c) =
                    // c (1 - 2 / (1 + exp(2 score / c))) first if a cap is given; no maximum, no sum, nothing to rescale
                    const float sc = scale_log2e * 0.6931471805599453f, cap2 = softcap > 0.f ? 2.885390081777927f / softcap : 0.f;
#pragma unroll
                    for (int r = 0; r < 16; r++) {
                        const int kr = key0 + 8 * (r / 4) + 4 * half + (r % 4);
                        float sv = st[r] * sc;
                        if (softcap > 0.f) sv = softcap * (1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + fast_exp2(sv * cap2)));
                        st[r] = (kr >= vlo && kr <= vhi) ? __builtin_amdgcn_rcpf(1.0f + fast_exp2(-1.4426950408889634f * (sv + hb))) : 0.f;
                    }
                } else {
                    const bool inside = (MODE == ATT_PLAIN || KEEP) &&
                                        __all(!col_ok || ((key0 >= vlo || (KEEP && key0 + KB <= keep)) && key0 + KB - 1 <= vhi)) != 0;
                    float mx = NEG_BIG, mn, corr, psum = 0.f;
                    if (inside) {                                   // the scale (positive) moves into the exponent's fma
#pragma unroll
                        for (int r = 0; r < 16; r++) mx = fmaxf(mx, st[r]);
                        mx = pair_max(mx) * scale_log2e;
                        mn = mx > m + MAX_SLACK ? mx : m;
                        corr = fast_exp2(m - mn);
#pragma unroll
                        for (int r = 0; r < 16; r++) {
                            st[r] = fast_exp2(fmaf(st[r], scale_log2e, -mn));
                            psum += st[r];
                        }
                    } else {
                        const float cap2 = MODE == ATT_SHAPED && softcap > 0.f ? 2.0f * LOG2E / softcap : 0.f;
                        float rel_b[16];
                        if constexpr (REL) rel_terms(ex, rel_s, my_head - g * cpt, my_head, pos, key0, half, rel_b);
#pragma unroll
                        for (int r = 0; r < 16; r++) {
                            const int kr = key0 + 8 * (r / 4) + 4 * half + (r % 4);
                            const bool vis = (kr >= vlo || (KEEP && kr < keep)) && kr <= vhi;
                            const float sv = MODE == ATT_SHAPED ? shaped_score(st[r], scale_log2e * 0.6931471805599453f, softcap, cap2, dist, r1, r2, (float)(pos - kr))
                                             : REL ? fmaf(st[r], scale_log2e, rel_b[r]) : st[r] * scale_log2e;
                            st[r] = vis ? sv : NEG_BIG;
                            mx = fmaxf(mx, st[r]);
                        }
                        mx = pair_max(mx);
                        mn = mx > m + MAX_SLACK ? mx : m;
                        corr = fast_exp2(m - mn);
#pragma unroll
                        for (int r = 0; r < 16; r++) {
                            const float p = st[r] > 0.5f * NEG_BIG ? fast_exp2(st[r] - mn) : 0.f;
                            st[r] = p;
                            psum += p;
                        }
                    }
                    psum = pair_sum(psum);
                    l = l * corr + psum;
                    m = mn;
                    if (__any(corr != 1.0f)) {                      // see above: only when a maximum moved
#pragma unroll
                        for (int db = 0; db < VDB; db++)
#pragma unroll
                            for (int r = 0; r < 16; r++) o[db][r] *= corr;
                    }
                }
                Frag pf[2];
#pragma unroll
                for (int kk = 0; kk < 2; kk++) {
                    uint32_t w[4];
#pragma unroll
                    for (int e = 0; e < 4; e++)
                        w[e] = prob_pair(st[8 * kk + 2 * e], st[8 * kk + 2 * e + 1]);
                    pf[kk].u = make_uint4(w[0], w[1], w[2], w[3]);
                }
                vread(1);
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int kk = 0; kk < 2; kk++)
#pragma unroll
                    for (int db = 0; db < VDB; db++)
                        o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[kk][db].v, pf[kk].v, o[db], 0, 0, 0);
            }
        };
        for (int b = wb; b < we; b += 2) {
            one_block(b);
            sstore((b & 1) ^ 1, at(b + 1), rk0, rv0);         // block b + 1
            gload(at(b + 3), rk0, rv0);
            __syncthreads();
            if (b + 1 >= we) break;
            one_block(b + 1);
            sstore(b & 1, at(b + 2), rk1, rv1);               // block b + 2
            gload(at(b + 4), rk1, rv1);
            __syncthreads();
        }
    }
    }
    if (!col_ok) return;
    if (SIG) {
        m = 0.f;
        l = (n_chunks == 1 || blockIdx.z == 0) ? 1.f : 0.f;
    }
    if (n_chunks > 1) {
        float* dst = partial + ((size_t)(my_tok * H + my_head) * n_chunks + blockIdx.z) * (DV + 2);
        if (half == 0) {
            dst[0] = m;
            dst[1] = l;
        }
#pragma unroll
        for (int db = 0; db < VDB; db++)
#pragma unroll
            for (int rg = 0; rg < 4; rg++)
                *reinterpret_cast<float4*>(dst + 2 + 32 * db + 8 * rg + 4 * half) =
                    make_float4(o[db][4 * rg], o[db][4 * rg + 1], o[db][4 * rg + 2], o[db][4 * rg + 3]);
        return;
    }
    const float inv = head_factor(ex, my_tok, my_head) / (sink ? l + exp2f((sink_w ? sink_w[my_head] * LOG2E : 0.f) - m) : l);          // the term that has no value
    if (ex.out_f32) {
        float* dst32 = reinterpret_cast<float*>(out) + (size_t)my_tok * ldo + my_head * DV;
#pragma unroll
        for (int db = 0; db < VDB; db++)
#pragma unroll
            for (int rg = 0; rg < 4; rg++)
                *reinterpret_cast<float4*>(dst32 + 32 * db + 8 * rg + 4 * half) =
                    make_float4(o[db][4 * rg] * inv, o[db][4 * rg + 1] * inv, o[db][4 * rg + 2] * inv, o[db][4 * rg + 3] * inv);
        return;
    }
    uint16_t* dst = out + (size_t)my_tok * ldo + my_head * DV;
#pragma unroll
    for (int db = 0; db < VDB; db++)
#pragma unroll
        for (int rg = 0; rg < 4; rg++) {
            uint2 v;
            v.x = (uint32_t)bf16_bits(o[db][4 * rg] * inv) | ((uint32_t)bf16_bits(o[db][4 * rg + 1] * inv) << 16);
            v.y = (uint32_t)bf16_bits(o[db][4 * rg + 2] * inv) | ((uint32_t)bf16_bits(o[db][4 * rg + 3] * inv) << 16);
            *reinterpret_cast<uint2*>(dst + 32 * db + 8 * rg + 4 * half) = v;
        }
}


// log2 of the page size, or -1 if it is not a power of two (the kernels shift and mask by it).
static inline int page_shift(int page_tokens) {
    int s = 0;
    while ((1 << s) < page_tokens) s++;
    return (1 << s) == page_tokens ? s : -1;
}

// The table of distance terms is staged in LDS up to this many bytes a block.
#define REL_LDS_BYTES (32 << 10)

inline AttnExtra attn_extra(const AttnArgs& a) {
    AttnExtra e = {};
    e.rel = a.rel;
    e.rel_n = a.rel_n;
    e.rel_lds = a.rel && (size_t)(a.n_heads / a.n_kv_heads) * a.rel_n * sizeof(float) <= REL_LDS_BYTES;
    e.keep = a.keep_first;
    e.v_share = a.v_share > 0 ? a.v_share : 1;
    e.vw = a.v_width > 0 ? a.v_width : a.kv_width;
    e.gate = a.gate;
    e.gate_bf16 = a.gate_bf16;
    e.ldg = a.ldg;
    e.out_mul = a.out_mul;
    e.out_f32 = a.out_f32;
    return e;
}
inline size_t attn_rel_lds(const AttnArgs& a) {
    return a.rel && attn_extra(a).rel_lds ? (size_t)(a.n_heads / a.n_kv_heads) * a.rel_n * sizeof(float) : 0;
}

template <int NDB, int MODE, int VDB, bool FUSED>
static int launch_step(const AttnArgs& a, const AttnCut& c) {
    dim3 grid(c.tiles, a.n_kv_heads, c.n_chunks);
    const float sl = a.scale * 1.4426950408889634f;
#define ATTN_ARGS(PARTIAL)                                                                                              \
    (const uint16_t*)a.q, a.ldq, (const uint16_t*)a.k_cache, (const uint16_t*)a.v_cache, a.kv_width, a.block_table,      \
        a.max_blocks, a.token_slot, a.positions, a.q_start, a.n_seqs, (uint16_t*)a.out, a.ldo, PARTIAL, a.n_heads,         \
        page_shift(a.page_tokens), a.window, a.mask_chunk, sl, c.tpt, c.cpt, c.chunk_keys, c.n_chunks, a.max_q_len <= c.tpt, a.raw, a.ld_raw,      \
        a.cos_sin, a.slot_map, a.n_kv_heads, a.sink, a.v_rot, a.softcap, a.head_bias, a.sink_w, a.dist_scale, a.dist_rate, attn_extra(a)
    const size_t lds = MODE == ATT_REL ? attn_rel_lds(a) : 0;
    if (c.n_chunks > 1) attn_mfma_kernel<NDB, true, FUSED, MODE, VDB><<<grid, WAVE, lds, a.stream>>>(ATTN_ARGS((float*)a.workspace));
    else attn_mfma_kernel<NDB, false, FUSED, MODE, VDB><<<grid, WAVE, lds, a.stream>>>(ATTN_ARGS(nullptr));
#undef ATTN_ARGS
    HFA_LAUNCH_CHECK("attn_mfma");
    return 0;
}

template <int NDB, int MODE, int VDB>
static int launch_prompt(const AttnArgs& a, const AttnCut& c) {
    dim3 grid(a.n_kv_heads, c.tiles, c.n_chunks);
    const size_t lds = MODE == ATT_REL ? attn_rel_lds(a) : 0;
#define PREFILL_ARGS                                                                                                       \
    (const uint16_t*)a.q, a.ldq, (const uint16_t*)a.k_cache, (const uint16_t*)a.v_cache, a.kv_width, a.block_table,            \
        a.max_blocks, a.token_slot, a.positions, a.q_start, a.n_seqs, (uint16_t*)a.out, a.ldo, page_shift(a.page_tokens),      \
        a.window, a.mask_chunk, a.scale * 1.4426950408889634f, c.tpt, c.cpt, c.prompt_tiles, c.pair_from, (float*)a.workspace, a.n_heads,   \
        c.chunk_keys, c.n_chunks, a.sink, a.v_rot, a.softcap, a.head_bias, a.sink_w, a.dist_scale, a.dist_rate, attn_extra(a)
    if (a.page_tokens <= 32) attn_prefill_kernel<NDB, true, MODE, VDB><<<grid, 4 * WAVE, lds, a.stream>>>(PREFILL_ARGS);
    else attn_prefill_kernel<NDB, false, MODE, VDB><<<grid, 4 * WAVE, lds, a.stream>>>(PREFILL_ARGS);
#undef PREFILL_ARGS
    HFA_LAUNCH_CHECK("attn_prefill");
    return 0;
}
