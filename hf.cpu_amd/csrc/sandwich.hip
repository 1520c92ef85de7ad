// Parts of layers that norm a sublayer's result before it joins the residual stream, and what such designs bring with
// them: an embedding with a scale and a sinusoidal position vector, the norm of a (gated) branch added into the stream,
// an activation made of normed powers, a scale on fp32 rows, the per-head norm of queries and keys with the store of
// keys and values, and the mixing of attention outputs across heads.
//
//   hfa_embed_pos         x[t] = table[token] * scale + sinusoid(position)
//   hfa_rmsnorm_add       out[r] (+)= scale * rmsnorm(branch[r]) * w, the branch as its last products left it; and a rounded copy of out
//   hfa_polynorm          out = a N(z) + b N(z^2) + c N(z^3) + e, N dividing a row by its root mean square
//   hfa_scale_rows        x *= s
//   hfa_head_norm_store   per head: q, k <- rms norm (with a weight of one head's size, shared, or none) before or after a
//                         rotation; q to a matrix, k and v to their cache rows
//   hfa_diff_mix          out[t, h] = c * a / rms(a), a = map 1 of head h minus a factor times map 2
//   hfa_round_rows        an fp32 matrix in bf16
//   hfa_talk_mix          out[t, h] = sigmoid(gate[t, h]) * sum_g talk[h, g] * A[t, g, values of h's group]
#include "api.h"
#include "common.h"

// ---- embedding with a scale and a sinusoidal position vector ------------------------------------------------------
// Entry 2i of the position vector is sin(p f_i), entry 2i + 1 cos(p f_i), f_i = base^(-2i / width) (inv_freq, rounded
// from 64-bit on the host); the angle is one fp32 product.
template <typename T>
__global__ void embed_pos_kernel(const T* __restrict__ table, const int* __restrict__ tokens, const int* __restrict__ positions,
                                 const float* __restrict__ inv_freq, float* __restrict__ x, int width, int vocab, float scale) {
    const int t = blockIdx.x;
    int tok = tokens[t];
    tok = tok < 0 ? 0 : (tok >= vocab ? vocab - 1 : tok);
    const T* row = table + (size_t)tok * width;
    float* dst = x + (size_t)t * width;
    const float pos = positions ? (float)positions[t] : 0.f;
    for (int i = threadIdx.x; i < width; i += blockDim.x) {
        float v = to_f32(row[i]) * scale;
        if (positions) {
            const float ang = pos * inv_freq[i >> 1];
            v += (i & 1) ? cosf(ang) : sinf(ang);
        }
        dst[i] = v;
    }
}

extern "C" int hfa_embed_pos(const void* table, int table_dtype, const int* tokens, const int* positions, const float* inv_freq,
                             float* x, int n_tokens, int width, int vocab, float scale, hipStream_t stream) {
    HFA_REQUIRE(table && tokens && x && n_tokens > 0 && width > 0 && vocab > 0, "embed_pos: bad arguments");
    HFA_REQUIRE(!positions || inv_freq, "embed_pos: positions come with their frequencies");
    HFA_REQUIRE(table_dtype == HFA_F32 || table_dtype == HFA_BF16, "embed_pos: unknown dtype %d", table_dtype);
    if (table_dtype == HFA_F32)
        embed_pos_kernel<float><<<n_tokens, 256, 0, stream>>>((const float*)table, tokens, positions, inv_freq, x, width, vocab, scale);
    else
        embed_pos_kernel<bf16><<<n_tokens, 256, 0, stream>>>((const bf16*)table, tokens, positions, inv_freq, x, width, vocab, scale);
    HFA_LAUNCH_CHECK("embed_pos");
    return 0;
}

// ---- the norm of a branch's result, added into the stream -----------------------------------------------------------
// One block a row, all in fp32. The branch's value at a column is
//   b = [ y | the sum over the planes of a product whose K was split ] * sigmoid(row_gate[r]) + sum_k pairs[r * top + k]
// (an absent part is left out: the result of experts is `pairs`, that of a shared expert `y` with its gate), then times
// sigmoid(gate + gate_bias) element by element; out (+)= scale * b / sqrt(mean(b^2) + eps) * w, or, w null, scale * b. `copy`
// receives the new out in bf16: what a sublayer reads that has no norm in front of it. VW columns a thread and turn.
#define JOIN_PLANES 8
template <int VW>
struct JoinVec { float v[VW]; };
template <int VW>
__device__ __forceinline__ JoinVec<VW> join_load(const float* p) {
    JoinVec<VW> r;
    if constexpr (VW == 4) {
        const float4 u = *reinterpret_cast<const float4*>(p);
        r.v[0] = u.x; r.v[1] = u.y; r.v[2] = u.z; r.v[3] = u.w;
    } else {
        r.v[0] = *p;
    }
    return r;
}
struct JoinArgs {
    const float* y; int ldy;
    const float* partial; int splits; size_t plane;
    const float* row_gate; int ld_row_gate;
    const float* pairs; int top;
    const void* gate; int gate_bf16, ldg;
    const float* gate_bias;
    const float* w;
    float* out; int ldo;
    uint16_t* copy; int ldc;
    int width; float eps, scale; int accumulate;
};

template <int VW>
__global__ __launch_bounds__(1024) void rmsnorm_add_kernel(JoinArgs p) {
    __shared__ float red[17];
    const int r = blockIdx.x;
    const float row_factor = p.row_gate ? 1.0f / (1.0f + expf(-p.row_gate[(size_t)r * p.ld_row_gate])) : 1.f;
    constexpr int KEEP = 8 / VW * (VW == 4 ? 2 : 1);          // 16 columns a thread stay in registers (8 one at a time)
    JoinVec<VW> keep[KEEP];
    auto value = [&](int c) {
        JoinVec<VW> b = {};
        if (p.partial) {
            const float* src = p.partial + (size_t)r * p.width + c;
            for (int s0 = 0; s0 < p.splits; s0 += JOIN_PLANES) {          // batches of loads that do not wait for one another
                JoinVec<VW> q[JOIN_PLANES];
#pragma unroll
                for (int u = 0; u < JOIN_PLANES; u++) q[u] = s0 + u < p.splits ? join_load<VW>(src + (s0 + u) * p.plane) : JoinVec<VW>{};
#pragma unroll
                for (int u = 0; u < JOIN_PLANES; u++)
#pragma unroll
                    for (int e = 0; e < VW; e++) b.v[e] += q[u].v[e];
            }
        } else if (p.y) {
            b = join_load<VW>(p.y + (size_t)r * p.ldy + c);
        }
#pragma unroll
        for (int e = 0; e < VW; e++) b.v[e] *= row_factor;
        if (p.pairs) {
            const float* src = p.pairs + (size_t)r * p.top * p.width + c;
            JoinVec<VW> sum = {};
            for (int k0 = 0; k0 < p.top; k0 += 4) {
                JoinVec<VW> q[4];
#pragma unroll
                for (int u = 0; u < 4; u++) q[u] = k0 + u < p.top ? join_load<VW>(src + (size_t)(k0 + u) * p.width) : JoinVec<VW>{};
#pragma unroll
                for (int u = 0; u < 4; u++)
#pragma unroll
                    for (int e = 0; e < VW; e++) sum.v[e] += q[u].v[e];
            }
#pragma unroll
            for (int e = 0; e < VW; e++) b.v[e] += sum.v[e];
        }
        if (p.gate) {
#pragma unroll
            for (int e = 0; e < VW; e++) {
                const size_t i = (size_t)r * p.ldg + c + e;
                const float z = (p.gate_bf16 ? to_f32(((const bf16*)p.gate)[i]) : ((const float*)p.gate)[i]) + (p.gate_bias ? p.gate_bias[c + e] : 0.f);
                b.v[e] *= 1.0f / (1.0f + expf(-z));
            }
        }
        return b;
    };
    const int stride = blockDim.x * VW, c0 = threadIdx.x * VW;
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
        const int c = c0 + k * stride;
        keep[k] = c < p.width ? value(c) : JoinVec<VW>{};
#pragma unroll
        for (int e = 0; e < VW; e++) ss = fmaf(keep[k].v[e], keep[k].v[e], ss);
    }
    for (int c = c0 + KEEP * stride; c < p.width; c += stride) {
        const JoinVec<VW> b = value(c);
#pragma unroll
        for (int e = 0; e < VW; e++) ss = fmaf(b.v[e], b.v[e], ss);
    }
    const float inv = p.w ? p.scale / sqrtf(block_sum(ss, red) / (float)p.width + p.eps) : p.scale;
    float* dst = p.out + (size_t)r * p.ldo;
    auto finish = [&](int c, const JoinVec<VW>& b) {
        JoinVec<VW> z, o = {};
        if (p.accumulate) o = join_load<VW>(dst + c);
#pragma unroll
        for (int e = 0; e < VW; e++) z.v[e] = o.v[e] + (p.w ? b.v[e] * inv * p.w[c + e] : b.v[e] * inv);
        if constexpr (VW == 4) {
            *reinterpret_cast<float4*>(dst + c) = make_float4(z.v[0], z.v[1], z.v[2], z.v[3]);
            if (p.copy)
                *reinterpret_cast<uint2*>(p.copy + (size_t)r * p.ldc + c) =
                    make_uint2((uint32_t)bf16_bits(z.v[0]) | ((uint32_t)bf16_bits(z.v[1]) << 16),
                               (uint32_t)bf16_bits(z.v[2]) | ((uint32_t)bf16_bits(z.v[3]) << 16));
        } else {
            dst[c] = z.v[0];
            if (p.copy) p.copy[(size_t)r * p.ldc + c] = bf16_bits(z.v[0]);
        }
    };
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
        const int c = c0 + k * stride;
        if (c < p.width) finish(c, keep[k]);
    }
    for (int c = c0 + KEEP * stride; c < p.width; c += stride) finish(c, value(c));
}

extern "C" int hfa_rmsnorm_add(const float* y, int ldy, const float* partial, int splits, const float* row_gate, int ld_row_gate,
                               const float* pairs, int top, const void* gate, int gate_dtype, int ldg, const float* gate_bias,
                               const float* w, float* out, int ldo, void* copy, int ldc, int n_rows, int width, float eps, float scale,
                               int accumulate, hipStream_t stream) {
    HFA_REQUIRE((y || partial || pairs) && out && n_rows > 0 && width > 0 && (!y || ldy >= width) && ldo >= width && (!gate || ldg >= width) &&
                    (!copy || ldc >= width) && (!pairs || top > 0) && (!partial || splits > 0), "rmsnorm_add: bad arguments");
    HFA_REQUIRE(!gate || gate_dtype == HFA_F32 || gate_dtype == HFA_BF16, "rmsnorm_add: unknown gate dtype %d", gate_dtype);
    HFA_REQUIRE(gate || !gate_bias, "rmsnorm_add: a gate's bias without the gate");
    const JoinArgs p = {y, ldy, partial, splits, (size_t)n_rows * width, row_gate, ld_row_gate, pairs, top, gate, gate && gate_dtype == HFA_BF16,
                        ldg, gate_bias, w, out, ldo, (uint16_t*)copy, ldc, width, eps, scale, accumulate};
    const bool vec = width % 4 == 0 && (!y || (ldy % 4 == 0 && ((uintptr_t)y & 15) == 0)) && ((uintptr_t)partial & 15) == 0 && ((uintptr_t)pairs & 15) == 0 &&
                     ldo % 4 == 0 && ((uintptr_t)out & 15) == 0 && (!copy || (ldc % 4 == 0 && ((uintptr_t)copy & 7) == 0));
    if (vec) {
        // few rows: a row's loads are shared by as many threads as it has groups of four columns
        int threads = n_rows >= 512 ? 256 : 1024;
        while (threads > 64 && threads / 2 * 4 >= width) threads /= 2;
        rmsnorm_add_kernel<4><<<n_rows, threads, 0, stream>>>(p);
    } else {
        rmsnorm_add_kernel<1><<<n_rows, 256, 0, stream>>>(p);
    }
    HFA_LAUNCH_CHECK("rmsnorm_add");
    return 0;
}

// ---- an fp32 matrix in bf16 ------------------------------------------------------------------------------------------
__global__ void round_rows_kernel(const float* __restrict__ x, int ldx, uint16_t* __restrict__ out, int ldo, int width, size_t total) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (size_t)gridDim.x * blockDim.x) {
        const size_t r = i / width, c = i % width;
        out[r * ldo + c] = bf16_bits(x[r * ldx + c]);
    }
}

extern "C" int hfa_round_rows(const float* x, int ldx, void* out, int ldo, int n_rows, int width, hipStream_t stream) {
    HFA_REQUIRE(x && out && n_rows > 0 && width > 0 && ldx >= width && ldo >= width, "round_rows: bad arguments");
    const size_t total = (size_t)n_rows * width;
    const int blocks = (int)((total + 255) / 256 < 65535 ? (total + 255) / 256 : 65535);
    round_rows_kernel<<<blocks, 256, 0, stream>>>(x, ldx, (uint16_t*)out, ldo, width, total);
    HFA_LAUNCH_CHECK("round_rows");
    return 0;
}

// ---- an activation of normed powers ----------------------------------------------------------------------------------
// out = a N(z) + b N(z^2) + c N(z^3) + e over a row, N(u) = u / sqrt(mean(u^2) + eps); coef = (a, b, c, e) on the device.
// The three sums of squares (of z, z^2 and z^3) are taken in one pass, in fp32, in a fixed order.
template <typename TI, typename TO>
__global__ __launch_bounds__(1024) void polynorm_kernel(const TI* __restrict__ z, int ldz, const float* __restrict__ coef,
                                                      TO* __restrict__ out, int ldo, int width, float eps) {
    __shared__ float red[17];
    const int r = blockIdx.x;
    const TI* src = z + (size_t)r * ldz;
    float s1 = 0.f, s2 = 0.f, s3 = 0.f;
#pragma unroll 4
    for (int i = threadIdx.x; i < width; i += blockDim.x) {
        const float v = to_f32(src[i]), v2 = v * v, v3 = v2 * v;
        s1 = fmaf(v, v, s1);
        s2 = fmaf(v2, v2, s2);
        s3 = fmaf(v3, v3, s3);
    }
    const float n = (float)width;
    const float i1 = coef[0] / sqrtf(block_sum(s1, red) / n + eps);
    const float i2 = coef[1] / sqrtf(block_sum(s2, red) / n + eps);
    const float i3 = coef[2] / sqrtf(block_sum(s3, red) / n + eps);
    const float e = coef[3];
    TO* dst = out + (size_t)r * ldo;
#pragma unroll 4
    for (int i = threadIdx.x; i < width; i += blockDim.x) {
        const float v = to_f32(src[i]), v2 = v * v;
        dst[i] = from_f32<TO>(v * i1 + v2 * i2 + v2 * v * i3 + e);
    }
}

extern "C" int hfa_polynorm(const void* z, int z_dtype, int ldz, const float* coef, void* out, int out_dtype, int ldo, int n_rows,
                            int width, float eps, hipStream_t stream) {
    HFA_REQUIRE(z && coef && out && n_rows > 0 && width > 0 && ldz >= width && ldo >= width, "polynorm: bad arguments");
    HFA_REQUIRE((z_dtype == HFA_F32 || z_dtype == HFA_BF16) && (out_dtype == HFA_F32 || out_dtype == HFA_BF16), "polynorm: unknown dtype");
    const int threads = width >= 4096 ? 1024 : 256;       // few rows in a decode step: a wide row is shared by more threads
#define PN(TI, TO) polynorm_kernel<TI, TO><<<n_rows, threads, 0, stream>>>((const TI*)z, ldz, coef, (TO*)out, ldo, width, eps)
    if (z_dtype == HFA_F32) { if (out_dtype == HFA_F32) PN(float, float); else PN(float, bf16); }
    else { if (out_dtype == HFA_F32) PN(bf16, float); else PN(bf16, bf16); }
#undef PN
    HFA_LAUNCH_CHECK("polynorm");
    return 0;
}

// ---- x *= s on fp32 rows ---------------------------------------------------------------------------------------------
__global__ void scale_rows_kernel(float* __restrict__ x, int ld, int width, float s, size_t total) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (size_t)gridDim.x * blockDim.x) {
        float* p = x + (i / width) * ld + i % width;
        *p = *p * s;
    }
}

extern "C" int hfa_scale_rows(float* x, int ld, int n_rows, int width, float s, hipStream_t stream) {
    HFA_REQUIRE(x && n_rows > 0 && width > 0 && ld >= width, "scale_rows: bad arguments");
    const size_t total = (size_t)n_rows * width;
    const int blocks = (int)((total + 255) / 256 < 65535 ? (total + 255) / 256 : 65535);
    scale_rows_kernel<<<blocks, 256, 0, stream>>>(x, ld, width, s, total);
    HFA_LAUNCH_CHECK("scale_rows");
    return 0;
}

// ---- queries and keys normed head by head; keys and values to the cache ------------------------------------------------
// Rows [q: H D | k: G D | v: GV Dv] (fp32 or bf16). Every q head and every k head is (norm_q, norm_k) divided by sqrt(mean(head^2) +
// eps) and multiplied by a weight of D values that all heads share (q_w, k_w; null: 1), and (cs not null) its first rot_dim
// dimensions are turned, i with i + rot_dim / 2, by the token's angles (cs: hfa_rope_table's rows [cosines | sines]); norm_after:
// the rotation comes first and the norm after it. q goes to q_out ([T, H D], the cache's dtype), k to cache row slot_map[t], v to
// the same row with the page transposed ([page][column][offset]).
struct HeadNorm {
    int H, G, D, GV, Dv;
    const float* q_w; const float* k_w;
    int norm_q, norm_k, norm_after;
    float eps;
    const float* cs; int rot_dim;
    const int* slot_map; int page_tokens;
};

// One head's values by S neighbouring lanes (a power of two), D <= S NE: lane l holds values l, l + S, ...
template <typename TI, int S, int NE>
__device__ __forceinline__ void normed_head(const TI* __restrict__ src, const HeadNorm& p, bool is_key, int t, int l, float (&v)[NE]) {
    const int half = p.rot_dim / 2;
    const float* cs = p.cs ? p.cs + (size_t)t * p.rot_dim : nullptr;
    const float* w = is_key ? p.k_w : p.q_w;
    const bool norm = is_key ? p.norm_k : p.norm_q;
    float other[NE];
#pragma unroll
    for (int i = 0; i < NE; i++) {
        const int c = l + i * S;
        v[i] = c < p.D ? to_f32(src[c]) : 0.f;
        other[i] = cs && c < p.rot_dim ? to_f32(src[c < half ? c + half : c - half]) : 0.f;
    }
    float ss = 0.f;
    auto turn = [&](float x, float y, int c) {              // c's place in its pair decides the sign
        return c < half ? x * cs[c] - y * cs[half + c] : x * cs[c - half] + y * cs[c];
    };
    if (norm && !p.norm_after) {
#pragma unroll
        for (int i = 0; i < NE; i++) ss = fmaf(v[i], v[i], ss);
    } else if (cs) {
#pragma unroll
        for (int i = 0; i < NE; i++) {
            const int c = l + i * S;
            if (c < p.rot_dim) v[i] = turn(v[i], other[i], c);
        }
    }
    if (norm && p.norm_after) {
#pragma unroll
        for (int i = 0; i < NE; i++) ss = fmaf(v[i], v[i], ss);
    }
    if (norm) {
#pragma unroll
        for (int off = S / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, WAVE);
        const float inv = 1.0f / sqrtf(ss / (float)p.D + p.eps);
#pragma unroll
        for (int i = 0; i < NE; i++) {
            const int c = l + i * S;
            if (c >= p.D) continue;
            v[i] *= inv * (w ? w[c] : 1.f);
            if (!p.norm_after && cs && c < p.rot_dim) {
                const int o = c < half ? c + half : c - half;
                v[i] = turn(v[i], other[i] * inv * (w ? w[o] : 1.f), c);
            }
        }
    }
}

// A block of four waves a token and 4 * 64 / S heads; the blocks of a token share its values out.
template <typename TI, typename TO, int S, int NE>
__global__ __launch_bounds__(256) void head_norm_store_kernel(const TI* __restrict__ qkv, int ld, HeadNorm p, TO* __restrict__ q_out, int ldq,
                                                             TO* __restrict__ k_cache, TO* __restrict__ v_cache) {
    const int t = blockIdx.x, l = threadIdx.x % S, H = p.H, G = p.G, D = p.D;
    const TI* row = qkv + (size_t)t * ld;
    const int KD = G * D, VD = p.GV * p.Dv;
    const int slot = p.slot_map[t];
    const int hs = blockIdx.y * (256 / S) + threadIdx.x / S;
    // (every lane of a wave takes part in the sums; lanes beyond the last head repeat it and store nothing)
    const int hc = hs < H + G ? hs : H + G - 1;
    float v[NE];
    normed_head<TI, S, NE>(row + hc * D, p, hc >= H, t, l, v);
    if (hs < H + G) {
        TO* dst = hs >= H ? k_cache + (size_t)slot * KD + (hs - H) * D : q_out + (size_t)t * ldq + hs * D;
#pragma unroll
        for (int i = 0; i < NE; i++)
            if (l + i * S < D) dst[l + i * S] = from_f32<TO>(v[i]);
    }
    for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < VD; c += gridDim.y * blockDim.x)
        v_cache[(size_t)(slot / p.page_tokens) * p.page_tokens * VD + (size_t)c * p.page_tokens + slot % p.page_tokens] =
            from_f32<TO>(to_f32(row[(H + G) * D + c]));
}

extern "C" int hfa_head_norm_store(const void* qkv, int in_dtype, int ld, int n_heads, int n_kv_heads, int head_dim, int n_v_heads, int v_head_dim,
                                   const float* q_w, const float* k_w, int norm_q, int norm_k, int norm_after, float eps, const float* cos_sin,
                                   int rot_dim, void* q_out, int ldq, void* k_cache, void* v_cache, int out_dtype, const int* slot_map,
                                   int page_tokens, int n_tokens, hipStream_t stream) {
    HFA_REQUIRE(qkv && q_out && k_cache && v_cache && slot_map && n_tokens > 0 && n_heads > 0 && n_kv_heads > 0 && head_dim > 0 &&
                    n_v_heads > 0 && v_head_dim > 0 && page_tokens > 0, "head_norm_store: bad arguments");
    HFA_REQUIRE(ld >= (n_heads + n_kv_heads) * head_dim + n_v_heads * v_head_dim && ldq >= n_heads * head_dim,
                "head_norm_store: a row is shorter than its heads");
    HFA_REQUIRE((in_dtype == HFA_F32 || in_dtype == HFA_BF16) && (out_dtype == HFA_F32 || out_dtype == HFA_BF16),
                "head_norm_store: unknown dtype");
    HFA_REQUIRE(head_dim <= 1024 && (!cos_sin || (rot_dim > 0 && rot_dim % 2 == 0 && rot_dim <= head_dim)),
                "head_norm_store: heads of %d values (at most 1024), of which an even number within the head is turned", head_dim);
    const HeadNorm p = {n_heads, n_kv_heads, head_dim, n_v_heads, v_head_dim, q_w, k_w, norm_q, norm_k, norm_after, eps, cos_sin,
                        cos_sin ? rot_dim : 0, slot_map, page_tokens};
#define HNS(TI, TO, S, NE)                                                                                                       \
    head_norm_store_kernel<TI, TO, S, NE><<<dim3(n_tokens, (n_heads + n_kv_heads + 256 / S - 1) / (256 / S)), 256, 0, stream>>>(     \
        (const TI*)qkv, ld, p, (TO*)q_out, ldq, (TO*)k_cache, (TO*)v_cache)
#define HNS_SIZES(TI, TO)                            \
    do {                                             \
        if (head_dim <= 32) HNS(TI, TO, 16, 2);      \
        else if (head_dim <= 64) HNS(TI, TO, 32, 2); \
        else if (head_dim <= 128) HNS(TI, TO, 64, 2); \
        else if (head_dim <= 256) HNS(TI, TO, 64, 4); \
        else HNS(TI, TO, 64, 16);                    \
    } while (0)
    if (in_dtype == HFA_F32) { if (out_dtype == HFA_F32) HNS_SIZES(float, float); else HNS_SIZES(float, bf16); }
    else { if (out_dtype == HFA_F32) HNS_SIZES(bf16, float); else HNS_SIZES(bf16, bf16); }
#undef HNS_SIZES
#undef HNS
    HFA_LAUNCH_CHECK("head_norm_store");
    return 0;
}

// ---- two attention maps of a head as one -----------------------------------------------------------------------------
// a [T][G][2][R][Dv] (fp32; the two maps of the R heads of each of G groups): out[t, g R + r] = c d / sqrt(mean(d^2) + eps) with
// d = a[t, g, 0, r] - factor[0] a[t, g, 1, r]. S lanes a head, 256 / S heads a block.
template <typename TO, int S, int NE>
__global__ __launch_bounds__(256) void diff_mix_kernel(const float* __restrict__ a, int lda, const float* __restrict__ factor, float c, float eps,
                                                      TO* __restrict__ out, int ldo, int H, int R, int Dv) {
    const int t = blockIdx.x, l = threadIdx.x % S, hs = blockIdx.y * (256 / S) + threadIdx.x / S;
    const int h = hs < H ? hs : H - 1, g = h / R, r = h % R;
    const float* a1 = a + (size_t)t * lda + (size_t)(2 * g * R + r) * Dv;
    const float* a2 = a1 + (size_t)R * Dv;
    const float f = factor[0];
    float d[NE], ss = 0.f;
#pragma unroll
    for (int i = 0; i < NE; i++) {
        const int x = l + i * S;
        d[i] = x < Dv ? a1[x] - f * a2[x] : 0.f;
        ss = fmaf(d[i], d[i], ss);
    }
#pragma unroll
    for (int off = S / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, WAVE);
    const float inv = c / sqrtf(ss / (float)Dv + eps);
    if (hs >= H) return;
#pragma unroll
    for (int i = 0; i < NE; i++)
        if (l + i * S < Dv) out[(size_t)t * ldo + (size_t)h * Dv + l + i * S] = from_f32<TO>(d[i] * inv);
}

extern "C" int hfa_diff_mix(const float* a, int lda, const float* factor, float c, float eps, void* out, int out_dtype, int ldo, int n_tokens,
                            int n_heads, int n_kv_heads, int v_head_dim, hipStream_t stream) {
    HFA_REQUIRE(a && factor && out && n_tokens > 0 && n_heads > 0 && n_kv_heads > 0 && n_heads % n_kv_heads == 0 && v_head_dim > 0,
                "diff_mix: bad arguments");
    HFA_REQUIRE(lda >= 2 * n_heads * v_head_dim && ldo >= n_heads * v_head_dim && v_head_dim <= 1024, "diff_mix: a row is shorter than its heads, "
                "or a head has more than 1024 values");
    HFA_REQUIRE(out_dtype == HFA_F32 || out_dtype == HFA_BF16, "diff_mix: unknown dtype %d", out_dtype);
#define DM(TO, S, NE)                                                                                                            \
    diff_mix_kernel<TO, S, NE><<<dim3(n_tokens, (n_heads + 256 / S - 1) / (256 / S)), 256, 0, stream>>>(a, lda, factor, c, eps, (TO*)out, ldo, \
                                                                                                        n_heads, n_heads / n_kv_heads, v_head_dim)
#define DM_SIZES(TO)                             \
    do {                                         \
        if (v_head_dim <= 64) DM(TO, 32, 2);     \
        else if (v_head_dim <= 128) DM(TO, 64, 2); \
        else if (v_head_dim <= 256) DM(TO, 64, 4); \
        else DM(TO, 64, 16);                     \
    } while (0)
    if (out_dtype == HFA_F32) DM_SIZES(float); else DM_SIZES(bf16);
#undef DM_SIZES
#undef DM
    HFA_LAUNCH_CHECK("diff_mix");
    return 0;
}

// ---- attention weights mixed across heads, as a sum of attention outputs ------------------------------------------------
// Mixing the heads' softmax weights, weight_h <- sum_g talk[h, g] weight_g, before head h applies them to the values of its
// own group c(h) is, by linearity, out_h = sum_g talk[h, g] A(g, c(h)), where A(g, c) is what head g's weights give on the
// values of group c. `cross` holds these: [T][G rounds][H heads][Dv], round r of head g being its weights on the values
// of group (c(g) + r) mod G (hfa_paged_attention with cross_values). gate (null: none): out is multiplied by
// sigmoid(gate[t, h Dv + d]). Sums in fp32 in the order of g.
// A block a (token, head): with few tokens (a decode step) there are still heads x tokens blocks to fill the machine.
template <typename TA, typename TG, typename TO>
__global__ __launch_bounds__(128) void talk_mix_kernel(const TA* __restrict__ cross, const float* __restrict__ talk,
                                                      const TG* __restrict__ gate, int ldg, TO* __restrict__ out, int ldo, int H,
                                                      int G, int Dv) {
    extern __shared__ float talk_s[];                      // row h of the mix, and where each head's round for h's group lies
    int* at_s = reinterpret_cast<int*>(talk_s + H);
    const int t = blockIdx.x, h = blockIdx.y, per = H / G, c = h / per;
    for (int g = threadIdx.x; g < H; g += blockDim.x) {
        talk_s[g] = talk[h * H + g];
        at_s[g] = (((c - g / per + G) % G) * H + g) * Dv;
    }
    __syncthreads();
    const TA* A = cross + (size_t)t * G * H * Dv;
    for (int d = threadIdx.x; d < Dv; d += blockDim.x) {
        float acc = 0.f;
#pragma unroll 4
        for (int g = 0; g < H; g++) acc = fmaf(talk_s[g], to_f32(A[at_s[g] + d]), acc);
        const int i = h * Dv + d;
        if (gate) acc *= 1.0f / (1.0f + expf(-to_f32(gate[(size_t)t * ldg + i])));
        out[(size_t)t * ldo + i] = from_f32<TO>(acc);
    }
}

extern "C" int hfa_talk_mix(const void* cross, int cross_dtype, const float* talk, const void* gate, int gate_dtype, int ldg, void* out,
                            int out_dtype, int ldo, int n_tokens, int n_heads, int n_kv_heads, int v_head_dim, hipStream_t stream) {
    HFA_REQUIRE(cross && talk && out && n_tokens > 0 && n_heads > 0 && n_kv_heads > 0 && n_heads % n_kv_heads == 0 && v_head_dim > 0,
                "talk_mix: bad arguments");
    HFA_REQUIRE(n_heads <= 128, "talk_mix: %d heads (at most 128)", n_heads);
    HFA_REQUIRE(ldo >= n_heads * v_head_dim && (!gate || ldg >= n_heads * v_head_dim), "talk_mix: a row is shorter than its heads");
    const size_t lds = (size_t)n_heads * (sizeof(float) + sizeof(int));
    const int code = (cross_dtype == HFA_BF16 ? 4 : 0) + ((gate && gate_dtype == HFA_BF16) ? 2 : 0) + (out_dtype == HFA_BF16 ? 1 : 0);
#define TM(TA, TG, TO)                                                                                                          \
    talk_mix_kernel<TA, TG, TO><<<dim3(n_tokens, n_heads), 128, lds, stream>>>((const TA*)cross, talk, (const TG*)gate, ldg, (TO*)out, ldo, n_heads, \
                                                                n_kv_heads, v_head_dim)
    switch (code) {
        case 0: TM(float, float, float); break;
        case 1: TM(float, float, bf16); break;
        case 2: TM(float, bf16, float); break;
        case 3: TM(float, bf16, bf16); break;
        case 4: TM(bf16, float, float); break;
        case 5: TM(bf16, float, bf16); break;
        case 6: TM(bf16, bf16, float); break;
        default: TM(bf16, bf16, bf16); break;
    }
#undef TM
    HFA_LAUNCH_CHECK("talk_mix");
    return 0;
}
