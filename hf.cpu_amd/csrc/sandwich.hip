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
//                         rotation; q to a matrix, k and v to their cache rows (or, without keys, v to a matrix)
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
                                 const float* __restrict__ inv_freq, float* __restrict__ x, int width, int vocab, float scale,
                                 uint16_t* __restrict__ copy) {
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
        if (copy) copy[(size_t)t * width + i] = bf16_bits(v);
    }
}

extern "C" int hfa_embed_pos(const void* table, int table_dtype, const int* tokens, const int* positions, const float* inv_freq,
                             float* x, int n_tokens, int width, int vocab, float scale, void* copy, hipStream_t stream) {
    HFA_REQUIRE(table && tokens && x && n_tokens > 0 && width > 0 && vocab > 0, "embed_pos: bad arguments");
    HFA_REQUIRE(!positions || inv_freq, "embed_pos: positions come with their frequencies");
    HFA_REQUIRE(table_dtype == HFA_F32 || table_dtype == HFA_BF16, "embed_pos: unknown dtype %d", table_dtype);
    if (table_dtype == HFA_F32)
        embed_pos_kernel<float><<<n_tokens, 256, 0, stream>>>((const float*)table, tokens, positions, inv_freq, x, width, vocab, scale, (uint16_t*)copy);
    else
        embed_pos_kernel<bf16><<<n_tokens, 256, 0, stream>>>((const bf16*)table, tokens, positions, inv_freq, x, width, vocab, scale, (uint16_t*)copy);
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
    float* dst = p.out + (size_t)r * p.ldo;
    // what the last lines need from memory is asked for with the branch, so that no trip waits behind the block's sum
    JoinVec<VW> old[KEEP], wv[KEEP];
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
        const int c = c0 + k * stride;
        old[k] = p.accumulate && c < p.width ? join_load<VW>(dst + c) : JoinVec<VW>{};
        wv[k] = p.w && c < p.width ? join_load<VW>(p.w + c) : JoinVec<VW>{};
    }
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
    auto finish = [&](int c, const JoinVec<VW>& b, const JoinVec<VW>& o, const JoinVec<VW>& w) {
        JoinVec<VW> z;
#pragma unroll
        for (int e = 0; e < VW; e++) z.v[e] = o.v[e] + (p.w ? b.v[e] * inv * w.v[e] : b.v[e] * inv);
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
        if (c < p.width) finish(c, keep[k], old[k], wv[k]);
    }
    for (int c = c0 + KEEP * stride; c < p.width; c += stride)
        finish(c, value(c), p.accumulate ? join_load<VW>(dst + c) : JoinVec<VW>{}, p.w ? join_load<VW>(p.w + c) : JoinVec<VW>{});
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
    const bool vec = width % 4 == 0 && ((uintptr_t)w & 15) == 0 && (!y || (ldy % 4 == 0 && ((uintptr_t)y & 15) == 0)) && ((uintptr_t)partial & 15) == 0 && ((uintptr_t)pairs & 15) == 0 &&
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
// Rows [q: H D | k: G D | v: GV Dv | extra] (fp32, bf16, or the partial sums of a product whose K was split, plus its bias). Every q
// head and every k head is (norm_q, norm_k) divided by sqrt(mean(head^2) + eps) and multiplied by a weight of D values that all heads
// share (q_w, k_w; null: 1), and (cs not null) its first rot_dim dimensions are turned, i with i + rot_dim / 2, by the token's angles
// (cs: hfa_rope_table's rows [cosines | sines]); norm_after: the rotation comes first and the norm after it. q goes to q_out ([T, H D]),
// k to cache row slot_map[t], v to the same row with the page transposed ([page][column][offset]); without a cache (k_cache null) there
// are no k heads and v goes to v_rows ([T, GV Dv]). The extra columns go to `extra` in fp32 (null: they are left alone).
struct HeadNorm {
    int H, G, D, GV, Dv;
    const float* q_w; const float* k_w;
    int norm_q, norm_k, norm_after;
    float eps;
    const float* cs; int rot_dim;
    const int* slot_map; int page_tokens;
    const float* partial; int splits, width; size_t plane;       // partial sums: [splits][T][width], or null
    const float* bias;                                           // [width], with partial sums
    float* extra; int n_extra, ld_extra;
    int ldv;                                                     // of v_rows
};

template <typename TI>
struct HeadRow {
    const TI* row;
    const float* sums;               // the token's row of the first plane, or null
    const HeadNorm* p;
    __device__ __forceinline__ float at(int c) const {
        if (!sums) return to_f32(row[c]);
        if (p->splits == 1) return p->bias ? sums[c] + p->bias[c] : sums[c];
        float v = 0.f;
        for (int s0 = 0; s0 < p->splits; s0 += JOIN_PLANES) {    // batches of loads that do not wait for one another
            float q[JOIN_PLANES];
#pragma unroll
            for (int u = 0; u < JOIN_PLANES; u++) q[u] = s0 + u < p->splits ? sums[(s0 + u) * p->plane + c] : 0.f;
#pragma unroll
            for (int u = 0; u < JOIN_PLANES; u++) v += q[u];
        }
        return p->bias ? v + p->bias[c] : v;
    }
    // eight neighbouring columns (c a multiple of 8, operands on 16 bytes)
    __device__ __forceinline__ void at8(int c, float (&v)[8]) const {
        if (sums) {
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] = p->bias ? p->bias[c + e] : 0.f;
            for (int s = 0; s < p->splits; s++) {
                const float4 a = *reinterpret_cast<const float4*>(sums + s * p->plane + c);
                const float4 b = *reinterpret_cast<const float4*>(sums + s * p->plane + c + 4);
                v[0] += a.x; v[1] += a.y; v[2] += a.z; v[3] += a.w;
                v[4] += b.x; v[5] += b.y; v[6] += b.z; v[7] += b.w;
            }
        } else if constexpr (sizeof(TI) == 2) {
            const uint4 u = *reinterpret_cast<const uint4*>(row + c);
            const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
            for (int e = 0; e < 4; e++) {
                v[2 * e] = __uint_as_float(w[e] << 16);
                v[2 * e + 1] = __uint_as_float(w[e] & 0xffff0000u);
            }
        } else {
            const float4 a = *reinterpret_cast<const float4*>(row + c), b = *reinterpret_cast<const float4*>(row + c + 4);
            v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
            v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
        }
    }
};
template <typename TI>
__device__ __forceinline__ HeadRow<TI> head_row(const TI* qkv, int ld, const HeadNorm& p, int t) {
    return {qkv + (size_t)t * ld, p.partial ? p.partial + (size_t)t * p.width : nullptr, &p};
}

// One head's values by S neighbouring lanes (a power of two), D <= S NE: lane l holds values l, l + S, ...
template <typename TI, int S, int NE>
__device__ __forceinline__ void normed_head(const HeadRow<TI>& src, int first, const HeadNorm& p, bool is_key, int t, int l, float (&v)[NE]) {
    const int half = p.rot_dim / 2;
    const float* cs = p.cs ? p.cs + (size_t)t * p.rot_dim : nullptr;
    const float* w = is_key ? p.k_w : p.q_w;
    const bool norm = is_key ? p.norm_k : p.norm_q;
    float other[NE];
#pragma unroll
    for (int i = 0; i < NE; i++) {
        const int c = l + i * S;
        v[i] = c < p.D ? src.at(first + c) : 0.f;
        other[i] = cs && c < p.rot_dim ? src.at(first + (c < half ? c + half : c - half)) : 0.f;
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

// A block of four waves a token and 4 * 64 / S heads; the blocks of a token share its values and extra columns out.
template <typename TI, typename TO, int S, int NE>
__global__ __launch_bounds__(256) void head_norm_store_kernel(const TI* __restrict__ qkv, int ld, HeadNorm p, TO* __restrict__ q_out, int ldq,
                                                             TO* __restrict__ k_cache, TO* __restrict__ v_out) {
    const int t = blockIdx.x, l = threadIdx.x % S, H = p.H, G = p.G, D = p.D;
    const HeadRow<TI> row = head_row(qkv, ld, p, t);
    const int KD = G * D, VD = p.GV * p.Dv;
    const int slot = p.slot_map ? p.slot_map[t] : 0;
    const int hs = blockIdx.y * (256 / S) + threadIdx.x / S;
    // (every lane of a wave takes part in the sums; lanes beyond the last head repeat it and store nothing)
    const int hc = hs < H + G ? hs : H + G - 1;
    float v[NE];
    normed_head<TI, S, NE>(row, hc * D, p, hc >= H, t, l, v);
    if (hs < H + G) {
        TO* dst = hs >= H ? k_cache + (size_t)slot * KD + (hs - H) * D : q_out + (size_t)t * ldq + hs * D;
#pragma unroll
        for (int i = 0; i < NE; i++)
            if (l + i * S < D) dst[l + i * S] = from_f32<TO>(v[i]);
    }
    const int v0 = (H + G) * D;
    for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < VD; c += gridDim.y * blockDim.x) {
        const size_t at = k_cache ? (size_t)(slot / p.page_tokens) * p.page_tokens * VD + (size_t)c * p.page_tokens + slot % p.page_tokens
                                  : (size_t)t * p.ldv + c;
        v_out[at] = from_f32<TO>(row.at(v0 + c));
    }
    if (p.extra)
        for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < p.n_extra; c += gridDim.y * blockDim.x)
            p.extra[(size_t)t * p.ld_extra + c] = row.at(v0 + VD + c);
}

// The same for prompt portions: HEAD_SHARES blocks take eight consecutive tokens, a share of the heads and of the values each; a head lies over L = D / 8 neighbouring lanes (4, 8 or 16) with
// eight values each, the other halves of its pairs come from the lanes that hold them, and the values of the eight tokens go
// through LDS, so that where the tokens' cache rows are neighbours on one page every value column is one 16-byte store.
#define HEAD_TOKENS 8
#define HEAD_SHARES 4
template <typename TO>
__device__ __forceinline__ void store8(TO* dst, const float (&v)[8]) {
    if constexpr (sizeof(TO) == 2) {
        uint32_t w[4];
#pragma unroll
        for (int e = 0; e < 4; e++) w[e] = (uint32_t)bf16_bits(v[2 * e]) | ((uint32_t)bf16_bits(v[2 * e + 1]) << 16);
        *reinterpret_cast<uint4*>(dst) = make_uint4(w[0], w[1], w[2], w[3]);
    } else {
        *reinterpret_cast<float4*>(dst) = make_float4(v[0], v[1], v[2], v[3]);
        *reinterpret_cast<float4*>(dst + 4) = make_float4(v[4], v[5], v[6], v[7]);
    }
}

template <typename TI, typename TO, int L>
__global__ __launch_bounds__(256) void head_norm_rows_kernel(const TI* __restrict__ qkv, int ld, HeadNorm p, TO* __restrict__ q_out, int ldq,
                                                            TO* __restrict__ k_cache, TO* __restrict__ v_out, int n_tokens) {
    extern __shared__ __attribute__((aligned(16))) uint16_t head_vt[];               // [HEAD_TOKENS][this block's values]
    constexpr int D = 8 * L, PER = 256 / L;
    const int t0 = blockIdx.x * HEAD_TOKENS, nt = n_tokens - t0 < HEAD_TOKENS ? n_tokens - t0 : HEAD_TOKENS;
    const int tid = threadIdx.x, l = tid % L, H = p.H, G = p.G, KD = G * D, VD = p.GV * p.Dv, v0 = (H + G) * D;
    const int half = p.rot_dim / 2, lanes_half = half / 8;                           // (half is a multiple of 8)
    const int heads = H + G, n_items = nt * heads;
    const bool turns = p.cs != nullptr && 8 * l < p.rot_dim, low = l < lanes_half;
    const int partner = low ? l + lanes_half : l - lanes_half;
    for (int i0 = blockIdx.y * PER; i0 < n_items; i0 += PER * HEAD_SHARES) {                                      // (uniform: every lane takes part in the exchanges)
        const int item = i0 + tid / L, it = item < n_items ? item : n_items - 1;
        const int t = t0 + it / heads, hs = it % heads;
        const bool is_key = hs >= H;
        const float* w = is_key ? p.k_w : p.q_w;
        const bool norm = is_key ? p.norm_k : p.norm_q;
        float v[8];
        head_row(qkv, ld, p, t).at8(hs * D + 8 * l, v);
        auto turn = [&]() {
            float o[8];
#pragma unroll
            for (int e = 0; e < 8; e++) o[e] = __shfl(v[e], turns ? partner : l, L);
            if (turns) {
                const float* cs = p.cs + (size_t)t * p.rot_dim + 8 * (low ? l : l - lanes_half);
                float cv[8], sv[8];
#pragma unroll
                for (int u = 0; u < 2; u++) {
                    *reinterpret_cast<float4*>(cv + 4 * u) = *reinterpret_cast<const float4*>(cs + 4 * u);
                    *reinterpret_cast<float4*>(sv + 4 * u) = *reinterpret_cast<const float4*>(cs + half + 4 * u);
                }
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] = low ? v[e] * cv[e] - o[e] * sv[e] : v[e] * cv[e] + o[e] * sv[e];
            }
        };
        if (p.cs && (p.norm_after || !norm)) turn();
        if (norm) {
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < 8; e++) ss = fmaf(v[e], v[e], ss);
#pragma unroll
            for (int off = L / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, L);
            const float inv = 1.0f / sqrtf(ss / (float)D + p.eps);
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] *= inv * (w ? w[8 * l + e] : 1.f);
            if (p.cs && !p.norm_after) turn();
        }
        if (item < n_items) {
            TO* dst = is_key ? k_cache + (size_t)p.slot_map[t] * KD + (hs - H) * D : q_out + (size_t)t * ldq + hs * D;
            store8(dst + 8 * l, v);
        }
    }
    if (p.extra)
        for (int i = blockIdx.y * 256 + tid; i < nt * p.n_extra; i += 256 * HEAD_SHARES)
            p.extra[(size_t)(t0 + i / p.n_extra) * p.ld_extra + i % p.n_extra] = head_row(qkv, ld, p, t0 + i / p.n_extra).at(v0 + VD + i % p.n_extra);
    // this block's columns of the values: v8 groups of eight from cv on
    const int all8 = VD / 8, share8 = (all8 + HEAD_SHARES - 1) / HEAD_SHARES, cv = (int)blockIdx.y * share8 * 8;
    const int v8 = all8 - cv / 8 < share8 ? all8 - cv / 8 : share8;
    if (v8 <= 0) return;                                                             // (uniform over the block)
    if (!k_cache) {
        for (int i = tid; i < nt * v8; i += 256) {
            const int t = t0 + i / v8, c = cv + i % v8 * 8;
            float v[8];
            head_row(qkv, ld, p, t).at8(v0 + c, v);
            store8(v_out + (size_t)t * p.ldv + c, v);
        }
        return;
    }
    if constexpr (sizeof(TO) == 2) {                                                 // (values into a cache: 16 bits only, see the launcher)
        for (int i = tid; i < nt * v8; i += 256) {
            float v[8];
            head_row(qkv, ld, p, t0 + i / v8).at8(v0 + cv + i % v8 * 8, v);
            store8(reinterpret_cast<TO*>(head_vt) + i / v8 * (8 * share8) + i % v8 * 8, v);
        }
        __shared__ int slots[HEAD_TOKENS];
        if (tid < HEAD_TOKENS) slots[tid] = tid < nt ? p.slot_map[t0 + tid] : -1;
        __syncthreads();
        const int P = p.page_tokens;
        bool run = nt == HEAD_TOKENS && P % 8 == 0 && slots[0] % 8 == 0;
        for (int t = 1; run && t < HEAD_TOKENS; t++) run = slots[t] == slots[0] + t;
        uint16_t* vc = reinterpret_cast<uint16_t*>(v_out);
        if (run) {
            uint16_t* page = vc + (size_t)(slots[0] / P) * P * VD + (size_t)cv * P + slots[0] % P;
            for (int c = tid; c < 8 * v8; c += 256) {
                uint16_t x[HEAD_TOKENS];
#pragma unroll
                for (int t = 0; t < HEAD_TOKENS; t++) x[t] = head_vt[t * 8 * share8 + c];
                *reinterpret_cast<uint4*>(page + (size_t)c * P) =
                    make_uint4(x[0] | ((uint32_t)x[1] << 16), x[2] | ((uint32_t)x[3] << 16), x[4] | ((uint32_t)x[5] << 16), x[6] | ((uint32_t)x[7] << 16));
            }
        } else {
            for (int i = tid; i < nt * 8 * v8; i += 256) {
                const int t = i / (8 * v8), c = i % (8 * v8), slot = slots[t];
                vc[(size_t)(slot / P) * P * VD + (size_t)(cv + c) * P + slot % P] = head_vt[t * 8 * share8 + c];
            }
        }
    }
}

extern "C" int hfa_head_norm_store(const void* qkv, int in_dtype, int ld, int n_heads, int n_kv_heads, int head_dim, int n_v_heads, int v_head_dim,
                                   const float* q_w, const float* k_w, int norm_q, int norm_k, int norm_after, float eps, const float* cos_sin,
                                   int rot_dim, void* q_out, int ldq, void* k_cache, void* v_out, int ldv, int out_dtype, const int* slot_map,
                                   int page_tokens, int n_tokens, const float* partial, int splits, int width, const float* partial_bias,
                                   float* extra, int n_extra, int ld_extra, hipStream_t stream) {
    HFA_REQUIRE(qkv && q_out && v_out && n_tokens > 0 && n_heads > 0 && head_dim > 0 && n_v_heads > 0 && v_head_dim > 0, "head_norm_store: bad arguments");
    HFA_REQUIRE(k_cache ? n_kv_heads > 0 && slot_map && page_tokens > 0 : n_kv_heads == 0 && ldv >= n_v_heads * v_head_dim,
                "head_norm_store: keys need a cache and its rows; without a cache there are none, and the values' rows have a stride");
    const int used = (n_heads + n_kv_heads) * head_dim + n_v_heads * v_head_dim + (extra ? n_extra : 0);
    HFA_REQUIRE(ld >= used && ldq >= n_heads * head_dim && (!extra || (n_extra > 0 && ld_extra >= n_extra)), "head_norm_store: a row is shorter than its heads");
    HFA_REQUIRE(!partial || (splits > 0 && width >= used), "head_norm_store: partial sums of rows shorter than their heads");
    HFA_REQUIRE((in_dtype == HFA_F32 || in_dtype == HFA_BF16) && (out_dtype == HFA_F32 || out_dtype == HFA_BF16),
                "head_norm_store: unknown dtype");
    HFA_REQUIRE(head_dim <= 1024 && (!cos_sin || (rot_dim > 0 && rot_dim % 2 == 0 && rot_dim <= head_dim)),
                "head_norm_store: heads of %d values (at most 1024), of which an even number within the head is turned", head_dim);
    const int vd = n_v_heads * v_head_dim;
    const HeadNorm p = {n_heads, n_kv_heads, head_dim, n_v_heads, v_head_dim, q_w, k_w, norm_q, norm_k, norm_after, eps, cos_sin,
                        cos_sin ? rot_dim : 0, slot_map, page_tokens > 0 ? page_tokens : 1, partial, splits, width, (size_t)n_tokens * width, partial_bias,
                        extra, n_extra, ld_extra, ldv};
    // eight tokens a block: prompt-sized calls whose rows are made of 16-byte pieces
    const int in_step = in_dtype == HFA_F32 ? 4 : 8, out_step = out_dtype == HFA_F32 ? 4 : 8;
    const bool rows = n_tokens >= 512 && (head_dim == 32 || head_dim == 64 || head_dim == 128) && v_head_dim * n_v_heads % 8 == 0 && p.rot_dim % 16 == 0 &&
                      (k_cache == nullptr || (out_dtype == HFA_BF16 && (vd / 8 + HEAD_SHARES - 1) / HEAD_SHARES * 8 * HEAD_TOKENS * 2 <= (48 << 10))) &&
                      (partial ? width % 4 == 0 && ((uintptr_t)partial & 15) == 0 : ld % in_step == 0 && ((uintptr_t)qkv & 15) == 0) &&
                      ldq % out_step == 0 && (k_cache || ldv % out_step == 0) && (((uintptr_t)q_out | (uintptr_t)k_cache | (uintptr_t)v_out | (uintptr_t)cos_sin) & 15) == 0;
#define HNR(TI, TO, L)                                                                                                                \
    head_norm_rows_kernel<TI, TO, L><<<dim3((n_tokens + HEAD_TOKENS - 1) / HEAD_TOKENS, HEAD_SHARES), 256,                          \
                                           k_cache ? (vd / 8 + HEAD_SHARES - 1) / HEAD_SHARES * 8 * HEAD_TOKENS * 2 : 0, stream>>>(   \
        (const TI*)qkv, ld, p, (TO*)q_out, ldq, (TO*)k_cache, (TO*)v_out, n_tokens)
#define HNS(TI, TO, S, NE)                                                                                                       \
    head_norm_store_kernel<TI, TO, S, NE><<<dim3(n_tokens, (n_heads + n_kv_heads + 256 / S - 1) / (256 / S)), 256, 0, stream>>>(     \
        (const TI*)qkv, ld, p, (TO*)q_out, ldq, (TO*)k_cache, (TO*)v_out)
#define HNS_SIZES(TI, TO)                            \
    do {                                             \
        if (rows && head_dim == 32) HNR(TI, TO, 4);  \
        else if (rows && head_dim == 64) HNR(TI, TO, 8); \
        else if (rows) HNR(TI, TO, 16);              \
        else if (head_dim <= 32) HNS(TI, TO, 16, 2); \
        else if (head_dim <= 64) HNS(TI, TO, 32, 2); \
        else if (head_dim <= 128) HNS(TI, TO, 64, 2); \
        else if (head_dim <= 256) HNS(TI, TO, 64, 4); \
        else HNS(TI, TO, 64, 16);                    \
    } while (0)
    if (in_dtype == HFA_F32) { if (out_dtype == HFA_F32) HNS_SIZES(float, float); else HNS_SIZES(float, bf16); }
    else { if (out_dtype == HFA_F32) HNS_SIZES(bf16, float); else HNS_SIZES(bf16, bf16); }
#undef HNS_SIZES
#undef HNS
#undef HNR
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
