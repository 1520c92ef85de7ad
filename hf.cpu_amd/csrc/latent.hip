// Attention whose keys and values are expanded from one latent a token: what lies between the projections and the attention
// kernels. With the expansion folded into the queries (q' = Wuk^T q) and taken out of the values (o = Wuv sum p c), the cache
// holds one key/value head a token: key [rotated part | latent], value [latent].
//
//   hfa_latent_store   norm of the latent, rotation of the key's and the queries' rotated parts, the store into the cache
//   hfa_head_rows      the heads' products (the keys' expansion into the queries, the values' after the weighted sum, with
//                      a gate) for the few rows of a decode step, in one launch
#include "api.h"
#include "common.h"

#define LATENT_MAX_ROT 512

// One block a token. down[t] = [latent before its norm: C | rotated key part: R] (fp32); q[t] head by head [D | R].
template <typename TQ, typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(const float* __restrict__ down, int ld_down, const TQ* __restrict__ q, int ldq,
                                                          const float* __restrict__ w, float eps, const int* __restrict__ positions,
                                                          const float* __restrict__ inv_freq, int rot_dim, int pairing,
                                                          T* __restrict__ q_out, int ld_out, T* __restrict__ k_cache, T* __restrict__ v_cache,
                                                          const int* __restrict__ slot_map, int page_tokens, int H, int D, int R, int C) {
    __shared__ float red[17];
    __shared__ float cos_s[LATENT_MAX_ROT / 2], sin_s[LATENT_MAX_ROT / 2];
    const int t = blockIdx.x, tid = threadIdx.x, half = rot_dim / 2;
    const float* dr = down + (size_t)t * ld_down;
    const float pos = rot_dim > 0 ? (float)positions[t] : 0.f;
    for (int i = tid; i < half; i += blockDim.x) sincosf(pos * inv_freq[i], &sin_s[i], &cos_s[i]);
    float ss = 0.f;
    for (int i = tid; i < C; i += blockDim.x) ss = fmaf(dr[i], dr[i], ss);
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)C + eps);          // (its barriers also cover the angles)
    const size_t slot = (size_t)slot_map[t];
    T* key = k_cache + slot * (R + C);
    T* val = v_cache + slot / page_tokens * page_tokens * C + slot % page_tokens;
    for (int i = tid; i < C; i += blockDim.x) {
        const T c = from_f32<T>(dr[i] * inv * w[i]);
        key[R + i] = c;
        val[(size_t)i * page_tokens] = c;
    }
    // the rotated parts of the heads and of the key: pairs of dimensions, then the dimensions that pass (rot_dim < R)
    const int items = half + (R - rot_dim), total = (H + 1) * items;
    const TQ* qr = q + (size_t)t * ldq;
    for (int it = tid; it < total; it += blockDim.x) {
        const int h = it / items, j = it % items;
        auto in = [&](int i) { return h < H ? to_f32(qr[(size_t)h * (D + R) + D + i]) : dr[C + i]; };
        T* dst = h < H ? q_out + (size_t)t * ld_out + (size_t)h * (R + C) : key;
        if (j < half) {
            const int i0 = pairing == 1 ? 2 * j : j, i1 = pairing == 1 ? 2 * j + 1 : j + half;
            const float a = in(i0), b = in(i1);
            dst[i0] = from_f32<T>(a * cos_s[j] - b * sin_s[j]);
            dst[i1] = from_f32<T>(b * cos_s[j] + a * sin_s[j]);
        } else {
            const int i = rot_dim + (j - half);
            dst[i] = from_f32<T>(in(i));
        }
    }
}

extern "C" int hfa_latent_store(const float* down, int ld_down, const void* q, int q_dtype, int ldq, const float* w, float eps,
                                const int* positions, const float* inv_freq, int rot_dim, int pairing, void* q_out, int ld_out,
                                void* k_cache, void* v_cache, int dtype, const int* slot_map, int page_tokens, int n_tokens, int n_heads,
                                int dim, int rot, int latent, hipStream_t stream) {
    HFA_REQUIRE(down && q && w && q_out && k_cache && v_cache && slot_map && page_tokens > 0 && n_tokens > 0 && n_heads > 0 && dim >= 0 &&
                    rot >= 0 && latent > 0, "latent_store: bad arguments");
    HFA_REQUIRE(rot <= LATENT_MAX_ROT && rot_dim >= 0 && rot_dim % 2 == 0 && rot_dim <= rot && (rot_dim == 0 || (positions && inv_freq)) &&
                    (pairing == 0 || pairing == 1), "latent_store: a rotated part of %d (at most %d), %d of it turned", rot, LATENT_MAX_ROT, rot_dim);
    HFA_REQUIRE(ld_down >= latent + rot && ldq >= n_heads * (dim + rot) && ld_out >= n_heads * (rot + latent),
                "latent_store: a row is shorter than its parts");
    HFA_REQUIRE((q_dtype == HFA_F32 || q_dtype == HFA_BF16) && (dtype == HFA_F32 || (dtype == HFA_BF16)) && !(q_dtype == HFA_BF16 && dtype == HFA_F32),
                "latent_store: the queries are fp32 or of the cache's type");
#define LS(TQ, T) latent_store_kernel<TQ, T><<<n_tokens, 256, 0, stream>>>(down, ld_down, (const TQ*)q, ldq, w, eps, positions, inv_freq, rot_dim, \
                                                                         pairing, (T*)q_out, ld_out, (T*)k_cache, (T*)v_cache, slot_map,         \
                                                                         page_tokens, n_heads, dim, rot, latent)
    if (dtype == HFA_F32) LS(float, float);
    else if (q_dtype == HFA_BF16) LS(bf16, bf16);
    else LS(float, bf16);
#undef LS
    HFA_LAUNCH_CHECK("latent_store");
    return 0;
}

// ---- the heads' products for few rows -----------------------------------------------------------------------------
// A block of four waves owns 32 outputs of one head for 32 rows: A = 32 rows of W_h from memory in operand layout, B = 32
// activation rows. The waves share out the steps of 16 along K; the partial sums meet in LDS and wave v finishes the outputs
// 8 v + 0 .. 7 of the 32 (element r of a lane is output 8 (r / 4) + 4 half + r % 4 of the lane's row).
typedef __bf16 hr_bf16x8 __attribute__((ext_vector_type(8)));
typedef float hr_floatx16 __attribute__((ext_vector_type(16)));
union HrFrag {
    uint4 u;
    hr_bf16x8 v;
};
__device__ __forceinline__ uint32_t hr_pair(float a, float b) { return (uint32_t)bf16_bits(a) | ((uint32_t)bf16_bits(b) << 16); }

__device__ __forceinline__ uint4 hr_load(const uint16_t* p) { return *reinterpret_cast<const uint4*>(p); }
__device__ __forceinline__ uint4 hr_load(const float* p) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    return make_uint4(hr_pair(a.x, a.y), hr_pair(a.z, a.w), hr_pair(b.x, b.y), hr_pair(b.z, b.w));
}

template <typename TA>
__global__ __launch_bounds__(4 * WAVE) void head_rows_kernel(const TA* __restrict__ a, int lda, int a_head, const uint16_t* __restrict__ w,
                                                           uint16_t* __restrict__ out, int ldo, int out_head, const float* __restrict__ gate,
                                                           int ldg, int n_rows, int N, int K) {
    __shared__ float part_s[4][16][WAVE];
    const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE, col = lane & 31, half = lane >> 5;
    const int n0 = blockIdx.x * 32, h = blockIdx.y, row = blockIdx.z * 32 + col;
    const bool ok = row < n_rows;
    const int r = ok ? row : n_rows - 1;
    const TA* ap = a + (size_t)r * lda + (size_t)h * a_head + half * 8;
    const uint16_t* wp = w + ((size_t)h * N + n0 + col) * K + half * 8;
    hr_floatx16 st;
#pragma unroll
    for (int i = 0; i < 16; i++) st[i] = 0.f;
    const int steps = K / 16;
#pragma unroll 4
    for (int ks = wave; ks < steps; ks += 4) {
        HrFrag fa, fw;
        fw.u = hr_load(wp + ks * 16);
        fa.u = hr_load(ap + ks * 16);
        st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fw.v, fa.v, st, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 16; i++) part_s[wave][i][lane] = st[i];
    __syncthreads();
    if (!ok) return;
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; e++) {
        const int i = 4 * wave + e;
        v[e] = ((part_s[0][i][lane] + part_s[1][i][lane]) + part_s[2][i][lane]) + part_s[3][i][lane];
    }
    const int n = n0 + 8 * wave + 4 * half;
    if (gate) {
        const float* g = gate + (size_t)row * ldg + (size_t)h * N + n;
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] *= 1.0f / (1.0f + expf(-g[e]));
    }
    *reinterpret_cast<uint2*>(out + (size_t)row * ldo + (size_t)h * out_head + n) = make_uint2(hr_pair(v[0], v[1]), hr_pair(v[2], v[3]));
}

extern "C" int hfa_head_rows(const void* a, int a_dtype, int lda, int a_head, const void* w, void* out, int ldo, int out_head,
                             const float* gate, int ldg, int n_rows, int n_heads, int N, int K, hipStream_t stream) {
    HFA_REQUIRE(a && w && out && n_rows > 0 && n_heads > 0 && N > 0 && K > 0, "head_rows: bad arguments");
    HFA_REQUIRE(N % 32 == 0 && K % 16 == 0 && n_heads <= 65535 && (n_rows + 31) / 32 <= 65535, "head_rows: %d outputs of %d values a head", N, K);
    HFA_REQUIRE(lda >= (n_heads - 1) * a_head + K && ldo >= (n_heads - 1) * out_head + N && a_head >= 0 && out_head >= N && (!gate || ldg >= n_heads * N),
                "head_rows: a row is shorter than its heads");
    const int al = a_dtype == HFA_F32 ? 4 : 8;
    HFA_REQUIRE((a_dtype == HFA_F32 || a_dtype == HFA_BF16) && lda % al == 0 && a_head % al == 0 && ldo % 4 == 0 && out_head % 4 == 0 &&
                    ((uintptr_t)a & 15) == 0 && ((uintptr_t)w & 15) == 0 && ((uintptr_t)out & 7) == 0, "head_rows: an operand is not aligned");
    dim3 grid(N / 32, n_heads, (n_rows + 31) / 32);
    if (a_dtype == HFA_F32)
        head_rows_kernel<float><<<grid, 4 * WAVE, 0, stream>>>((const float*)a, lda, a_head, (const uint16_t*)w, (uint16_t*)out, ldo, out_head,
                                                               gate, ldg, n_rows, N, K);
    else
        head_rows_kernel<uint16_t><<<grid, 4 * WAVE, 0, stream>>>((const uint16_t*)a, lda, a_head, (const uint16_t*)w, (uint16_t*)out, ldo, out_head,
                                                                  gate, ldg, n_rows, N, K);
    HFA_LAUNCH_CHECK("head_rows");
    return 0;
}
