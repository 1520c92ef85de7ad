// Attention whose keys and values are expanded from one latent a token: what lies between the projections and the attention
// kernels. With the expansion folded into the queries (q' = Wuk^T q) and taken out of the values (o = Wuv sum p c), the cache
// holds one key/value head a token: key [rotated part | latent], value [latent].
//
//   hfa_latent_store   norm of the latent, rotation of the key's and the queries' rotated parts, the store into the cache;
//                      for few rows also the products that fold the keys' expansion into the queries, in the same launch
//   hfa_head_rows      the heads' products (the values' expansion after the weighted sum, with a gate) for the few rows of
//                      a decode step, in one launch
#include "api.h"
#include "common.h"

#define LATENT_MAX_ROT 512
#define LATENT_THREADS 256

struct LatentRow {               // what the store of a step's rows needs
    const float* down; int ld_down;
    const float* w; float eps;
    const int* positions; const float* inv_freq;
    int rot_dim, pairing;
    int ld_out;
    const int* slot_map; int page_tokens;
    int H, D, R, C;
};

// One block a token. down[t] = [latent before its norm: C | rotated key part: R] (fp32); q[t] head by head [D | R].
template <typename TQ, typename T>
__device__ __forceinline__ void latent_store_row(const LatentRow& a, const TQ* __restrict__ q, int ldq, T* __restrict__ q_out,
                                                 T* __restrict__ k_cache, T* __restrict__ v_cache, int t, float* red, float* cos_s, float* sin_s) {
    const int tid = threadIdx.x, half = a.rot_dim / 2, R = a.R, C = a.C, H = a.H, D = a.D;
    const float* dr = a.down + (size_t)t * a.ld_down;
    // everything that the norm and the store want from memory is asked for before the angles are formed
    const size_t slot = (size_t)a.slot_map[t];
    float v[2], g[2];
#pragma unroll
    for (int u = 0; u < 2; u++) {
        const int i = tid + u * LATENT_THREADS;
        v[u] = i < C ? dr[i] : 0.f;
        g[u] = i < C ? a.w[i] : 0.f;
    }
    const float pos = a.rot_dim > 0 ? (float)a.positions[t] : 0.f;
    for (int i = tid; i < half; i += LATENT_THREADS) sincosf(pos * a.inv_freq[i], &sin_s[i], &cos_s[i]);
    float ss = v[0] * v[0] + v[1] * v[1];
    for (int i = tid + 2 * LATENT_THREADS; i < C; i += LATENT_THREADS) ss = fmaf(dr[i], dr[i], ss);
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)C + a.eps);          // (its barriers also cover the angles)
    T* key = k_cache + slot * (R + C);
    T* val = v_cache + slot / a.page_tokens * a.page_tokens * C + slot % a.page_tokens;
    for (int i = tid, u = 0; i < C; i += LATENT_THREADS, u++) {
        const T c = from_f32<T>(u < 2 ? v[u & 1] * inv * g[u & 1] : dr[i] * inv * a.w[i]);
        key[R + i] = c;
        val[(size_t)i * a.page_tokens] = c;
    }
    // the rotated parts of the heads and of the key: pairs of dimensions, then the dimensions that pass (rot_dim < R)
    const int items = half + (R - a.rot_dim), total = (H + 1) * items;
    const TQ* qr = q + (size_t)t * ldq;
    for (int it = tid; it < total; it += LATENT_THREADS) {
        const int h = it / items, j = it % items;
        auto in = [&](int i) { return h < H ? to_f32(qr[(size_t)h * (D + R) + D + i]) : dr[C + i]; };
        T* dst = h < H ? q_out + (size_t)t * a.ld_out + (size_t)h * (R + C) : key;
        if (j < half) {
            const int i0 = a.pairing == 1 ? 2 * j : j, i1 = a.pairing == 1 ? 2 * j + 1 : j + half;
            const float x0 = in(i0), x1 = in(i1);
            dst[i0] = from_f32<T>(x0 * cos_s[j] - x1 * sin_s[j]);
            dst[i1] = from_f32<T>(x1 * cos_s[j] + x0 * sin_s[j]);
        } else {
            const int i = a.rot_dim + (j - half);
            dst[i] = from_f32<T>(in(i));
        }
    }
}

template <typename TQ, typename T>
__global__ __launch_bounds__(LATENT_THREADS) void latent_store_kernel(LatentRow a, const TQ* __restrict__ q, int ldq, T* __restrict__ q_out,
                                                                     T* __restrict__ k_cache, T* __restrict__ v_cache) {
    __shared__ float red[17];
    __shared__ float cos_s[LATENT_MAX_ROT / 2], sin_s[LATENT_MAX_ROT / 2];
    latent_store_row<TQ, T>(a, q, ldq, q_out, k_cache, v_cache, blockIdx.x, red, cos_s, sin_s);
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

__device__ __forceinline__ uint4 hr_load(const bf16* p) { return *reinterpret_cast<const uint4*>(p); }
__device__ __forceinline__ uint4 hr_load(const float* p) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    return make_uint4(hr_pair(a.x, a.y), hr_pair(a.z, a.w), hr_pair(b.x, b.y), hr_pair(b.z, b.w));
}

struct HeadRows {
    int lda, a_head;
    const uint16_t* w;
    uint16_t* out; int ldo, out_head;
    const float* gate; int ldg;
    int n_rows, N, K;
};

template <typename TA>
__device__ __forceinline__ void head_rows_block(const HeadRows& p, const TA* __restrict__ a, int n0, int h, int row0, float (&part_s)[4][16][WAVE]) {
    const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE, col = lane & 31, half = lane >> 5;
    const int row = row0 + col;
    const bool ok = row < p.n_rows;
    const int r = ok ? row : p.n_rows - 1;
    const TA* ap = a + (size_t)r * p.lda + (size_t)h * p.a_head + half * 8;
    const uint16_t* wp = p.w + ((size_t)h * p.N + n0 + col) * p.K + half * 8;
    hr_floatx16 st;
#pragma unroll
    for (int i = 0; i < 16; i++) st[i] = 0.f;
    const int steps = p.K / 16;
#pragma unroll 8
    for (int ks = wave; ks < steps; ks += 4) {
        HrFrag fa, fw;
        fw.u = *reinterpret_cast<const uint4*>(wp + ks * 16);
        fa.u = hr_load(ap + ks * 16);
        st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fw.v, fa.v, st, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 16; i++) part_s[wave][i][lane] = st[i];
    const int n = n0 + 8 * wave + 4 * half;
    float g[4] = {0.f, 0.f, 0.f, 0.f};
    if (p.gate) {
#pragma unroll
        for (int e = 0; e < 4; e++) g[e] = p.gate[(size_t)r * p.ldg + (size_t)h * p.N + n + e];
    }
    __syncthreads();
    if (!ok) return;
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; e++) {
        const int i = 4 * wave + e;
        v[e] = ((part_s[0][i][lane] + part_s[1][i][lane]) + part_s[2][i][lane]) + part_s[3][i][lane];
        if (p.gate) v[e] *= 1.0f / (1.0f + expf(-g[e]));
    }
    *reinterpret_cast<uint2*>(p.out + (size_t)row * p.ldo + (size_t)h * p.out_head + n) = make_uint2(hr_pair(v[0], v[1]), hr_pair(v[2], v[3]));
}

template <typename TA>
__global__ __launch_bounds__(4 * WAVE) void head_rows_kernel(HeadRows p, const TA* __restrict__ a) {
    __shared__ float part_s[4][16][WAVE];
    head_rows_block<TA>(p, a, blockIdx.x * 32, blockIdx.y, blockIdx.z * 32, part_s);
}

// Both for few rows: blocks 0 .. n_fold - 1 fold, the rest store a row each. They read the same queries and write different
// parts of them.
template <typename TQ>
__global__ __launch_bounds__(4 * WAVE) void latent_fold_store_kernel(LatentRow a, HeadRows p, const TQ* __restrict__ q, int ldq,
                                                                    bf16* __restrict__ q_out, bf16* __restrict__ k_cache,
                                                                    bf16* __restrict__ v_cache, int n_fold) {
    __shared__ float part_s[4][16][WAVE];
    __shared__ float red[17];
    __shared__ float cos_s[LATENT_MAX_ROT / 2], sin_s[LATENT_MAX_ROT / 2];
    const int b = blockIdx.x;
    if (b < n_fold) {
        const int nx = p.N / 32;
        head_rows_block<TQ>(p, q, b % nx * 32, b / nx % a.H, b / nx / a.H * 32, part_s);
    } else {
        latent_store_row<TQ, bf16>(a, q, ldq, q_out, k_cache, v_cache, b - n_fold, red, cos_s, sin_s);
    }
}

static int check_head_rows(const char* what, const HeadRows& p, const void* a, int a_dtype, int n_heads) {
    HFA_REQUIRE(a && p.w && p.out && p.n_rows > 0 && n_heads > 0 && p.N > 0 && p.K > 0, "%s: bad arguments", what);
    HFA_REQUIRE(p.N % 32 == 0 && p.K % 16 == 0 && n_heads <= 65535 && (p.n_rows + 31) / 32 <= 65535, "%s: %d outputs of %d values a head", what, p.N, p.K);
    HFA_REQUIRE(p.lda >= (n_heads - 1) * p.a_head + p.K && p.ldo >= (n_heads - 1) * p.out_head + p.N && p.a_head >= 0 && p.out_head >= p.N &&
                    (!p.gate || p.ldg >= n_heads * p.N), "%s: a row is shorter than its heads", what);
    const int al = a_dtype == HFA_F32 ? 4 : 8;
    HFA_REQUIRE((a_dtype == HFA_F32 || a_dtype == HFA_BF16) && p.lda % al == 0 && p.a_head % al == 0 && p.ldo % 4 == 0 && p.out_head % 4 == 0 &&
                    ((uintptr_t)a & 15) == 0 && ((uintptr_t)p.w & 15) == 0 && ((uintptr_t)p.out & 7) == 0, "%s: an operand is not aligned", what);
    return 0;
}

extern "C" int hfa_latent_store(const float* down, int ld_down, const void* q, int q_dtype, int ldq, const float* w, float eps,
                                const int* positions, const float* inv_freq, int rot_dim, int pairing, void* q_out, int ld_out,
                                void* k_cache, void* v_cache, int dtype, const int* slot_map, int page_tokens, int n_tokens, int n_heads,
                                int dim, int rot, int latent, const void* fold, hipStream_t stream) {
    HFA_REQUIRE(down && q && w && q_out && k_cache && v_cache && slot_map && page_tokens > 0 && n_tokens > 0 && n_heads > 0 && dim >= 0 &&
                    rot >= 0 && latent > 0, "latent_store: bad arguments");
    HFA_REQUIRE(rot <= LATENT_MAX_ROT && rot_dim >= 0 && rot_dim % 2 == 0 && rot_dim <= rot && (rot_dim == 0 || (positions && inv_freq)) &&
                    (pairing == 0 || pairing == 1), "latent_store: a rotated part of %d (at most %d), %d of it turned", rot, LATENT_MAX_ROT, rot_dim);
    HFA_REQUIRE(ld_down >= latent + rot && ldq >= n_heads * (dim + rot) && ld_out >= n_heads * (rot + latent),
                "latent_store: a row is shorter than its parts");
    HFA_REQUIRE((q_dtype == HFA_F32 || q_dtype == HFA_BF16) && (dtype == HFA_F32 || dtype == HFA_BF16) && !(q_dtype == HFA_BF16 && dtype == HFA_F32),
                "latent_store: the queries are fp32 or of the cache's type");
    const LatentRow a = {down, ld_down, w, eps, positions, inv_freq, rot_dim, pairing, ld_out, slot_map, page_tokens, n_heads, dim, rot, latent};
    if (fold) {
        const HeadRows p = {ldq, dim + rot, (const uint16_t*)fold, (uint16_t*)q_out + rot, ld_out, rot + latent, nullptr, 0, n_tokens, latent, dim};
        HFA_REQUIRE(dtype == HFA_BF16, "latent_store: the fold is of the bf16 engine");
        const int rc = check_head_rows("latent_store", p, q, q_dtype, n_heads);
        if (rc) return rc;
        const long n_fold = (long)(latent / 32) * n_heads * ((n_tokens + 31) / 32);
        HFA_REQUIRE(n_fold + n_tokens < (1L << 31), "latent_store: the step exceeds the grid");
        const int blocks = (int)n_fold + n_tokens;
        if (q_dtype == HFA_F32)
            latent_fold_store_kernel<float><<<blocks, 4 * WAVE, 0, stream>>>(a, p, (const float*)q, ldq, (bf16*)q_out, (bf16*)k_cache, (bf16*)v_cache, (int)n_fold);
        else
            latent_fold_store_kernel<bf16><<<blocks, 4 * WAVE, 0, stream>>>(a, p, (const bf16*)q, ldq, (bf16*)q_out, (bf16*)k_cache, (bf16*)v_cache, (int)n_fold);
        HFA_LAUNCH_CHECK("latent_store");
        return 0;
    }
#define LS(TQ, T) latent_store_kernel<TQ, T><<<n_tokens, LATENT_THREADS, 0, stream>>>(a, (const TQ*)q, ldq, (T*)q_out, (T*)k_cache, (T*)v_cache)
    if (dtype == HFA_F32) LS(float, float);
    else if (q_dtype == HFA_BF16) LS(bf16, bf16);
    else LS(float, bf16);
#undef LS
    HFA_LAUNCH_CHECK("latent_store");
    return 0;
}

extern "C" int hfa_head_rows(const void* a, int a_dtype, int lda, int a_head, const void* w, void* out, int ldo, int out_head,
                             const float* gate, int ldg, int n_rows, int n_heads, int N, int K, hipStream_t stream) {
    const HeadRows p = {lda, a_head, (const uint16_t*)w, (uint16_t*)out, ldo, out_head, gate, ldg, n_rows, N, K};
    const int rc = check_head_rows("head_rows", p, a, a_dtype, n_heads);
    if (rc) return rc;
    dim3 grid(N / 32, n_heads, (n_rows + 31) / 32);
    if (a_dtype == HFA_F32) head_rows_kernel<float><<<grid, 4 * WAVE, 0, stream>>>(p, (const float*)a);
    else head_rows_kernel<bf16><<<grid, 4 * WAVE, 0, stream>>>(p, (const bf16*)a);
    HFA_LAUNCH_CHECK("head_rows");
    return 0;
}
