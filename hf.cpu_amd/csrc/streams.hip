// Residuals that are several streams side by side (hyper-connections): x is [token][stream][width], fp32. A sublayer reads one
// weighted sum of the streams, normed; its result y goes into every stream while the streams are mixed among themselves:
//
//   new_b = sum_a mix[a, b] old_a + out[b] y          u = sum_b in[b] new_b          n = u / sqrt(mean(u^2) + eps) * w
//
// One kernel does the end of a sublayer and the beginning of the next, so that the streams are read and written once a
// sublayer: hfa_stream_step takes the update that the sublayer before left undone (its result y, finished or as the partial
// sums of a product whose K was split), writes the new streams, and forms the next sublayer's normed input. Where every
// request brings one token, the causal convolution over the normed inputs that some designs put in front of a sublayer is
// done on the way too, from the request's state row.
//
//   hfa_stream_step    the above; parts of it can be left out (no update before the first sublayer but the copies of the
//                      embedding; no input after the last one)
//   hfa_stream_sum     out[r] = sum_b new_b of chosen rows, with an update that is still undone (nothing is written back)
#include "api.h"
#include "common.h"

#define STREAMS_MAX 32
#define STREAM_WIDTH_MAX 12288           // the sublayer's input lies in LDS until its norm is known
#define STREAM_TAPS_MAX 8
#define STREAM_PLANES 8                  // partial sums are fetched in batches of this many

template <int VW> struct Vec { float v[VW]; };
template <int VW> __device__ __forceinline__ Vec<VW> vload(const float* p) {
    Vec<VW> r;
    if constexpr (VW == 4) {
        const float4 f = *reinterpret_cast<const float4*>(p);
        r.v[0] = f.x; r.v[1] = f.y; r.v[2] = f.z; r.v[3] = f.w;
    } else {
        r.v[0] = *p;
    }
    return r;
}
template <int VW> __device__ __forceinline__ void vstore(float* p, const Vec<VW>& r) {
    if constexpr (VW == 4) *reinterpret_cast<float4*>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
    else *p = r.v[0];
}
template <int VW> __device__ __forceinline__ void vstore(bf16* p, const Vec<VW>& r) {
    if constexpr (VW == 4)
        *reinterpret_cast<uint2*>(p) = make_uint2((uint32_t)bf16_bits(r.v[0]) | ((uint32_t)bf16_bits(r.v[1]) << 16),
                                                  (uint32_t)bf16_bits(r.v[2]) | ((uint32_t)bf16_bits(r.v[3]) << 16));
    else *p = from_f32<bf16>(r.v[0]);
}

// The sublayer's result at row t, columns c .. c + VW - 1: stored, or the sum of `splits` partial sums in ascending order.
template <int VW>
__device__ __forceinline__ Vec<VW> branch_at(const float* __restrict__ y, int ldy, const float* __restrict__ partial, int splits, int n_rows,
                                             int width, int t, int c) {
    if (splits == 0) return vload<VW>(y + (size_t)t * ldy + c);
    Vec<VW> s;
#pragma unroll
    for (int e = 0; e < VW; e++) s.v[e] = 0.f;
    for (int s0 = 0; s0 < splits; s0 += STREAM_PLANES) {
        Vec<VW> p[STREAM_PLANES];
#pragma unroll
        for (int u = 0; u < STREAM_PLANES; u++) {
            if (s0 + u < splits) p[u] = vload<VW>(partial + ((size_t)(s0 + u) * n_rows + t) * width + c);
            else
#pragma unroll
                for (int e = 0; e < VW; e++) p[u].v[e] = 0.f;
        }
#pragma unroll
        for (int u = 0; u < STREAM_PLANES; u++)
#pragma unroll
            for (int e = 0; e < VW; e++) s.v[e] += p[u].v[e];
    }
    return s;
}

// The streams at row t, columns c ..: as stored (mode 0), all equal to y (mode 1), or updated (mode 2). NS: streams at compile
// time, 0: `S` of them. The weights' addresses are the same for every lane: they are read through the scalar unit.
template <int NS, int VW>
__device__ __forceinline__ void streams_at(Vec<VW>* nw, const float* __restrict__ x, int S, int width, int mode, const float* __restrict__ y,
                                           int ldy, const float* __restrict__ partial, int splits, int n_rows, const float* __restrict__ mix,
                                           const float* __restrict__ out_w, int t, int c) {
    constexpr int CAP = NS ? NS : STREAMS_MAX;
    const int n = NS ? NS : S;
    if (mode == 1) {
        const Vec<VW> b = branch_at<VW>(y, ldy, partial, splits, n_rows, width, t, c);
#pragma unroll
        for (int s = 0; s < CAP; s++)
            if (s < n) nw[s] = b;
        return;
    }
    Vec<VW> old[CAP];
#pragma unroll
    for (int s = 0; s < CAP; s++)
        if (s < n) old[s] = vload<VW>(x + ((size_t)t * n + s) * width + c);
    if (mode == 0) {
#pragma unroll
        for (int s = 0; s < CAP; s++)
            if (s < n) nw[s] = old[s];
        return;
    }
    const Vec<VW> b = branch_at<VW>(y, ldy, partial, splits, n_rows, width, t, c);
#pragma unroll
    for (int to = 0; to < CAP; to++) {
        if (to >= n) continue;
        Vec<VW> a;
#pragma unroll
        for (int e = 0; e < VW; e++) a.v[e] = out_w[to] * b.v[e];
#pragma unroll
        for (int from = 0; from < CAP; from++)
            if (from < n)
#pragma unroll
                for (int e = 0; e < VW; e++) a.v[e] = fmaf(mix[from * n + to], old[from].v[e], a.v[e]);
        nw[to] = a;
    }
}

// One block a token. ITEMS: groups of VW columns that a thread takes, held in registers between the two halves (and what the
// second half wants from memory is asked for in the first); 0: any number, with the input in LDS.
template <int NS, int VW, int ITEMS, typename TO>
__global__ __launch_bounds__(1024) void stream_step_kernel(
    float* __restrict__ x, int S, int width, int mode, const float* __restrict__ y, int ldy, const float* __restrict__ partial, int splits,
    const float* __restrict__ mix, const float* __restrict__ out_w, const float* __restrict__ in_w, const float* __restrict__ norm_w,
    float eps, TO* __restrict__ out, int ldo, const float* __restrict__ taps, int K, float* __restrict__ state, size_t state_ld,
    const int* __restrict__ slots, int n_rows) {
    constexpr int CAP = NS ? NS : STREAMS_MAX, KEEP = ITEMS ? ITEMS : 1;
    extern __shared__ float u_s[];
    __shared__ float red[17];
    const int t = blockIdx.x, n = NS ? NS : S, stride = blockDim.x * VW, c0 = threadIdx.x * VW;
    float* st = taps && K > 1 ? state + (size_t)slots[t] * state_ld : nullptr;
    Vec<VW> keep[KEEP], gain[KEEP], past[KEEP];               // the input, the norm's weight, the convolution's sum over earlier inputs
    Vec<VW> now[KEEP];                                        // the current token's taps
    float ss = 0.f;

    // new streams and the input at columns c ..
    auto first_half = [&](int c) {
        Vec<VW> nw[CAP], u;
        streams_at<NS, VW>(nw, x, S, width, mode, y, ldy, partial, splits, n_rows, mix, out_w, t, c);
#pragma unroll
        for (int e = 0; e < VW; e++) u.v[e] = 0.f;
#pragma unroll
        for (int s = 0; s < CAP; s++) {
            if (s >= n) continue;
            if (mode != 0) vstore<VW>(x + ((size_t)t * n + s) * width + c, nw[s]);
            if (in_w) {
                const float w = in_w[s];
#pragma unroll
                for (int e = 0; e < VW; e++) u.v[e] = fmaf(w, nw[s].v[e], u.v[e]);
            }
        }
#pragma unroll
        for (int e = 0; e < VW; e++) ss = fmaf(u.v[e], u.v[e], ss);
        return u;
    };
    // the request's only token of this step: the inputs before it are its state's, oldest first, which move up by one
    auto history = [&](int c) {
        Vec<VW> acc;
#pragma unroll
        for (int e = 0; e < VW; e++) acc.v[e] = 0.f;
#pragma unroll
        for (int j0 = 0; j0 < STREAM_TAPS_MAX - 1; j0 += 3) {
            if (j0 >= K - 1) continue;
            // three at a time, all asked for before the first is used (past the last one, the last one again)
            Vec<VW> p[3], w[3];
#pragma unroll
            for (int u = 0; u < 3; u++) {
                const int j = j0 + u < K - 1 ? j0 + u : K - 2;
                p[u] = vload<VW>(st + (size_t)j * width + c);
                w[u] = vload<VW>(taps + (size_t)j * width + c);
            }
#pragma unroll
            for (int u = 0; u < 3; u++) {
                if (j0 + u >= K - 1) continue;
#pragma unroll
                for (int e = 0; e < VW; e++) acc.v[e] = fmaf(w[u].v[e], p[u].v[e], acc.v[e]);
                if (j0 + u > 0) vstore<VW>(st + (size_t)(j0 + u - 1) * width + c, p[u]);
            }
        }
        return acc;
    };
    auto current = [&](int c) {
        return vload<VW>(taps + (size_t)(K - 1) * width + c);
    };
    auto finish = [&](int c, Vec<VW> v, float inv, const Vec<VW>& w, const Vec<VW>& acc, const Vec<VW>& tap) {
#pragma unroll
        for (int e = 0; e < VW; e++) v.v[e] = v.v[e] * inv * w.v[e];
        if (taps) {
            if (K > 1) vstore<VW>(st + (size_t)(K - 2) * width + c, v);
#pragma unroll
            for (int e = 0; e < VW; e++) v.v[e] = fmaf(tap.v[e], v.v[e], acc.v[e]);
        }
        vstore<VW>(out + (size_t)t * ldo + c, v);
    };

    if constexpr (ITEMS > 0) {
#pragma unroll
        for (int i = 0; i < ITEMS; i++) {
            const int c = c0 + i * stride;
            if (c >= width) continue;
            if (in_w) {
                gain[i] = vload<VW>(norm_w + c);
                if (taps) {
                    past[i] = history(c);
                    now[i] = current(c);
                }
            }
            keep[i] = first_half(c);
        }
    } else {
        for (int c = c0; c < width; c += stride) {
            const Vec<VW> u = first_half(c);
            if (in_w) vstore<VW>(u_s + c, u);
        }
    }
    if (!in_w) return;                                        // uniform
    // the sum of squares over the block, in a fixed order; one barrier
    ss = wave_sum(ss);
    if ((threadIdx.x & (WAVE - 1)) == 0) red[threadIdx.x / WAVE] = ss;
    __syncthreads();
    float total = 0.f;
    for (int i = 0; i < (int)(blockDim.x / WAVE); i++) total += red[i];
    const float inv = 1.0f / sqrtf(total / (float)width + eps);
    if constexpr (ITEMS > 0) {
#pragma unroll
        for (int i = 0; i < ITEMS; i++) {
            const int c = c0 + i * stride;
            if (c < width) finish(c, keep[i], inv, gain[i], past[i], now[i]);
        }
    } else {
        for (int c = c0; c < width; c += stride) {
            Vec<VW> acc, tap;
            if (taps) {
                acc = history(c);
                tap = current(c);
            }
            finish(c, vload<VW>(u_s + c), inv, vload<VW>(norm_w + c), acc, tap);
        }
    }
}

template <int NS, int VW>
__global__ __launch_bounds__(256) void stream_sum_kernel(const float* __restrict__ x, int S, int width, int mode, const float* __restrict__ y,
                                                        int ldy, const float* __restrict__ partial, int splits, const float* __restrict__ mix,
                                                        const float* __restrict__ out_w, const int* __restrict__ rows, float* __restrict__ out,
                                                        int n_rows) {
    constexpr int CAP = NS ? NS : STREAMS_MAX;
    const int n = NS ? NS : S, r = blockIdx.x, t = rows ? rows[r] : r;
    for (int c = threadIdx.x * VW; c < width; c += blockDim.x * VW) {
        Vec<VW> nw[CAP], sum;
        streams_at<NS, VW>(nw, x, S, width, mode, y, ldy, partial, splits, n_rows, mix, out_w, t, c);
#pragma unroll
        for (int e = 0; e < VW; e++) sum.v[e] = 0.f;
#pragma unroll
        for (int s = 0; s < CAP; s++)
            if (s < n)
#pragma unroll
                for (int e = 0; e < VW; e++) sum.v[e] += nw[s].v[e];
        vstore<VW>(out + (size_t)r * width + c, sum);
    }
}

static int check_update(const char* what, const float* x, int n_streams, int width, int mode, const float* y, int ldy, const float* partial,
                        int splits, const float* mix, const float* out_w, int n_rows) {
    HFA_REQUIRE(x && n_rows > 0 && width > 0 && width <= STREAM_WIDTH_MAX && n_streams > 0 && n_streams <= STREAMS_MAX,
                "%s: %d streams of %d values (at most %d of %d)", what, n_streams, width, STREAMS_MAX, STREAM_WIDTH_MAX);
    HFA_REQUIRE(mode >= 0 && mode <= 2 && splits >= 0, "%s: bad mode", what);
    HFA_REQUIRE(mode == 0 || (splits > 0 ? partial != nullptr : (y != nullptr && ldy >= width)), "%s: an update without a sublayer's result", what);
    HFA_REQUIRE(mode != 2 || (mix && out_w), "%s: an update without its weights", what);
    return 0;
}

static bool aligned16(const void* p) { return ((uintptr_t)p & 15) == 0; }

#define STREAM_COUNTS(GO)             \
    switch (n_streams) {              \
        case 1: GO(1); break;         \
        case 2: GO(2); break;         \
        case 3: GO(3); break;         \
        case 4: GO(4); break;         \
        case 5: GO(5); break;         \
        case 6: GO(6); break;         \
        case 7: GO(7); break;         \
        case 8: GO(8); break;         \
        default: GO(0); break;        \
    }

extern "C" int hfa_stream_step(float* x, int n_streams, int width, int mode, const float* y, int ldy, const float* partial, int splits,
                               const float* mix, const float* out_w, const float* in_w, const float* norm_w, float eps, void* out,
                               int out_dtype, int ldo, const float* taps, int n_taps, float* state, size_t state_ld, const int* slots,
                               int n_rows, hipStream_t stream) {
    const int rc = check_update("stream_step", x, n_streams, width, mode, y, ldy, partial, splits, mix, out_w, n_rows);
    if (rc) return rc;
    HFA_REQUIRE(in_w || mode != 0, "stream_step: nothing to do");
    HFA_REQUIRE(!in_w || (norm_w && out && ldo >= width && (out_dtype == HFA_F32 || out_dtype == HFA_BF16)), "stream_step: no place for the input");
    HFA_REQUIRE(!taps || (in_w && n_taps >= 1 && n_taps <= STREAM_TAPS_MAX && (n_taps == 1 || (state && slots && state_ld >= (size_t)(n_taps - 1) * width))),
                "stream_step: a convolution over 1 to %d inputs with the state of its earlier ones", STREAM_TAPS_MAX);
    const bool vec = width % 4 == 0 && aligned16(x) && (mode == 0 || (splits > 0 ? aligned16(partial) : aligned16(y) && ldy % 4 == 0)) &&
                     (!in_w || (aligned16(norm_w) && aligned16(out) && ldo % 4 == 0)) &&
                     (!taps || (aligned16(taps) && (n_taps == 1 || (aligned16(state) && state_ld % 4 == 0))));
    // few tokens: a block takes its token's row at once; many: two groups of columns a thread
    const int groups = (width + (vec ? 3 : 0)) / (vec ? 4 : 1);
    const bool few = n_rows < 256 && groups <= 1024;
    int threads = ((few ? groups : (groups + 1) / 2) + 63) / 64 * 64;
    const bool two = threads <= 1024;
    if (!two) threads = 256;
    const size_t lds = in_w && !few && !two ? (size_t)((width + 3) / 4 * 4) * sizeof(float) : 0;
#define STEP_GO4(NS, VW, ITEMS, TO)                                                                                                  \
    stream_step_kernel<NS, VW, ITEMS, TO><<<n_rows, threads, lds, stream>>>(x, n_streams, width, mode, y, ldy, partial, splits, mix, out_w, \
                                                                           in_w, norm_w, eps, (TO*)out, ldo, taps, n_taps, state, state_ld,  \
                                                                           slots, n_rows)
#define STEP_GO3(NS, VW, TO)                          \
    do {                                              \
        if (few) STEP_GO4(NS, VW, 1, TO);             \
        else if (two) STEP_GO4(NS, VW, 2, TO);        \
        else STEP_GO4(NS, VW, 0, TO);                 \
    } while (0)
#define STEP_GO(NS)                                                                 \
    do {                                                                            \
        if (in_w && out_dtype == HFA_BF16) {                                        \
            if (vec) STEP_GO3(NS, 4, bf16); else STEP_GO3(NS, 1, bf16);             \
        } else {                                                                    \
            if (vec) STEP_GO3(NS, 4, float); else STEP_GO3(NS, 1, float);           \
        }                                                                           \
    } while (0)
    STREAM_COUNTS(STEP_GO)
#undef STEP_GO
#undef STEP_GO3
#undef STEP_GO4
    HFA_LAUNCH_CHECK("stream_step");
    return 0;
}

extern "C" int hfa_stream_sum(const float* x, int n_streams, int width, int mode, const float* y, int ldy, const float* partial, int splits,
                              const float* mix, const float* out_w, const int* rows, float* out, int n_out, int n_rows, hipStream_t stream) {
    const int rc = check_update("stream_sum", x, n_streams, width, mode, y, ldy, partial, splits, mix, out_w, n_rows);
    if (rc) return rc;
    HFA_REQUIRE(out && n_out > 0 && (rows || n_out == n_rows), "stream_sum: without row indices every row is summed");
    const bool vec = width % 4 == 0 && aligned16(x) && aligned16(out) &&
                     (mode == 0 || (splits > 0 ? aligned16(partial) : aligned16(y) && ldy % 4 == 0));
#define SUM_GO2(NS, VW) stream_sum_kernel<NS, VW><<<n_out, 256, 0, stream>>>(x, n_streams, width, mode, y, ldy, partial, splits, mix, out_w, rows, out, n_rows)
#define SUM_GO(NS)                                \
    do {                                          \
        if (vec) SUM_GO2(NS, 4); else SUM_GO2(NS, 1); \
    } while (0)
    STREAM_COUNTS(SUM_GO)
#undef SUM_GO
#undef SUM_GO2
    HFA_LAUNCH_CHECK("stream_sum");
    return 0;
}
