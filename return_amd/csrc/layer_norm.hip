// Layer norms of 32-bit stream rows, behind a sublayer and in front of one, and what goes with such models:
//   layer_norm_add     h[r] += (y[r] - mean) / sqrt(mean((y[r] - mean)^2) + eps) * w in 32-bit; x[r] (null: not wanted) is
//                      the new h[r] in the storage type, what the next sublayer's first product reads. The normed y never
//                      leaves 32-bit.
//   stream_layer_norm  h[r] += a[r] + sum_k wb[r][k] b[r][k] + extra[r] * sigmoid(logit[r]) in 32-bit (each term may be
//                      missing; wb null: factors of one), then x[r] = norm(h[r]) w + bias in the storage type. With a list
//                      of rows the sum is formed for those rows only and h stays as it is: x[i] belongs to row rows[i].
//   stream_rows        x[r] = h[r] in the storage type
//   softcap            z <- c tanh(z / c) in place, 32-bit
// A workgroup takes a row; the row's elements stay in registers between the mean, the sum of squared deviations and the
// result (up to LN_G groups of four neighbours a thread; other rows are read again, element by element). Every read of
// the row is asked for before the first sum.
#include "common.h"
#include <algorithm>

#define LN_THREADS 256
#define LN_G 4

__device__ __forceinline__ void ln_load4(const float* p, float (&v)[4]) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
}
__device__ __forceinline__ void ln_load4(const bf16* p, float (&v)[4]) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
    v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
}
__device__ __forceinline__ void ln_store4(float* p, const float (&v)[4]) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ void ln_store4(bf16* p, const float (&v)[4]) {
    uint2 t;
    t.x = (uint32_t)f2bf_bits(v[0]) | ((uint32_t)f2bf_bits(v[1]) << 16);
    t.y = (uint32_t)f2bf_bits(v[2]) | ((uint32_t)f2bf_bits(v[3]) << 16);
    *reinterpret_cast<uint2*>(p) = t;
}

// VEC: H is a multiple of four up to 4 * LN_G * LN_THREADS and everything is aligned to four elements.
template <typename T, bool VEC>
__global__ __launch_bounds__(LN_THREADS) void layer_norm_add_kernel(const T* __restrict__ y, float* __restrict__ h,
                                                                    const float* __restrict__ w, float eps,
                                                                    T* __restrict__ x, int H) {
    __shared__ float scratch[16];
    const size_t r = blockIdx.x;
    const T* yr = y + r * H;
    float* hr = h + r * H;
    T* xr = x != nullptr ? x + r * H : nullptr;
    if constexpr (VEC) {
        float v[LN_G][4], hv[LN_G][4], wv[LN_G][4];
        float sum = 0.f;
#pragma unroll
        for (int g = 0; g < LN_G; ++g) {
            const int c = (threadIdx.x + g * LN_THREADS) * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[g][e] = hv[g][e] = wv[g][e] = 0.f;
            if (c < H) {
                ln_load4(yr + c, v[g]);
                ln_load4(hr + c, hv[g]);
                ln_load4(w + c, wv[g]);
            }
        }
#pragma unroll
        for (int g = 0; g < LN_G; ++g) sum += (v[g][0] + v[g][1]) + (v[g][2] + v[g][3]);
        const float mean = block_sum(sum, scratch) / (float)H;
        float ss = 0.f;
#pragma unroll
        for (int g = 0; g < LN_G; ++g) {
            const bool in = (threadIdx.x + g * LN_THREADS) * 4 < H;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                v[g][e] = in ? v[g][e] - mean : 0.f;
                ss = fmaf(v[g][e], v[g][e], ss);
            }
        }
        const float rstd = 1.0f / sqrtf(block_sum(ss, scratch) / (float)H + eps);
#pragma unroll
        for (int g = 0; g < LN_G; ++g) {
            const int c = (threadIdx.x + g * LN_THREADS) * 4;
            if (c < H) {
#pragma unroll
                for (int e = 0; e < 4; ++e) v[g][e] = hv[g][e] + v[g][e] * rstd * wv[g][e];
                ln_store4(hr + c, v[g]);
                if (xr != nullptr) ln_store4(xr + c, v[g]);
            }
        }
    } else {
        float sum = 0.f;
        for (int c = threadIdx.x; c < H; c += LN_THREADS) sum += to_f(yr[c]);
        const float mean = block_sum(sum, scratch) / (float)H;
        float ss = 0.f;
        for (int c = threadIdx.x; c < H; c += LN_THREADS) {
            const float d = to_f(yr[c]) - mean;
            ss = fmaf(d, d, ss);
        }
        const float rstd = 1.0f / sqrtf(block_sum(ss, scratch) / (float)H + eps);
        for (int c = threadIdx.x; c < H; c += LN_THREADS) {
            const float v = hr[c] + (to_f(yr[c]) - mean) * rstd * w[c];
            hr[c] = v;
            if (xr != nullptr) xr[c] = from_f<T>(v);
        }
    }
}

// What enters the stream in front of a norm (each pointer may be null).
template <typename T>
struct LnTerms {
    const T* a;                 // [R][H]
    const T* b;                 // [R][nb][H]: nb rows a stream row, in their order
    int nb;
    const float* wb;            // [R][nb]
    const T* extra;             // [R][H]
    const float* logit;         // one number a row, ld_logit elements apart
    long long ld_logit;
};

// a + sum_k wb b_k + extra * gate for element c of row r (the same order whatever the form)
template <typename T>
__device__ __forceinline__ float ln_terms(const LnTerms<T>& d, size_t r, int H, int c, float gate) {
    float v = d.a != nullptr ? to_f(d.a[r * H + c]) : 0.f;
    if (d.b != nullptr) {
        float s = 0.f;
        for (int k = 0; k < d.nb; ++k)
            s = fmaf(d.wb != nullptr ? d.wb[r * d.nb + k] : 1.0f, to_f(d.b[(r * d.nb + k) * H + c]), s);
        if (d.extra != nullptr) s = fmaf(to_f(d.extra[r * H + c]), gate, s);
        v += s;
    }
    return v;
}

// G > 0: groups of four neighbours a thread (H a multiple of four, at most 4 G threads); G 0: element by element
template <typename T, int G>
__global__ __launch_bounds__(1024) void stream_layer_norm_kernel(float* __restrict__ h, const int* __restrict__ rows,
                                                                 const LnTerms<T> d, const float* __restrict__ w,
                                                                 const float* __restrict__ bias, float eps,
                                                                 T* __restrict__ x, int H) {
    __shared__ float scratch[16];
    const int nt = blockDim.x;
    const size_t r = rows != nullptr ? (size_t)rows[blockIdx.x] : (size_t)blockIdx.x;
    float* hr = h + r * H;
    T* xr = x + (size_t)blockIdx.x * H;
    const bool adds = d.a != nullptr || d.b != nullptr;
    const bool keep = adds && rows == nullptr;
    const float gate = d.extra != nullptr ? 1.0f / (1.0f + expf(-d.logit[r * d.ld_logit])) : 0.f;
    if constexpr (G > 0) {
        float v[G][4], av[G][4], sv[G][4], ev[G][4], wv[G][4], bv[G][4];
#pragma unroll
        for (int g = 0; g < G; ++g) {
            const int c = (threadIdx.x + g * nt) * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[g][e] = av[g][e] = sv[g][e] = ev[g][e] = wv[g][e] = bv[g][e] = 0.f;
            if (c < H) {
                ln_load4(hr + c, v[g]);
                if (d.a != nullptr) ln_load4(d.a + r * H + c, av[g]);
                if (d.extra != nullptr) ln_load4(d.extra + r * H + c, ev[g]);
                ln_load4(w + c, wv[g]);
                if (bias != nullptr) ln_load4(bias + c, bv[g]);
            }
        }
        if (d.b != nullptr) {
            // several rows at a time, all their reads asked for before the first sum (a row beyond the last counts nothing)
            constexpr int KU = 4 / G;
            for (int k0 = 0; k0 < d.nb; k0 += KU) {
                float t[KU][G][4], f[KU];
#pragma unroll
                for (int u = 0; u < KU; ++u) {
                    const int k = min(k0 + u, d.nb - 1);
                    f[u] = k0 + u >= d.nb ? 0.f : d.wb != nullptr ? d.wb[r * d.nb + k] : 1.0f;
#pragma unroll
                    for (int g = 0; g < G; ++g) {
                        const int c = (threadIdx.x + g * nt) * 4;
                        t[u][g][0] = t[u][g][1] = t[u][g][2] = t[u][g][3] = 0.f;
                        if (c < H && k0 + u < d.nb) ln_load4(d.b + (r * d.nb + k) * H + c, t[u][g]);
                    }
                }
#pragma unroll
                for (int u = 0; u < KU; ++u)
#pragma unroll
                    for (int g = 0; g < G; ++g)
#pragma unroll
                        for (int e = 0; e < 4; ++e) sv[g][e] = fmaf(f[u], t[u][g][e], sv[g][e]);
            }
        }
        float sum = 0.f;
#pragma unroll
        for (int g = 0; g < G; ++g) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                if (d.extra != nullptr) sv[g][e] = fmaf(ev[g][e], gate, sv[g][e]);
                v[g][e] += av[g][e] + sv[g][e];
            }
            sum += (v[g][0] + v[g][1]) + (v[g][2] + v[g][3]);
        }
        if (keep) {
#pragma unroll
            for (int g = 0; g < G; ++g) {
                const int c = (threadIdx.x + g * nt) * 4;
                if (c < H) ln_store4(hr + c, v[g]);
            }
        }
        const float mean = block_sum(sum, scratch) / (float)H;
        float ss = 0.f;
#pragma unroll
        for (int g = 0; g < G; ++g) {
            const bool in = (threadIdx.x + g * nt) * 4 < H;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                v[g][e] = in ? v[g][e] - mean : 0.f;
                ss = fmaf(v[g][e], v[g][e], ss);
            }
        }
        const float rstd = 1.0f / sqrtf(block_sum(ss, scratch) / (float)H + eps);
#pragma unroll
        for (int g = 0; g < G; ++g) {
            const int c = (threadIdx.x + g * nt) * 4;
            if (c < H) {
#pragma unroll
                for (int e = 0; e < 4; ++e) v[g][e] = fmaf(v[g][e] * rstd, wv[g][e], bv[g][e]);
                ln_store4(xr + c, v[g]);
            }
        }
    } else {
        // the sums are formed again in every pass where the row is not kept (rows wanted alone)
        auto value = [&](int c) { return hr[c] + (adds ? ln_terms(d, r, H, c, gate) : 0.f); };
        float sum = 0.f;
        for (int c = threadIdx.x; c < H; c += nt) {
            const float v = value(c);
            if (keep) hr[c] = v;
            sum += v;
        }
        auto again = [&](int c) { return keep ? hr[c] : value(c); };      // (the thread's own store)
        const float mean = block_sum(sum, scratch) / (float)H;
        float ss = 0.f;
        for (int c = threadIdx.x; c < H; c += nt) {
            const float t = again(c) - mean;
            ss = fmaf(t, t, ss);
        }
        const float rstd = 1.0f / sqrtf(block_sum(ss, scratch) / (float)H + eps);
        for (int c = threadIdx.x; c < H; c += nt)
            xr[c] = from_f<T>(fmaf((again(c) - mean) * rstd, w[c], bias != nullptr ? bias[c] : 0.f));
    }
}

static bool ln_vec_ok(int H, const void* p0, const void* p1, const void* p2, const void* p3) {
    auto al = [](const void* p) { return p == nullptr || ((uintptr_t)p & 15) == 0; };
    return H % 4 == 0 && H <= 4 * LN_G * LN_THREADS && al(p0) && al(p1) && al(p2) && al(p3);
}

extern "C" int ra_layer_norm_add(float* h, const void* y, const float* w, float eps, void* x, int rows, int H, int dtype,
                                 void* stream) {
    if (rows <= 0) return RA_OK;
    if (H < 1 || h == nullptr || y == nullptr || w == nullptr) return RA_ERR_ARG;
    hipStream_t st = (hipStream_t)stream;
    const bool vec = ln_vec_ok(H, h, y, w, x);
#define LN_ADD(T_, V_)                                                                                               \
    hipLaunchKernelGGL((layer_norm_add_kernel<T_, V_>), dim3(rows), dim3(LN_THREADS), 0, st, (const T_*)y, h, w, eps, \
                       (T_*)x, H)
    if (dtype == RA_DTYPE_F32) {
        if (vec) LN_ADD(float, true); else LN_ADD(float, false);
    } else if (dtype == RA_DTYPE_BF16) {
        if (vec) LN_ADD(bf16, true); else LN_ADD(bf16, false);
    } else {
        return RA_ERR_ARG;
    }
#undef LN_ADD
    return ra_launch_status();
}

// a [R][H]; b [R][nb][H] with factors wb [R][nb] (null: one); extra [R][H] with logit (32-bit, ld_logit apart): each may
// be null (extra only beside b). row_ids (null: all rows, and the stream is updated) lists the rows wanted.
extern "C" int ra_stream_layer_norm(float* h, const void* a, const void* b, int nb, const float* wb, const void* extra,
                                    const float* logit, long long ld_logit, const float* w, const float* bias, float eps,
                                    void* out, const int* row_ids, int rows, int H, int dtype, void* stream) {
    if (rows <= 0) return RA_OK;
    if (H < 1 || h == nullptr || w == nullptr || out == nullptr || (b != nullptr && nb < 1) || (wb != nullptr && b == nullptr) ||
        (extra == nullptr) != (logit == nullptr) || (extra != nullptr && (b == nullptr || ld_logit < 1)))
        return RA_ERR_ARG;
    hipStream_t st = (hipStream_t)stream;
    auto al = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    const bool vec = H % 4 == 0 && H <= 16 * 1024 && al(h) && al(a) && al(b) && al(extra) && al(w) && al(bias) && al(out);
    // few rows: one group of four neighbours a thread, so that all of a row is on its way at once; many rows: 256 threads
    // with as many groups as the row has; rows beyond 4,096 elements: four groups a thread
    const int groups = rows <= 256 && H <= 4096 ? 1 : H <= 1024 ? 1 : H <= 2048 ? 2 : 4;
    const int threads = groups == 4 ? (H <= 4096 ? 256 : H <= 8192 ? 512 : 1024) : std::max(64, (H / (4 * groups) + 63) / 64 * 64);
#define LN_STREAM(T_, G_)                                                                                             \
    do {                                                                                                              \
        const LnTerms<T_> d = {(const T_*)a, (const T_*)b, nb, wb, (const T_*)extra, logit, ld_logit};                \
        hipLaunchKernelGGL((stream_layer_norm_kernel<T_, G_>), dim3(rows), dim3(threads), 0, st, h, row_ids, d, w, bias, eps, \
                           (T_*)out, H);                                                                              \
    } while (0)
    if (dtype == RA_DTYPE_F32) {
        if (!vec) LN_STREAM(float, 0); else if (groups == 1) LN_STREAM(float, 1); else if (groups == 2) LN_STREAM(float, 2);
        else LN_STREAM(float, 4);
    } else if (dtype == RA_DTYPE_BF16) {
        if (!vec) LN_STREAM(bf16, 0); else if (groups == 1) LN_STREAM(bf16, 1); else if (groups == 2) LN_STREAM(bf16, 2);
        else LN_STREAM(bf16, 4);
    } else {
        return RA_ERR_ARG;
    }
#undef LN_STREAM
    return ra_launch_status();
}

template <typename T>
__global__ void stream_rows_kernel(const float* __restrict__ h, T* __restrict__ x, size_t n) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x)
        x[i] = from_f<T>(h[i]);
}

extern "C" int ra_stream_rows(const float* h, void* x, long long n, int dtype, void* stream) {
    if (n <= 0) return RA_OK;
    const unsigned blocks = (unsigned)std::min<long long>((n + 255) / 256, 65535LL * 16);
    hipStream_t st = (hipStream_t)stream;
    if (dtype == RA_DTYPE_F32)
        hipLaunchKernelGGL(stream_rows_kernel<float>, dim3(blocks), dim3(256), 0, st, h, (float*)x, (size_t)n);
    else if (dtype == RA_DTYPE_BF16)
        hipLaunchKernelGGL(stream_rows_kernel<bf16>, dim3(blocks), dim3(256), 0, st, h, (bf16*)x, (size_t)n);
    else
        return RA_ERR_ARG;
    return ra_launch_status();
}

__global__ void softcap_kernel(float* __restrict__ z, float cap, size_t n) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x)
        z[i] = cap * tanhf(z[i] / cap);
}

extern "C" int ra_softcap(float* z, float cap, long long n, void* stream) {
    if (n <= 0) return RA_OK;
    if (!(cap > 0.f)) return RA_ERR_ARG;
    const unsigned blocks = (unsigned)std::min<long long>((n + 255) / 256, 65535LL * 16);
    hipLaunchKernelGGL(softcap_kernel, dim3(blocks), dim3(256), 0, (hipStream_t)stream, z, cap, (size_t)n);
    return ra_launch_status();
}
