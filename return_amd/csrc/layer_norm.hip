// Row kernels of a layer whose sublayers read the residual stream as it is and enter it through a layer norm of their
// output, and what goes with such a model:
//   layer_norm_add   h[r] += (y[r] - mean) / sqrt(mean((y[r] - mean)^2) + eps) * w in 32-bit; x[r] (null: not wanted) is
//                    the new h[r] in the storage type, what the next sublayer's first product reads. The normed y never
//                    leaves 32-bit.
//   layer_norm_rows  out[i] = the same norm of h[rows[i]] (rows null: of h[i])
//   stream_rows      x[r] = h[r] in the storage type
//   softcap          z <- c tanh(z / c) in place, 32-bit
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

// ADD: h[r] += norm(y[r]) w, x[r] = h[r]; else x[r] = norm(y[rows[r]]) w with y the 32-bit stream.
// VEC: H is a multiple of four up to 4 * LN_G * LN_THREADS and everything is aligned to four elements.
template <typename Y, typename T, bool ADD, bool VEC>
__global__ __launch_bounds__(LN_THREADS) void layer_norm_kernel(const Y* __restrict__ y, const int* __restrict__ rows,
                                                                float* __restrict__ h, const float* __restrict__ w,
                                                                float eps, T* __restrict__ x, int H) {
    __shared__ float scratch[16];
    const size_t r = blockIdx.x;
    const Y* yr = y + (rows != nullptr ? (size_t)rows[r] : r) * H;
    float* hr = ADD ? h + r * H : nullptr;
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
                if (ADD) ln_load4(hr + c, hv[g]);
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
                if (ADD) ln_store4(hr + c, v[g]);
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
            float v = (to_f(yr[c]) - mean) * rstd * w[c];
            if (ADD) {
                v += hr[c];
                hr[c] = v;
            }
            if (xr != nullptr) xr[c] = from_f<T>(v);
        }
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
    hipLaunchKernelGGL((layer_norm_kernel<T_, T_, true, V_>), dim3(rows), dim3(LN_THREADS), 0, st, (const T_*)y,     \
                       (const int*)nullptr, h, w, eps, (T_*)x, H)
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

extern "C" int ra_layer_norm_rows(const float* h, const float* w, float eps, void* out, const int* row_ids, int rows, int H,
                                  int dtype, void* stream) {
    if (rows <= 0) return RA_OK;
    if (H < 1 || h == nullptr || w == nullptr || out == nullptr) return RA_ERR_ARG;
    hipStream_t st = (hipStream_t)stream;
    const bool vec = ln_vec_ok(H, h, w, out, nullptr);
#define LN_ROWS(T_, V_)                                                                                              \
    hipLaunchKernelGGL((layer_norm_kernel<float, T_, false, V_>), dim3(rows), dim3(LN_THREADS), 0, st, h, row_ids,   \
                       (float*)nullptr, w, eps, (T_*)out, H)
    if (dtype == RA_DTYPE_F32) {
        if (vec) LN_ROWS(float, true); else LN_ROWS(float, false);
    } else if (dtype == RA_DTYPE_BF16) {
        if (vec) LN_ROWS(bf16, true); else LN_ROWS(bf16, false);
    } else {
        return RA_ERR_ARG;
    }
#undef LN_ROWS
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
