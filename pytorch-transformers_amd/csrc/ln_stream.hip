// LayerNorm (mean, biased variance, weight and bias), or an RMS norm (no mean, no bias: v / sqrt(mean(v^2) + eps) * w), around
// a residual stream that is held in 32-bit whatever the model's compute type.  One launch does what stands between two sublayers of a block that norms a sublayer's
// output as well as its input:
//
//   s = x                                  the stream (32-bit), if given
//   s += mult * (LN(y) * wy + by)          a sublayer's output y (compute type) normed, scaled and added, if given
//   s += add                               another 32-bit tensor of the stream's shape (rows of its own), if given
//   s += vec                               one 32-bit vector for every row, if given
//   out_wide = s                           if wanted
//   out_narrow = LN(s) * w + b             in the compute type, if w is given; without w, s itself in the compute type
//
// `rows` gathers: output row m is made of input row rows[m] (the final norm on the wanted rows alone).
// One workgroup per row; a thread keeps its VPT elements in registers over all passes; every sum over a row is taken
// in 32-bit in an order that depends on the row's length alone.
#include "common.h"
#include "pta_kernels.h"

template <typename T, int VPT>
__global__ __launch_bounds__(256) void layernorm_stream_kernel(T* __restrict__ out_narrow, float* __restrict__ out_wide,
                                                               const float* __restrict__ x, const T* __restrict__ y, long y_ld,
                                                               const float* __restrict__ wy, const float* __restrict__ by,
                                                               float mult, const float* __restrict__ add,
                                                               const float* __restrict__ vec, const int* __restrict__ rows,
                                                               const float* __restrict__ w, const float* __restrict__ b,
                                                               float eps, int H) {
    __shared__ float red[16];
    const int m = blockIdx.x;
    const long src = rows ? rows[m] : m;
    const float inv_h = 1.0f / (float)H;
    float s[VPT], yv[VPT];
#pragma unroll
    for (int k = 0; k < VPT; ++k) {  // every load of the first pass asked for at once
        const int i = threadIdx.x + k * blockDim.x;
        s[k] = (x && i < H) ? x[src * H + i] : 0.f;
        yv[k] = (y && i < H) ? Io<T>::ld(y + src * y_ld + i) : 0.f;
    }
    if (y) {
        float wv[VPT], bv[VPT];
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            wv[k] = i < H ? wy[i] : 0.f;
            bv[k] = i < H ? by[i] : 0.f;
        }
        float t = 0.f;
#pragma unroll
        for (int k = 0; k < VPT; ++k) t += yv[k];
        const float mean = block_sum(t, red) * inv_h;
        t = 0.f;
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            const float dlt = i < H ? yv[k] - mean : 0.f;
            t += dlt * dlt;
        }
        const float inv = 1.0f / sqrtf(block_sum(t, red) * inv_h + eps);
#pragma unroll
        for (int k = 0; k < VPT; ++k) s[k] += mult * ((yv[k] - mean) * inv * wv[k] + bv[k]);
    }
    if (add) {
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            if (i < H) s[k] += add[src * H + i];
        }
    }
    if (vec) {
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            if (i < H) s[k] += vec[i];
        }
    }
    if (out_wide) {
#pragma unroll
        for (int k = 0; k < VPT; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            if (i < H) out_wide[(long)m * H + i] = s[k];
        }
    }
    if (!w) {
        if (out_narrow) {
#pragma unroll
            for (int k = 0; k < VPT; ++k) {
                const int i = threadIdx.x + k * blockDim.x;
                if (i < H) Io<T>::st(out_narrow + (long)m * H + i, s[k]);
            }
        }
        return;
    }
    float wv[VPT], bv[VPT];
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = threadIdx.x + k * blockDim.x;
        wv[k] = i < H ? w[i] : 0.f;
        bv[k] = i < H ? b[i] : 0.f;
    }
    float t = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = threadIdx.x + k * blockDim.x;
        t += i < H ? s[k] : 0.f;
    }
    const float mean = block_sum(t, red) * inv_h;
    t = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = threadIdx.x + k * blockDim.x;
        const float dlt = i < H ? s[k] - mean : 0.f;
        t += dlt * dlt;
    }
    const float inv = 1.0f / sqrtf(block_sum(t, red) * inv_h + eps);
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = threadIdx.x + k * blockDim.x;
        if (i < H) Io<T>::st(out_narrow + (long)m * H + i, (s[k] - mean) * inv * wv[k] + bv[k]);
    }
}

// The same with RMS norms in place of LN.  A thread holds its V neighbouring elements (four where rows and pointers allow it)
// VPT times over.
template <typename T, int V>
__device__ __forceinline__ void stream_load(const T* p, float (&v)[V]) {
    if constexpr (V == 4 && sizeof(T) == 4) {
        const float4 f = *reinterpret_cast<const float4*>(p);
        v[0] = f.x; v[1] = f.y; v[2] = f.z; v[3] = f.w;
    } else if constexpr (V == 4) {
        const uint2 u = *reinterpret_cast<const uint2*>(p);
        v[0] = bf16_bits_to_f32((bf16_t)(u.x & 0xffffu)); v[1] = bf16_bits_to_f32((bf16_t)(u.x >> 16));
        v[2] = bf16_bits_to_f32((bf16_t)(u.y & 0xffffu)); v[3] = bf16_bits_to_f32((bf16_t)(u.y >> 16));
    } else {
        v[0] = Io<T>::ld(p);
    }
}

template <typename T, int V>
__device__ __forceinline__ void stream_store(T* p, const float (&v)[V]) {
    if constexpr (V == 4 && sizeof(T) == 4) {
        *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    } else if constexpr (V == 4) {
        *reinterpret_cast<uint2*>(p) = make_uint2((uint32_t)f32_to_bf16_bits(v[0]) | ((uint32_t)f32_to_bf16_bits(v[1]) << 16),
                                                  (uint32_t)f32_to_bf16_bits(v[2]) | ((uint32_t)f32_to_bf16_bits(v[3]) << 16));
    } else {
        Io<T>::st(p, v[0]);
    }
}

template <typename T, int VPT, int V>
__global__ __launch_bounds__(256) void rmsnorm_stream_kernel(T* __restrict__ out_narrow, float* __restrict__ out_wide,
                                                             const float* __restrict__ x, const T* __restrict__ y, long y_ld,
                                                             const float* __restrict__ wy, float mult,
                                                             const float* __restrict__ add, const float* __restrict__ vec,
                                                             const int* __restrict__ rows, const float* __restrict__ w, float eps,
                                                             int H) {
    __shared__ float red[16];
    const int m = blockIdx.x;
    const long src = rows ? rows[m] : m;
    const float inv_h = 1.0f / (float)H;
    float s[VPT][V], yv[VPT][V], wv[VPT][V];
#pragma unroll
    for (int k = 0; k < VPT; ++k) {  // every load of the first pass asked for at once
        const int i = (threadIdx.x + k * blockDim.x) * V;
#pragma unroll
        for (int e = 0; e < V; ++e) s[k][e] = 0.f, yv[k][e] = 0.f, wv[k][e] = 0.f;
        if (i >= H) continue;
        if (x) stream_load<float, V>(x + src * H + i, s[k]);
        if (y) {
            stream_load<T, V>(y + src * y_ld + i, yv[k]);
            stream_load<float, V>(wy + i, wv[k]);
        }
    }
    if (y) {
        float t = 0.f;
#pragma unroll
        for (int k = 0; k < VPT; ++k)
#pragma unroll
            for (int e = 0; e < V; ++e) t += yv[k][e] * yv[k][e];
        const float by = mult / sqrtf(block_sum(t, red) * inv_h + eps);
#pragma unroll
        for (int k = 0; k < VPT; ++k)
#pragma unroll
            for (int e = 0; e < V; ++e) s[k][e] += yv[k][e] * by * wv[k][e];
    }
    float t = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * blockDim.x) * V;
        if (i >= H) continue;
        float a[V];
        if (add) {
            stream_load<float, V>(add + src * H + i, a);
#pragma unroll
            for (int e = 0; e < V; ++e) s[k][e] += a[e];
        }
        if (vec) {
            stream_load<float, V>(vec + i, a);
#pragma unroll
            for (int e = 0; e < V; ++e) s[k][e] += a[e];
        }
        if (out_wide) stream_store<float, V>(out_wide + (long)m * H + i, s[k]);
        if (w) stream_load<float, V>(w + i, wv[k]);
        else if (out_narrow) stream_store<T, V>(out_narrow + (long)m * H + i, s[k]);
#pragma unroll
        for (int e = 0; e < V; ++e) t += s[k][e] * s[k][e];
    }
    if (!w) return;
    const float inv = 1.0f / sqrtf(block_sum(t, red) * inv_h + eps);
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = (threadIdx.x + k * blockDim.x) * V;
        if (i >= H) continue;
#pragma unroll
        for (int e = 0; e < V; ++e) s[k][e] = s[k][e] * inv * wv[k][e];
        stream_store<T, V>(out_narrow + (long)m * H + i, s[k]);
    }
}

template <typename T>
static int launch_rms_stream(void* out_narrow, float* out_wide, const float* x, const void* y, long y_ld, const float* wy,
                             float mult, const float* add, const float* vec, const int* rows, const float* w, float eps, int M,
                             int H, hipStream_t s) {
    // four elements a load wherever a model's rows lie so; which it is follows from the row's length and the pointers, not
    // from the number of rows
    uintptr_t at = (uintptr_t)out_narrow | (uintptr_t)out_wide | (uintptr_t)x | (uintptr_t)y | (uintptr_t)wy | (uintptr_t)add |
                   (uintptr_t)vec | (uintptr_t)w;
    const bool four = H % 4 == 0 && y_ld % 4 == 0 && at % 16 == 0;
    const int n = four ? H / 4 : H;
    const int threads = n <= 64 ? 64 : n <= 128 ? 128 : 256;
    const int vpt = (n + threads - 1) / threads;
#define PTA_RMS_STREAM(VPT_, V_)                                                                                            \
    hipLaunchKernelGGL((rmsnorm_stream_kernel<T, VPT_, V_>), dim3(M), dim3(threads), 0, s, (T*)out_narrow, out_wide, x,       \
                       (const T*)y, y_ld, wy, mult, add, vec, rows, w, eps, H)
    if (four) {
        if (vpt <= 1) PTA_RMS_STREAM(1, 4);
        else if (vpt <= 2) PTA_RMS_STREAM(2, 4);
        else if (vpt <= 4) PTA_RMS_STREAM(4, 4);
        else if (vpt <= 8) PTA_RMS_STREAM(8, 4);
        else return pta_fail("layernorm_stream: rows of %d features are more than the 8192 the kernel holds", H);
    } else {
        if (vpt <= 1) PTA_RMS_STREAM(1, 1);
        else if (vpt <= 4) PTA_RMS_STREAM(4, 1);
        else if (vpt <= 16) PTA_RMS_STREAM(16, 1);
        else if (vpt <= 32) PTA_RMS_STREAM(32, 1);
        else return pta_fail("layernorm_stream: rows of %d features are more than the 8192 the kernel holds", H);
    }
#undef PTA_RMS_STREAM
    return pta_check_launch("layernorm_stream");
}

template <typename T>
static int launch_ln_stream(void* out_narrow, float* out_wide, const float* x, const void* y, long y_ld, const float* wy,
                            const float* by, float mult, const float* add, const float* vec, const int* rows, const float* w,
                            const float* b, float eps, int M, int H, hipStream_t s) {
    // the block's size follows from the row's length alone
    const int threads = H <= 64 ? 64 : H <= 128 ? 128 : 256;
    const int vpt = (H + threads - 1) / threads;
#define PTA_LN_STREAM(V)                                                                                                    \
    hipLaunchKernelGGL((layernorm_stream_kernel<T, V>), dim3(M), dim3(threads), 0, s, (T*)out_narrow, out_wide, x, (const T*)y, \
                       y_ld, wy, by, mult, add, vec, rows, w, b, eps, H)
    if (vpt <= 1) PTA_LN_STREAM(1);
    else if (vpt <= 2) PTA_LN_STREAM(2);
    else if (vpt <= 4) PTA_LN_STREAM(4);
    else if (vpt <= 8) PTA_LN_STREAM(8);
    else if (vpt <= 16) PTA_LN_STREAM(16);
    else if (vpt <= 32) PTA_LN_STREAM(32);
    else return pta_fail("layernorm_stream: rows of %d features are more than the 8192 the kernel holds", H);
#undef PTA_LN_STREAM
    return pta_check_launch("layernorm_stream");
}

extern "C" int pta_layernorm_stream(void* out_narrow, float* out_wide, const float* x, const void* y, long y_ld,
                                    const float* wy, const float* by, float mult, const float* add, const float* vec,
                                    const int* rows, const float* w, const float* b, float eps, int M, int H, int rms, int dtype,
                                    void* stream) {
    PTA_REQUIRE(M > 0 && H > 0, "layernorm_stream: sizes must be positive (M=%d H=%d)", M, H);
    PTA_REQUIRE(x || y, "layernorm_stream: neither a stream nor a sublayer's output given");
    PTA_REQUIRE(!y || (wy && (by || rms) && y_ld >= H), "layernorm_stream: a sublayer's output needs its norm's weight and bias");
    PTA_REQUIRE(rms || (w != nullptr) == (b != nullptr), "layernorm_stream: weight and bias come together");
    PTA_REQUIRE(!rms || (!by && !b), "layernorm_stream: RMS norms have no bias");
    PTA_REQUIRE(!w || out_narrow, "layernorm_stream: a norm of the stream needs a place for its output");
    PTA_REQUIRE(out_narrow || out_wide, "layernorm_stream: nothing to write");
    hipStream_t s = (hipStream_t)stream;
    PTA_REQUIRE(dtype == PTA_F32 || dtype == PTA_BF16, "layernorm_stream: unknown dtype %d", dtype);
    if (rms)
        return dtype == PTA_F32
                   ? launch_rms_stream<float>(out_narrow, out_wide, x, y, y_ld, wy, mult, add, vec, rows, w, eps, M, H, s)
                   : launch_rms_stream<bf16_t>(out_narrow, out_wide, x, y, y_ld, wy, mult, add, vec, rows, w, eps, M, H, s);
    if (dtype == PTA_F32)
        return launch_ln_stream<float>(out_narrow, out_wide, x, y, y_ld, wy, by, mult, add, vec, rows, w, b, eps, M, H, s);
    return launch_ln_stream<bf16_t>(out_narrow, out_wide, x, y, y_ld, wy, by, mult, add, vec, rows, w, b, eps, M, H, s);
}
