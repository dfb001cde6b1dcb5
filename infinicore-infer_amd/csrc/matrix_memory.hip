// Mixers whose state is a matrix S [dk, dv] per head, in float32, read by q and written by k and v:
//
//     S <- decay * S;   u = scale * (v - S^T k)  (delta rule)   or   u = scale * v;   S <- S + k u^T;   o = q_scale * S^T q
//
// with one decay per key channel (it acts on S's rows) or one per head, both given as factors.  The read-out sees the
// token's own write.  With `extra` a head has one more column whose v is 1 at every token: its read-out (the sum of the
// decayed keys against q) normalises the others.
//
//   * ic_delta_prep: the delta rule's rows: convolution and silu on q, k, v, unit length per head for q and k, the step
//     sizes sigmoid(b), one decay per head where the rule has that, and the convolution's state,
//   * ic_memory_gates: exponential input and forget gates held in logarithms against a running maximum, as factors,
//   * ic_matrix_step: one token per request, ic_matrix_scan: portions,
//   * ic_gated_head_norm: o per head to unit root mean square, a weight, a gate.
//
// A step's tokens are rows 0..T-1; request r owns rows req_start[r] .. req_start[r+1]-1 and the state slot
// state_slots[r].  A head's state lies column by column ([dv (+1)][dk]), so that the lanes that share a column read and
// write whole lines.
#include "short_conv.h"

__device__ __forceinline__ float mm_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float mm_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float mm_silu(float z) { return z / (1.0f + expf(-z)); }
// Activations with the hardware's exponential and reciprocal (a last place or two off).
__device__ __forceinline__ float mm_sigmoid_fast(float z) { return __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }
__device__ __forceinline__ float mm_silu_fast(float z) { return z * mm_sigmoid_fast(z); }

// ---------------------------------------------------------------------------------------------
// rows[t] = [q (G dk) | k (G dk) | v (H dv) | ..]: every channel passes the convolution and silu; q and k heads are then
// divided by sqrt(sum of squares + unit_eps).  out [T, 2 G dk + H dv] float32; beta[t, h] = sigmoid(b[t, h]);
// with d.a: d.decay[t, h] = exp(-d.rate[h] softplus(a[t, h] + d.bias[h])), one decay factor per head.
// grid (T, ceil((2 G + H + 1) / 4)), a wave a head (the last one: the step sizes).  single: every request brings one
// token, and the wave moves the convolution's state on itself.
// ---------------------------------------------------------------------------------------------
constexpr int kPrepMaxPerLane = 16;

struct HeadDecay { const void* a; int a_stride; const float *rate, *bias; float* decay; };

// The step sizes and decay factors of tokens t0 .. t1 - 1, by one wave.
template <typename T>
__device__ __forceinline__ void head_steps(const T* b, int b_stride, float* beta, const HeadDecay& d, int H, int t0, int t1, int lane) {
    for (int e = t0 * H + lane; e < t1 * H; e += 64) {
        const int t = e / H, h = e - t * H;
        beta[e] = mm_sigmoid(to_f32(b[(size_t)t * b_stride + h]));
        if (d.a) d.decay[e] = expf(-d.rate[h] * mm_softplus(to_f32(((const T*)d.a)[(size_t)t * d.a_stride + h]) + d.bias[h]));
    }
}

template <typename T>
__global__ void __launch_bounds__(256)
delta_prep_kernel(const T* __restrict__ rows, int row_stride, const float* __restrict__ w, int taps, const T* __restrict__ b,
                  int b_stride, float* __restrict__ out, float* __restrict__ beta, int G, int H, int dk, int dv,
                  float unit_eps, float* __restrict__ state, long long state_stride, const int* __restrict__ token_req,
                  const int* __restrict__ req_start, const int* __restrict__ state_slots, int single, HeadDecay d) {
    const int t = blockIdx.x, lane = threadIdx.x & 63, head = blockIdx.y * 4 + (threadIdx.x >> 6);
    const int C = 2 * G * dk + H * dv;
    if (head > 2 * G + H) return;
    if (head == 2 * G + H) {
        head_steps<T>(b, b_stride, beta, d, H, t, t + 1, lane);
        return;
    }
    const int r = token_req[t], start = req_start[r];
    float* st = state + (long long)state_slots[r] * state_stride;
    const bool unit = head < 2 * G;
    const int n = unit ? dk : dv, c0 = unit ? head * dk : 2 * G * dk + (head - 2 * G) * dv;
    float val[kPrepMaxPerLane];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < kPrepMaxPerLane; ++j) {
        val[j] = 0.f;
        if (64 * j >= n) break;
        const int e = lane + 64 * j;
        if (e < n) {
            val[j] = mm_silu(conv_at<T>(rows, row_stride, w, taps, C, st, t, start, c0 + e));
            if (single && taps > 1) conv_shift(st, taps, C, c0 + e, to_f32(rows[(size_t)t * row_stride + c0 + e]));
        }
        ss += val[j] * val[j];
    }
    const float f = unit ? 1.0f / sqrtf(wave_sum(ss) + unit_eps) : 1.f;
    float* o = out + (size_t)t * C + c0;
#pragma unroll
    for (int j = 0; j < kPrepMaxPerLane; ++j) {
        if (64 * j >= n) break;
        const int e = lane + 64 * j;
        if (e < n) o[e] = val[j] * f;
    }
}

// The same for portions: a wave a head and kPrepTile consecutive tokens, two neighbouring channels a lane (n at most 128 NJ,
// even); every row is read once and waits in registers for the tokens behind it.
constexpr int kPrepTile = 16;

template <typename T> __device__ __forceinline__ float2 load_pair(const T* p) {
    if (sizeof(T) == 4) return *reinterpret_cast<const float2*>(p);
    const uint32_t v = *reinterpret_cast<const uint32_t*>(p);
    return make_float2(__uint_as_float(v << 16), __uint_as_float(v & 0xffff0000u));
}

template <typename T, int TMAX, int NJ>
__global__ void __launch_bounds__(256)
delta_prep_tile_kernel(const T* __restrict__ rows, int row_stride, const float* __restrict__ w, int taps, const T* __restrict__ b,
                       int b_stride, float* __restrict__ out, float* __restrict__ beta, int G, int H, int dk, int dv, float unit_eps,
                       const float* __restrict__ state, long long state_stride, const int* __restrict__ token_req,
                       const int* __restrict__ req_start, const int* __restrict__ state_slots, int n_tokens, HeadDecay d) {
    const int lane = threadIdx.x & 63, head = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int t0 = blockIdx.x * kPrepTile, t1 = min(n_tokens, t0 + kPrepTile);
    const int C = 2 * G * dk + H * dv;
    if (head > 2 * G + H) return;
    if (head == 2 * G + H) {
        head_steps<T>(b, b_stride, beta, d, H, t0, t1, lane);
        return;
    }
    const bool unit = head < 2 * G;
    const int n = unit ? dk : dv, c0 = unit ? head * dk : 2 * G * dk + (head - 2 * G) * dv;
    ConvWindow<T, TMAX> win[NJ][2];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int e = 2 * (lane + 64 * j), c = e < n ? c0 + e : c0;
        win[j][0].weights(w, taps, c);
        win[j][1].weights(w, taps, c + 1);
    }
    int next = t0;                                                   // the row where the window is filled anew
    constexpr int AHEAD = 8;                                         // rows on their way while others are computed on
    for (int ta = t0; ta < t1; ta += AHEAD) {
        float2 in[AHEAD][NJ];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i)
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
                const int e = 2 * (lane + 64 * j);
                in[i][j] = (ta + i < t1 && e < n) ? load_pair(rows + (size_t)(ta + i) * row_stride + c0 + e) : make_float2(0.f, 0.f);
            }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            const int t = ta + i;
            if (t >= t1) break;
            if (t == next) {
                const int r = token_req[t], start = req_start[r];
                next = req_start[r + 1];
                const float* st = state + (long long)state_slots[r] * state_stride;
#pragma unroll
                for (int j = 0; j < NJ; ++j) {
                    const int e = 2 * (lane + 64 * j), c = e < n ? c0 + e : c0;
                    win[j][0].restart(rows, row_stride, taps, C, st, t, start, c);
                    win[j][1].restart(rows, row_stride, taps, C, st, t, start, c + 1);
                }
            }
            float2 y[NJ];
            float ss = 0.f;
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
                y[j] = make_float2(mm_silu_fast(win[j][0].next(in[i][j].x)), mm_silu_fast(win[j][1].next(in[i][j].y)));
                if (2 * (lane + 64 * j) < n) ss += y[j].x * y[j].x + y[j].y * y[j].y;
            }
            const float f = unit ? __builtin_amdgcn_rsqf(group_sum<64>(ss) + unit_eps) : 1.f;
            float* o = out + (size_t)t * C + c0;
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
                const int e = 2 * (lane + 64 * j);
                if (e < n) *reinterpret_cast<float2*>(o + e) = make_float2(y[j].x * f, y[j].y * f);
            }
        }
    }
}

// Launches the tile kernel where it takes the sizes.
template <typename T>
static bool delta_prep_tiles(const T* rows, int row_stride, const float* w, int taps, const T* b, int b_stride, float* out, float* beta,
                             int G, int H, int dk, int dv, float unit_eps, const float* state, long long state_stride,
                             const int* token_req, const int* req_start, const int* state_slots, int T_, const HeadDecay& d, hipStream_t stream) {
    const int n = dk > dv ? dk : dv;
    if (T_ < 64 || n > 256 || dk % 2 || dv % 2 || row_stride % 2 || (uintptr_t)rows % (2 * sizeof(T)) || (uintptr_t)out % 8) return false;
    dim3 grid((T_ + kPrepTile - 1) / kPrepTile, (2 * G + H + 1 + 3) / 4), block(256);
#define IC_DP(TM, NJ_)                                                                                                          \
    hipLaunchKernelGGL((delta_prep_tile_kernel<T, TM, NJ_>), grid, block, 0, stream, rows, row_stride, w, taps, b, b_stride, out, \
                       beta, G, H, dk, dv, unit_eps, state, state_stride, token_req, req_start, state_slots, T_, d)
    if (taps <= 4) { if (n <= 128) IC_DP(4, 1); else IC_DP(4, 2); }
    else { if (n <= 128) IC_DP(8, 1); else IC_DP(8, 2); }
#undef IC_DP
    return true;
}

IC_EXPORT int ic_delta_prep(const void* rows, int row_stride, int dtype, const float* w, int taps, const void* b, int b_stride,
                            float* out, float* beta, int G, int H, int dk, int dv, float unit_eps, float* state,
                            long long state_stride, const int* token_req, const int* req_start, const int* state_slots, int T,
                            int R, int single, const void* a, int a_stride, const float* rate, const float* a_bias, float* decay,
                            hipStream_t stream) {
    if (T <= 0) return IC_OK;
    if (a && (!rate || !a_bias || !decay)) return IC_ERR_ARG;
    if ((long long)T * H > 0x7fffffff) return IC_ERR_TOO_LARGE;
    const HeadDecay d{a, a_stride, rate, a_bias, decay};
    if (G <= 0 || H <= 0 || dk <= 0 || dv <= 0 || taps < 1 || taps > kConvMaxTaps || R <= 0 || !state || !w) return IC_ERR_ARG;
    if (dk > 64 * kPrepMaxPerLane || dv > 64 * kPrepMaxPerLane) return IC_ERR_TOO_LARGE;
    if (single && T != R) return IC_ERR_ARG;
    const int C = 2 * G * dk + H * dv;
    dim3 grid(T, (2 * G + H + 1 + 3) / 4), block(256), sgrid((C + 255) / 256, R);
    if (dtype == IC_F32) {
        if (single || !delta_prep_tiles<float>((const float*)rows, row_stride, w, taps, (const float*)b, b_stride, out, beta, G, H, dk, dv, unit_eps,
                                           state, state_stride, token_req, req_start, state_slots, T, d, stream))
            hipLaunchKernelGGL(delta_prep_kernel<float>, grid, block, 0, stream, (const float*)rows, row_stride, w, taps, (const float*)b,
                           b_stride, out, beta, G, H, dk, dv, unit_eps, state, state_stride, token_req, req_start, state_slots, single, d);
        if (taps > 1 && !single)
            hipLaunchKernelGGL(conv_state_kernel<float>, sgrid, block, 0, stream, (const float*)rows, row_stride, nullptr, taps, C,
                               state, state_stride, req_start, state_slots);
    } else if (dtype == IC_BF16) {
        if (single || !delta_prep_tiles<bf16>((const bf16*)rows, row_stride, w, taps, (const bf16*)b, b_stride, out, beta, G, H, dk, dv, unit_eps,
                                           state, state_stride, token_req, req_start, state_slots, T, d, stream))
            hipLaunchKernelGGL(delta_prep_kernel<bf16>, grid, block, 0, stream, (const bf16*)rows, row_stride, w, taps, (const bf16*)b,
                           b_stride, out, beta, G, H, dk, dv, unit_eps, state, state_stride, token_req, req_start, state_slots, single, d);
        if (taps > 1 && !single)
            hipLaunchKernelGGL(conv_state_kernel<bf16>, sgrid, block, 0, stream, (const bf16*)rows, row_stride, nullptr, taps, C,
                               state, state_stride, req_start, state_slots);
    } else
        return IC_ERR_UNSUPPORTED;
    return ic_launch_status();
}

// ---------------------------------------------------------------------------------------------
// Exponential gates.  z [T, 2 H] float32 holds the input gates' pre-activations, then the forget gates'.
//   i = cap tanh((z_i + b_i) / cap),  f = logsigmoid(cap tanh((z_f + b_f) / cap)),  m_t = max(f_t + m_(t-1), i_t)
//   keep[t, h] = exp(f_t + m_(t-1) - m_t),  add[t, h] = exp(i_t - m_t),  floor[t, h] = exp(-m_t)
// A block per (request, head) takes its width in tokens at a time: the pairs (a, b) = (sum of f, largest i + later f) of a
// run of tokens combine as (a1 + a2, max(b1 + a2, b2)), and m_t = max(m_0 + a, b).  m_0 lives in the state (zero at the start).
// ---------------------------------------------------------------------------------------------
template <int WAVES>
__global__ void __launch_bounds__(64 * WAVES)
memory_gates_kernel(const float* __restrict__ z, int z_stride, const float* __restrict__ bi, const float* __restrict__ bf, float cap,
                    int H, float* __restrict__ keep, float* __restrict__ add, float* __restrict__ floor_, float* __restrict__ state,
                    long long state_stride, const int* __restrict__ req_start, const int* __restrict__ state_slots) {
    __shared__ float a_s[2][WAVES], b_s[2][WAVES];
    const int h = blockIdx.x, r = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int end = req_start[r + 1];
    float* st = state + (long long)state_slots[r] * state_stride + h;
    float m0 = *st;
    const float b_i = bi[h], b_f = bf[h];
    int half = 0;
    for (int t0 = req_start[r]; t0 < end; t0 += 64 * WAVES, half ^= 1) {
        const int t = t0 + threadIdx.x;
        const bool ok = t < end;
        float li = 0.f, lf = 0.f;
        if (ok) {
            const float* zr = z + (size_t)t * z_stride;
            li = cap * tanhf((zr[h] + b_i) / cap);
            lf = -mm_softplus(-cap * tanhf((zr[H + h] + b_f) / cap));
        }
        float a = lf, b = ok ? li : -INFINITY;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const float a1 = __shfl_up(a, o, kWave), b1 = __shfl_up(b, o, kWave);
            if (lane >= o) {
                b = fmaxf(b1 + a, b);
                a = a1 + a;
            }
        }
        float mw = m0;                                               // the maximum before this wave's tokens, and behind the block's
        if (WAVES > 1) {
            if (lane == 63) {
                a_s[half][wave] = a;
                b_s[half][wave] = b;
            }
            __syncthreads();
            float all = m0;
#pragma unroll
            for (int w = 0; w < WAVES; ++w) {
                if (w == wave) mw = all;
                all = fmaxf(all + a_s[half][w], b_s[half][w]);
            }
            m0 = all;
        }
        const float m = fmaxf(mw + a, b);
        const float before = __shfl_up(m, 1, kWave);
        const float m_prev = lane ? before : mw;
        if (ok) {
            const size_t i = (size_t)t * H + h;
            keep[i] = expf(lf + m_prev - m);
            add[i] = expf(li - m);
            floor_[i] = expf(-m);
        }
        if (WAVES == 1) m0 = __shfl(m, 63, kWave);
    }
    if (threadIdx.x == 0) *st = m0;
}

IC_EXPORT int ic_memory_gates(const float* z, int z_stride, const float* bi, const float* bf, float cap, int H, float* keep,
                              float* add, float* floor_, float* state, long long state_stride, const int* req_start,
                              const int* state_slots, int T, int R, hipStream_t stream) {
    if (R <= 0) return IC_OK;
    if (H <= 0 || R > 65535 || z_stride < 2 * H || !(cap > 0.f) || !state) return IC_ERR_ARG;
    if (T >= 256)                                                    // (some request brings many tokens, most likely)
        hipLaunchKernelGGL(memory_gates_kernel<16>, dim3(H, R), dim3(1024), 0, stream, z, z_stride, bi, bf, cap, H, keep, add, floor_, state,
                           state_stride, req_start, state_slots);
    else
        hipLaunchKernelGGL(memory_gates_kernel<1>, dim3(H, R), dim3(64), 0, stream, z, z_stride, bi, bf, cap, H, keep, add, floor_, state,
                           state_stride, req_start, state_slots);
    return ic_launch_status();
}

// ---------------------------------------------------------------------------------------------
// The recurrence.  L lanes share a column of S; lane p of them keeps the NI rows 4 (p + L j) .. + 3, j < NI / 4, of NC
// columns in registers, so a token costs NI multiplications by the decay, two (delta rule) or one sums of NI products,
// which the L lanes add up among themselves, and NI updates.  Both sums run over the decayed state before the token's
// write; the read-out's share of the write is (k . q) u, k . q being formed once per token for the whole block.
// ---------------------------------------------------------------------------------------------
struct MatrixMemoryArgs {
    const void *q, *k, *v;            // [T, ..]: query/key head h / per at offset (h / per) * dk, value head h at h * dv
    int q_stride, k_stride, v_stride;
    const float* decay;               // [T, H * dk] (per channel) or [T, H]
    const float* scale;               // [T, H] or null (1)
    int H, per, dk, dv, cols;         // cols = dv, or dv + 1 with the extra column
    float q_scale;
    float* out;                       // [T, H * dv]
    float* extra_out;                 // [T, H], with the extra column
    float* state;
    long long state_stride;
    const int *req_start, *state_slots;
    int vec;                          // rows and state made of whole 16-byte pieces
};

// NI rows of a column (global, rows dk): lane p's pieces of four.
template <int L, int NI> __device__ __forceinline__ void mm_load_state(const float* c, int dk, int p, bool vec, float* s) {
#pragma unroll
    for (int j = 0; j < NI / 4; ++j) {
        const int row = 4 * (p + L * j);
        if (vec) {
            float4 v = row < dk ? *reinterpret_cast<const float4*>(c + row) : make_float4(0.f, 0.f, 0.f, 0.f);
            s[4 * j] = v.x; s[4 * j + 1] = v.y; s[4 * j + 2] = v.z; s[4 * j + 3] = v.w;
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) s[4 * j + i] = row + i < dk ? c[row + i] : 0.f;
        }
    }
}
template <int L, int NI> __device__ __forceinline__ void mm_store_state(float* c, int dk, int p, bool vec, const float* s) {
#pragma unroll
    for (int j = 0; j < NI / 4; ++j) {
        const int row = 4 * (p + L * j);
        if (vec) {
            if (row < dk) *reinterpret_cast<float4*>(c + row) = make_float4(s[4 * j], s[4 * j + 1], s[4 * j + 2], s[4 * j + 3]);
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (row + i < dk) c[row + i] = s[4 * j + i];
        }
    }
}
// The same rows of a token's vector (element type T); the rest reads as zero.
template <typename T, int L, int NI> __device__ __forceinline__ void mm_load_row(const T* x, int dk, int p, bool vec, float* o) {
#pragma unroll
    for (int j = 0; j < NI / 4; ++j) {
        const int row = 4 * (p + L * j);
        if (vec && row < dk) {
            if (sizeof(T) == 4) {
                const float4 v = *reinterpret_cast<const float4*>(x + row);
                o[4 * j] = v.x; o[4 * j + 1] = v.y; o[4 * j + 2] = v.z; o[4 * j + 3] = v.w;
            } else {
                const uint2 v = *reinterpret_cast<const uint2*>(x + row);
                o[4 * j] = __uint_as_float(v.x << 16); o[4 * j + 1] = __uint_as_float(v.x & 0xffff0000u);
                o[4 * j + 2] = __uint_as_float(v.y << 16); o[4 * j + 3] = __uint_as_float(v.y & 0xffff0000u);
            }
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) o[4 * j + i] = (!vec && row + i < dk) ? to_f32(x[row + i]) : 0.f;
        }
    }
}

// One token of one column: s in registers, sums over the L lanes of the column.
template <int L, int NI, bool DELTA, bool CHANNEL>
__device__ __forceinline__ float mm_token(float* s, const float* k, const float* q, const float* g, float dec, float scale, float kq,
                                          float v) {
    float r1[2] = {0.f, 0.f}, r2[2] = {0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        if (CHANNEL) s[i] *= g[i];
        if (DELTA) r1[i & 1] += s[i] * k[i];
        r2[i & 1] += s[i] * q[i];
    }
    float sk = r1[0] + r1[1], sq = r2[0] + r2[1];
    if (!CHANNEL) { sk *= dec; sq *= dec; }
    if (DELTA) sk = group_sum<L>(sk);
    sq = group_sum<L>(sq);
    const float u = scale * (DELTA ? v - sk : v);
#pragma unroll
    for (int i = 0; i < NI; ++i) s[i] = (CHANNEL ? s[i] : dec * s[i]) + k[i] * u;
    return sq + kq * u;
}

// One token per request: no tile, every lane reads its own rows.  grid (ceil(cols / (256 / L)), H, R).
template <typename T, int L, int NI, bool DELTA, bool CHANNEL>
__global__ void __launch_bounds__(256) matrix_step_kernel(MatrixMemoryArgs a) {
    const int h = blockIdx.y, r = blockIdx.z, p = threadIdx.x % L;
    const int col = blockIdx.x * (256 / L) + threadIdx.x / L;
    if (a.req_start[r] >= a.req_start[r + 1]) return;
    const int t = a.req_start[r];
    const bool vec = a.vec != 0, live = col < a.cols;
    float* c = a.state + (long long)a.state_slots[r] * a.state_stride + ((size_t)h * a.cols + (live ? col : 0)) * a.dk;
    float s[NI], k[NI], q[NI], g[NI];
    mm_load_state<L, NI>(c, a.dk, p, vec, s);
    const int hk = h / a.per;
    mm_load_row<T, L, NI>((const T*)a.k + (size_t)t * a.k_stride + (size_t)hk * a.dk, a.dk, p, vec, k);
    mm_load_row<T, L, NI>((const T*)a.q + (size_t)t * a.q_stride + (size_t)hk * a.dk, a.dk, p, vec, q);
    if (CHANNEL) mm_load_row<float, L, NI>(a.decay + ((size_t)t * a.H + h) * a.dk, a.dk, p, vec, g);
    const float dec = CHANNEL ? 1.f : a.decay[(size_t)t * a.H + h];
    const float scale = a.scale ? a.scale[(size_t)t * a.H + h] : 1.f;
    const float v = col < a.dv ? to_f32(((const T*)a.v)[(size_t)t * a.v_stride + (size_t)h * a.dv + col]) : 1.f;
    float kq = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) kq += k[i] * q[i];
    kq = group_sum<L>(kq);
    const float o = a.q_scale * mm_token<L, NI, DELTA, CHANNEL>(s, k, q, g, dec, scale, kq, v);
    if (!live) return;
    mm_store_state<L, NI>(c, a.dk, p, vec, s);
    if (p == 0) {
        if (col < a.dv) a.out[((size_t)t * a.H + h) * a.dv + col] = o;
        else a.extra_out[(size_t)t * a.H + h] = o;
    }
}

// Portions: the tokens pass through LDS TT at a time (two tiles: one is computed on while the next one's rows are on
// their way into registers).  grid (ceil(cols / (256 / L * NC)), H, R).
template <typename T, int L, int NI, int NC, bool DELTA, bool CHANNEL>
__global__ void __launch_bounds__(256) matrix_scan_kernel(MatrixMemoryArgs a) {
    constexpr int ROW = L * NI;                                      // a token's vector in LDS, zeros behind dk
    constexpr int TT = (2048 / ROW < 16 ? 2048 / ROW : 16);          // tokens a tile
    constexpr int CG = 256 / L, CB = CG * NC;                        // columns a block
    constexpr int VE = 16 / (int)sizeof(T), PR = ROW / VE;           // 16-byte pieces of a vector
    constexpr int NP = (TT * PR + 255) / 256, NG = (TT * ROW / 4 + 255) / 256, NV = (TT * CB + 255) / 256;
    __shared__ __align__(16) float ks[2][TT][ROW], qs[2][TT][ROW], gs[CHANNEL ? 2 : 1][CHANNEL ? TT : 1][CHANNEL ? ROW : 4];
    __shared__ float vs[2][TT][CB];
    __shared__ __align__(16) float4 sc[2][TT];                       // decay per head, scale, k . q
    const int h = blockIdx.y, r = blockIdx.z, tid = threadIdx.x, p = tid % L, cg = tid / L, c0 = blockIdx.x * CB;
    const int begin = a.req_start[r], end = a.req_start[r + 1];
    if (begin >= end) return;
    const bool vec = a.vec != 0;
    const int hk = h / a.per;
    const T* kp = (const T*)a.k + (size_t)hk * a.dk;
    const T* qp = (const T*)a.q + (size_t)hk * a.dk;
    const T* vp = (const T*)a.v + (size_t)h * a.dv;
    const float* gp = a.decay + (CHANNEL ? (size_t)h * a.dk : (size_t)h);
    const int g_stride = CHANNEL ? a.H * a.dk : a.H;
    float* st = a.state + (long long)a.state_slots[r] * a.state_stride + (size_t)h * a.cols * a.dk;
    float s[NC][NI];
#pragma unroll
    for (int j = 0; j < NC; ++j) {
        const int col = c0 + cg + CG * j;
        if (col < a.cols) mm_load_state<L, NI>(st + (size_t)col * a.dk, a.dk, p, vec, s[j]);
        else
#pragma unroll
            for (int i = 0; i < NI; ++i) s[j][i] = 0.f;
    }
    uint4 pk[NP], pq[NP];
    float4 pg[NG];
    float pv[NV], ps[2];
    auto fetch = [&](int t0) {                                       // a tile's rows into registers (zeros behind dk and behind the portion)
        const int n = min(TT, end - t0);
        if (vec) {
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                const int e = tid + 256 * i, tt = e / PR, o = (e % PR) * VE;
                const bool ok = tt < n && o < a.dk;
                pk[i] = ok ? *reinterpret_cast<const uint4*>(kp + (size_t)(t0 + tt) * a.k_stride + o) : uint4{0u, 0u, 0u, 0u};
                pq[i] = ok ? *reinterpret_cast<const uint4*>(qp + (size_t)(t0 + tt) * a.q_stride + o) : uint4{0u, 0u, 0u, 0u};
            }
            if (CHANNEL) {
#pragma unroll
                for (int i = 0; i < NG; ++i) {
                    const int e = tid + 256 * i, tt = e / (ROW / 4), o = (e % (ROW / 4)) * 4;
                    pg[i] = (tt < n && o < a.dk) ? *reinterpret_cast<const float4*>(gp + (size_t)(t0 + tt) * g_stride + o)
                                                 : make_float4(0.f, 0.f, 0.f, 0.f);
                }
            }
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int e = tid + 256 * i, tt = e / CB, col = c0 + e % CB;
            pv[i] = tt >= n ? 0.f : col < a.dv ? to_f32(vp[(size_t)(t0 + tt) * a.v_stride + col]) : 1.f;
        }
        if (tid < n) {
            ps[0] = CHANNEL ? 1.f : gp[(size_t)(t0 + tid) * g_stride];
            ps[1] = a.scale ? a.scale[(size_t)(t0 + tid) * a.H + h] : 1.f;
        }
    };
    auto put = [&](int b, int t0) {                                  // .. and from there into LDS
        const int n = min(TT, end - t0);
        if (vec) {
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                const int e = tid + 256 * i, tt = e / PR, o = (e % PR) * VE;
                if (TT * PR % 256 && tt >= TT) continue;
                if (sizeof(T) == 4) {
                    *reinterpret_cast<uint4*>(&ks[b][tt][o]) = pk[i];
                    *reinterpret_cast<uint4*>(&qs[b][tt][o]) = pq[i];
                } else {
                    const uint4 x = pk[i], y = pq[i];
                    *reinterpret_cast<uint4*>(&ks[b][tt][o]) = uint4{x.x << 16, x.x & 0xffff0000u, x.y << 16, x.y & 0xffff0000u};
                    *reinterpret_cast<uint4*>(&ks[b][tt][o + 4]) = uint4{x.z << 16, x.z & 0xffff0000u, x.w << 16, x.w & 0xffff0000u};
                    *reinterpret_cast<uint4*>(&qs[b][tt][o]) = uint4{y.x << 16, y.x & 0xffff0000u, y.y << 16, y.y & 0xffff0000u};
                    *reinterpret_cast<uint4*>(&qs[b][tt][o + 4]) = uint4{y.z << 16, y.z & 0xffff0000u, y.w << 16, y.w & 0xffff0000u};
                }
            }
            if (CHANNEL) {
#pragma unroll
                for (int i = 0; i < NG; ++i) {
                    const int e = tid + 256 * i, tt = e / (ROW / 4), o = (e % (ROW / 4)) * 4;
                    if (TT * ROW / 4 % 256 && tt >= TT) continue;
                    *reinterpret_cast<float4*>(&gs[CHANNEL ? b : 0][CHANNEL ? tt : 0][CHANNEL ? o : 0]) = pg[i];
                }
            }
        } else {
            for (int e = tid; e < TT * ROW; e += 256) {
                const int tt = e / ROW, o = e % ROW;
                const bool ok = tt < n && o < a.dk;
                ks[b][tt][o] = ok ? to_f32(kp[(size_t)(t0 + tt) * a.k_stride + o]) : 0.f;
                qs[b][tt][o] = ok ? to_f32(qp[(size_t)(t0 + tt) * a.q_stride + o]) : 0.f;
                if (CHANNEL) gs[CHANNEL ? b : 0][CHANNEL ? tt : 0][CHANNEL ? o : 0] = ok ? gp[(size_t)(t0 + tt) * g_stride + o] : 0.f;
            }
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int e = tid + 256 * i, tt = e / CB;
            if (TT * CB % 256 && tt >= TT) continue;
            vs[b][tt][e % CB] = pv[i];
        }
        if (tid < n) {
            sc[b][tid].x = ps[0];
            sc[b][tid].y = ps[1];
        }
    };
    auto rows4 = [&](const float* row, float* o) {
#pragma unroll
        for (int j = 0; j < NI / 4; ++j) {
            const float4 v = *reinterpret_cast<const float4*>(row + 4 * (p + L * j));
            o[4 * j] = v.x; o[4 * j + 1] = v.y; o[4 * j + 2] = v.z; o[4 * j + 3] = v.w;
        }
    };
    fetch(begin);
    int b = 0;
    for (int t0 = begin; t0 < end; t0 += TT, b ^= 1) {
        const int n = min(TT, end - t0);
        put(b, t0);
        __syncthreads();
        for (int tt = cg; tt < n; tt += CG) {
            float k[NI], q[NI], d = 0.f;
            rows4(ks[b][tt], k);
            rows4(qs[b][tt], q);
#pragma unroll
            for (int i = 0; i < NI; ++i) d += k[i] * q[i];
            d = group_sum<L>(d);
            if (p == 0) sc[b][tt].z = d;
        }
        if (t0 + TT < end) fetch(t0 + TT);
        __syncthreads();
        float keep[NC];
#pragma unroll
        for (int j = 0; j < NC; ++j) keep[j] = 0.f;
        // Where the registers suffice a token's vectors are read one token ahead: nothing else hides the way out of LDS from a
        // wave that is alone on its unit.
        constexpr bool AHEAD = NI <= 8;
        float k[2][NI], q[2][NI], g[2][CHANNEL ? NI : 1], v[2][NC];
        float4 c[2];
        auto ahead = [&](int tt, int x) {
            rows4(ks[b][tt], k[x]);
            if (CHANNEL) rows4(gs[CHANNEL ? b : 0][CHANNEL ? tt : 0], g[x]);
            rows4(qs[b][tt], q[x]);
            c[x] = sc[b][tt];
#pragma unroll
            for (int j = 0; j < NC; ++j) v[x][j] = vs[b][tt][cg + CG * j];
            if (AHEAD) __builtin_amdgcn_sched_barrier(0);
        };
        auto token = [&](int tt, int x) {
            if (!AHEAD) ahead(tt, x);
#pragma unroll
            for (int j = 0; j < NC; ++j) {
                const float o = mm_token<L, NI, DELTA, CHANNEL>(s[j], k[x], q[x], g[x], c[x].x, c[x].y, c[x].z, v[x][j]);
                keep[j] = p == tt ? o : keep[j];
            }
        };
        if (AHEAD) ahead(0, 0);
        if (n == TT) {
#pragma unroll
            for (int tt = 0; tt < TT; ++tt) {
                if (AHEAD && tt + 1 < TT) ahead(tt + 1, (tt + 1) & 1);
                token(tt, tt & 1);
            }
        } else
            for (int tt = 0; tt < n; tt += 2) {
                if (AHEAD && tt + 1 < n) ahead(tt + 1, 1);
                token(tt, 0);
                if (tt + 1 >= n) break;
                if (AHEAD && tt + 2 < n) ahead(tt + 2, 0);
                token(tt + 1, 1);
            }
        if (p < n) {
#pragma unroll
            for (int j = 0; j < NC; ++j) {
                const int col = c0 + cg + CG * j;
                const size_t i = (size_t)(t0 + p) * a.H + h;
                if (col < a.dv) a.out[i * a.dv + col] = a.q_scale * keep[j];
                else if (col < a.cols) a.extra_out[i] = a.q_scale * keep[j];
            }
        }
    }
#pragma unroll
    for (int j = 0; j < NC; ++j) {
        const int col = c0 + cg + CG * j;
        if (col < a.cols) mm_store_state<L, NI>(st + (size_t)col * a.dk, a.dk, p, vec, s[j]);
    }
}

template <typename T, bool DELTA, bool CHANNEL>
static int matrix_memory_launch(const MatrixMemoryArgs& a, int R, int single, int columns_a_thread, hipStream_t stream) {
#define IC_MM(L_, NI_)                                                                                                      \
    do {                                                                                                                    \
        constexpr int CG = 256 / L_;                                                                                        \
        if (single)                                                                                                         \
            hipLaunchKernelGGL((matrix_step_kernel<T, L_, NI_, DELTA, CHANNEL>), dim3((a.cols + CG - 1) / CG, a.H, R), dim3(256), \
                               0, stream, a);                                                                               \
        else if (columns_a_thread == 2)                                                                                     \
            hipLaunchKernelGGL((matrix_scan_kernel<T, L_, NI_, 2, DELTA, CHANNEL>),                                          \
                               dim3((a.cols + 2 * CG - 1) / (2 * CG), a.H, R), dim3(256), 0, stream, a);                     \
        else                                                                                                                \
            hipLaunchKernelGGL((matrix_scan_kernel<T, L_, NI_, 1, DELTA, CHANNEL>), dim3((a.cols + CG - 1) / CG, a.H, R),    \
                               dim3(256), 0, stream, a);                                                                    \
    } while (0)
    if (a.dk <= 64) IC_MM(16, 4);
    else if (a.dk <= 128) IC_MM(16, 8);
    else if (a.dk <= 256) IC_MM(16, 16);
    else if (a.dk <= 512) IC_MM(64, 8);
    else if (a.dk <= 1024) IC_MM(64, 16);
    else return IC_ERR_TOO_LARGE;
#undef IC_MM
    return ic_launch_status();
}

// dtype: q's, k's and v's (float32 with the delta rule).  single: every request brings one token (ic_matrix_step's kernel).
IC_EXPORT int ic_matrix_memory(const void* q, int q_stride, const void* k, int k_stride, const void* v, int v_stride, int dtype,
                               const float* decay, int per_channel, const float* scale, int delta, int H, int per, int dk, int dv,
                               float q_scale, float* out, float* extra_out, float* state, long long state_stride,
                               const int* req_start, const int* state_slots, int R, int single, int columns_a_thread,
                               hipStream_t stream) {
    if (R <= 0) return IC_OK;
    if (H <= 0 || per <= 0 || H % per || dk <= 0 || dv <= 0 || !decay || !state || !out || R > 65535 || H > 65535) return IC_ERR_ARG;
    if (columns_a_thread != 1 && columns_a_thread != 2) return IC_ERR_ARG;
    const auto aligned = [](const void* p, long long stride, int elem) { return ((uintptr_t)p % 16) == 0 && stride * elem % 16 == 0; };
    const int es = dtype == IC_F32 ? 4 : 2;
    MatrixMemoryArgs a{q, k, v, q_stride, k_stride, v_stride, decay, scale, H, per, dk, dv, dv + (extra_out ? 1 : 0), q_scale, out,
                       extra_out, state, state_stride, req_start, state_slots, 0};
    a.vec = dk % (16 / es) == 0 && dk % 4 == 0 && aligned(q, q_stride, es) && aligned(k, k_stride, es) && aligned(state, state_stride, 4) &&
            (!per_channel || aligned(decay, (long long)H * dk, 4));
    if (delta) {
        if (dtype != IC_F32 || extra_out) return IC_ERR_UNSUPPORTED;
        return per_channel ? matrix_memory_launch<float, true, true>(a, R, single, columns_a_thread, stream)
                           : matrix_memory_launch<float, true, false>(a, R, single, columns_a_thread, stream);
    }
    if (dtype == IC_F32)
        return per_channel ? matrix_memory_launch<float, false, true>(a, R, single, columns_a_thread, stream)
                           : matrix_memory_launch<float, false, false>(a, R, single, columns_a_thread, stream);
    if (dtype == IC_BF16)
        return per_channel ? matrix_memory_launch<bf16, false, true>(a, R, single, columns_a_thread, stream)
                           : matrix_memory_launch<bf16, false, false>(a, R, single, columns_a_thread, stream);
    return IC_ERR_UNSUPPORTED;
}

// ---------------------------------------------------------------------------------------------
// out = rms(y / den) * w * gate(z) head by head, den = max(|num[t, h]|, floor[t, h]) + 1e-6 (num null: 1); gate 0 sigmoid,
// 1 silu.  w has w_heads * dv entries (w_heads H, or 1: shared by the heads).  A wave per (token, head).
// ---------------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
gated_head_norm_kernel(const float* __restrict__ y, const float* __restrict__ num, const float* __restrict__ floor_,
                       const T* __restrict__ z, int z_stride, const float* __restrict__ w, int w_shared, int H, int dv, float eps,
                       T* __restrict__ out, int gate, int n_heads_total) {
    const int lane = threadIdx.x & 63, item = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    if (item >= n_heads_total) return;
    const int t = item / H, h = item - t * H;
    const float* yr = y + (size_t)item * dv;
    const T* zr = z + (size_t)t * z_stride + (size_t)h * dv;
    const float* wr = w + (w_shared ? 0 : (size_t)h * dv);
    T* o = out + (size_t)item * dv;
    const float inv = num ? 1.0f / (fmaxf(fabsf(num[item]), floor_[item]) + 1e-6f) : 1.f;
    constexpr int KEEP = 4;
    float keep[KEEP];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
        const int e = lane + 64 * j;
        keep[j] = e < dv ? yr[e] * inv : 0.f;
        ss += keep[j] * keep[j];
    }
    for (int e = lane + 64 * KEEP; e < dv; e += 64) { const float v = yr[e] * inv; ss += v * v; }
    const float r = 1.0f / sqrtf(wave_sum(ss) / (float)dv + eps);
    auto put = [&](int e, float v) {
        const float g = to_f32(zr[e]);
        o[e] = from_f32<T>(v * r * wr[e] * (gate ? mm_silu_fast(g) : mm_sigmoid_fast(g)));
    };
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
        const int e = lane + 64 * j;
        if (e < dv) put(e, keep[j]);
    }
    for (int e = lane + 64 * KEEP; e < dv; e += 64) put(e, yr[e] * inv);
}

IC_EXPORT int ic_gated_head_norm(const float* y, const float* num, const float* floor_, const void* z, int z_stride, int dtype,
                                 const float* w, int w_shared, int T, int H, int dv, float eps, void* out, int gate,
                                 hipStream_t stream) {
    if (T <= 0) return IC_OK;
    if (H <= 0 || dv <= 0 || gate < 0 || gate > 1 || (num && !floor_)) return IC_ERR_ARG;
    const long long items = (long long)T * H;
    if (items > 0x7fffffff) return IC_ERR_ARG;
    dim3 grid((unsigned)((items + 3) / 4)), block(256);
    if (dtype == IC_F32)
        hipLaunchKernelGGL(gated_head_norm_kernel<float>, grid, block, 0, stream, y, num, floor_, (const float*)z, z_stride, w, w_shared,
                           H, dv, eps, (float*)out, gate, (int)items);
    else if (dtype == IC_BF16)
        hipLaunchKernelGGL(gated_head_norm_kernel<bf16>, grid, block, 0, stream, y, num, floor_, (const bf16*)z, z_stride, w, w_shared, H,
                           dv, eps, (bf16*)out, gate, (int)items);
    else
        return IC_ERR_UNSUPPORTED;
    return ic_launch_status();
}
