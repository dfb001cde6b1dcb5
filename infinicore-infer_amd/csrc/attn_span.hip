// Attention over the paged cache for mixers whose keys and values have different sizes per head and
// whose queries see a SPAN of the keys: the last `window` keys (window 0: all earlier keys) plus the
// first `keep_first` keys of the sequence, which are never dropped.  Query at position i sees key j when
//     j <= i  and  (window == 0  or  i - j < window  or  j < keep_first).
// `sink` adds one term to the softmax's denominator that has no value, exp(0) or, with `sinks` (one float32
// per head, a learned number), exp(sinks[h]):
//     p_j = exp(s_j) / (exp(sink_h) + sum_j exp(s_j)).
// `softcap` c > 0 bounds the scaled score before the softmax: s <- c tanh(s / c).  The sink is neither scaled nor capped.
// `slopes` (nullable, one float32 per head): slopes[h] * (i - j) is then taken off the score (a distance bias, behind the cap).
// `gate` (nullable): the result is multiplied element by element with sigmoid(gate[t, h * dv + d]).
// Scores, the running softmax and the sums are float32.
//
// Cache layout of one layer: K plane [num_pages, n_kv_heads, page_size, dk], V plane [.., dv].
//
// This file holds the general kernel (any sizes, float32 or bfloat16), which is also the yardstick of
// the others, a split-key kernel for single new tokens and a matrix-core kernel for prompt portions
// (key and value sizes 32, 64 or 128 each, and in a padded form every size up to 128 of whole 16-byte pieces).
#include "attn_span_prefill.h"

constexpr int kSpanMaxDim = 512;

// The visible keys of a query at `pos` as two runs: [0, n_kept) and [lo, pos].
struct SpanRuns {
    int n_kept;   // keys 0 .. n_kept-1 (the kept first keys that lie before the window)
    int lo;       // first key of the window
    int total;    // number of visible keys
};
__device__ __forceinline__ SpanRuns span_runs(int pos, int window, int keep_first) {
    SpanRuns r;
    r.lo = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
    r.n_kept = keep_first < r.lo ? keep_first : r.lo;
    if (r.n_kept < 0) r.n_kept = 0;
    r.total = r.n_kept + (pos - r.lo + 1);
    return r;
}
__device__ __forceinline__ int span_key(const SpanRuns& r, int i) { return i < r.n_kept ? i : r.lo + (i - r.n_kept); }

// One wave per (token, head): walks the visible keys 64 at a time.
template <typename T>
__global__ void __launch_bounds__(64)
attn_span_generic_kernel(const T* __restrict__ q, int q_stride, T* __restrict__ out, int out_stride,
                         const T* __restrict__ gate, int gate_stride,
                         const T* __restrict__ kcache, const T* __restrict__ vcache,
                         const int* __restrict__ block_tables, int bt_stride,
                         const int* __restrict__ token_req, const int* __restrict__ positions,
                         int nh, int nkvh, int dk, int dv, int page_size, float scale, int window, int keep_first,
                         int sink, const float* __restrict__ sinks, float softcap, const float* __restrict__ slopes) {
    __shared__ float qs[kSpanMaxDim];
    __shared__ float ps[64];
    __shared__ long long vrow[64];

    const int h = blockIdx.x % nh, t = blockIdx.x / nh, lane = threadIdx.x;
    const int kvh = h / (nh / nkvh);
    const int pos = positions[t];
    const int* bt = block_tables + (size_t)token_req[t] * bt_stride;
    const T* qp = q + (size_t)t * q_stride + (size_t)h * dk;
    for (int d = lane; d < dk; d += 64) qs[d] = to_f32(qp[d]);
    __syncthreads();

    const SpanRuns runs = span_runs(pos, window, keep_first);
    const int nd = (dv + 63) / 64;
    float acc[kSpanMaxDim / 64];
#pragma unroll
    for (int i = 0; i < kSpanMaxDim / 64; ++i) acc[i] = 0.f;
    float m = -INFINITY, l = 0.f;

    for (int ib = 0; ib < runs.total; ib += 64) {
        const int idx = ib + lane;
        const bool valid = idx < runs.total;
        float s = -INFINITY;
        long long vbase = 0;
        if (valid) {
            const int key = span_key(runs, idx);
            const int pg = bt[key / page_size];
            const int off = key % page_size;
            const long long rowi = ((long long)pg * nkvh + kvh) * page_size + off;
            vbase = rowi * dv;
            const T* kp = kcache + rowi * dk;
            float dot = 0.f;
            for (int d = 0; d < dk; ++d) dot += qs[d] * to_f32(kp[d]);
            s = dot * scale;
            if (softcap > 0.f) s = softcap * tanhf(s / softcap);
            if (slopes) s -= slopes[h] * (float)(pos - key);
        }
        const float m_new = fmaxf(m, wave_max(s));       // lane 0 of every chunk is valid: m_new is finite
        const float p = valid ? expf(s - m_new) : 0.f;
        const float corr = expf(m - m_new);               // exp(-inf) = 0 on the first chunk
        l = l * corr + wave_sum(p);
        m = m_new;
        __syncthreads();
        ps[lane] = p;
        vrow[lane] = vbase;
        __syncthreads();
        const int nk = (runs.total - ib < 64) ? runs.total - ib : 64;
#pragma unroll
        for (int i = 0; i < kSpanMaxDim / 64; ++i) {
            if (i < nd) {
                const int d = lane + 64 * i;
                float a = acc[i] * corr;
                if (d < dv)
                    for (int kk = 0; kk < nk; ++kk) a += ps[kk] * to_f32(vcache[vrow[kk] + d]);
                acc[i] = a;
            }
        }
    }
    if (sink) {                                           // the term exp(sink - m) joins the denominator
        const float sv = sinks ? sinks[h] : 0.f;
        const float m_new = fmaxf(m, sv);
        const float corr = expf(m - m_new);
        l = l * corr + expf(sv - m_new);
#pragma unroll
        for (int i = 0; i < kSpanMaxDim / 64; ++i) acc[i] *= corr;
    }
    T* op = out + (size_t)t * out_stride + (size_t)h * dv;
    const T* gp = gate ? gate + (size_t)t * gate_stride + (size_t)h * dv : nullptr;
    const float inv = 1.0f / l;
#pragma unroll
    for (int i = 0; i < kSpanMaxDim / 64; ++i) {
        const int d = lane + 64 * i;
        if (i < nd && d < dv) {
            float o = acc[i] * inv;
            if (gp) o *= 1.0f / (1.0f + expf(-to_f32(gp[d])));
            op[d] = from_f32<T>(o);
        }
    }
}

IC_EXPORT int ic_attn_span_generic(const void* q, int q_stride, void* out, int out_stride, const void* gate,
                                   int gate_stride, int dtype, const void* kcache, const void* vcache,
                                   const int* block_tables, int bt_stride, const int* token_req, const int* positions,
                                   int T, int nh, int nkvh, int dk, int dv, int page_size, float scale, int window,
                                   int keep_first, int sink, const float* sinks, float softcap, const float* slopes, hipStream_t stream) {
    if (T <= 0) return IC_OK;
    if (nh <= 0 || nkvh <= 0 || nh % nkvh || dk <= 0 || dk > kSpanMaxDim || dv <= 0 || dv > kSpanMaxDim ||
        page_size <= 0 || window < 0 || keep_first < 0)
        return IC_ERR_ARG;
    if ((long long)T * nh > 0x7fffffffLL) return IC_ERR_ARG;
    dim3 grid((unsigned)(T * nh)), block(64);
    if (dtype == IC_F32)
        hipLaunchKernelGGL(attn_span_generic_kernel<float>, grid, block, 0, stream, (const float*)q, q_stride, (float*)out,
                           out_stride, (const float*)gate, gate_stride, (const float*)kcache, (const float*)vcache,
                           block_tables, bt_stride, token_req, positions, nh, nkvh, dk, dv, page_size, scale, window,
                           keep_first, sink, sinks, softcap, slopes);
    else if (dtype == IC_BF16)
        hipLaunchKernelGGL(attn_span_generic_kernel<bf16>, grid, block, 0, stream, (const bf16*)q, q_stride, (bf16*)out,
                           out_stride, (const bf16*)gate, gate_stride, (const bf16*)kcache, (const bf16*)vcache,
                           block_tables, bt_stride, token_req, positions, nh, nkvh, dk, dv, page_size, scale, window,
                           keep_first, sink, sinks, softcap, slopes);
    else
        return IC_ERR_UNSUPPORTED;
    return ic_launch_status();
}

// =============================================================================================
// Single new tokens (decoding), split over the visible keys so that few requests fill the chip.
//
// Pass 1, grid (splits, kv heads, tokens), 256 threads: the visible keys of a token are numbered
// 0 .. total-1 (the kept first keys, then the window); a block streams its share once and serves
// every query head of the kv head, GQ (1, 2 or 4) at a time.  DK/VEC lanes share a key (VEC = 16 bytes of
// elements), so a wave reads whole contiguous rows; the same lanes read the value row in pieces
// of 16 bytes (a lane takes pieces sub, sub + LPK, .. when values are wider than keys, and none
// when its piece lies beyond a narrower value row).  Every lane keeps a float32 running softmax
// (base 2) for its keys; they are merged across the lane groups, the waves and, in pass 2, the
// splits, where the sink joins the denominator and the gate is applied.
// =============================================================================================
constexpr int kSdThreads = 256;
constexpr int kSdWaves = 4;
constexpr int kSdUnroll = 4;    // keys a lane group has in flight

template <typename T> struct SpanVec;
template <> struct SpanVec<float> {
    static constexpr int N = 4;
    __device__ static void load(const float* p, float* o) {
        const uint4 v = load_stream16(p);
        o[0] = __uint_as_float(v.x); o[1] = __uint_as_float(v.y); o[2] = __uint_as_float(v.z); o[3] = __uint_as_float(v.w);
    }
};
template <> struct SpanVec<bf16> {
    static constexpr int N = 8;
    __device__ static void load(const bf16* p, float* o) {
        const uint4 v = load_stream16(p);
        o[0] = __uint_as_float(v.x << 16); o[1] = __uint_as_float(v.x & 0xffff0000u);
        o[2] = __uint_as_float(v.y << 16); o[3] = __uint_as_float(v.y & 0xffff0000u);
        o[4] = __uint_as_float(v.z << 16); o[5] = __uint_as_float(v.z & 0xffff0000u);
        o[6] = __uint_as_float(v.w << 16); o[7] = __uint_as_float(v.w & 0xffff0000u);
    }
};

// PAD: the true sizes dk <= DK and dv <= DV (whole pieces of VEC) lie in memory, the rest counts as zero.
template <typename T, int DK, int DV, int GQ, bool PAD>
__global__ void __launch_bounds__(kSdThreads)
attn_span_decode_kernel(const T* __restrict__ q, int q_stride, const T* __restrict__ kcache, const T* __restrict__ vcache,
                        const int* __restrict__ block_tables, int bt_stride, const int* __restrict__ tok_list,
                        const int* __restrict__ token_req, const int* __restrict__ positions,
                        float* __restrict__ part_acc, float* __restrict__ part_ml, int nh, int nkvh, int page_size,
                        float scale, int window, int keep_first, int nsplit, int sink, const float* __restrict__ sinks,
                        float softcap, T* __restrict__ final_out, int out_stride, const T* __restrict__ gate, int gate_stride,
                        const float* __restrict__ slopes, int dk_true, int dv_true) {
    constexpr int VEC = SpanVec<T>::N;
    constexpr int LPK = DK / VEC;                  // lanes per key
    constexpr int LPV = DV / VEC;                  // 16-byte pieces of a value row
    constexpr int KPW = 64 / LPK;                  // keys per wave per step
    constexpr int NVS = (LPV + LPK - 1) / LPK;     // value pieces per lane
    static_assert(DK % VEC == 0 && DV % VEC == 0 && 64 % LPK == 0 && LPK <= 64, "sizes must split a wave evenly");
    const int dk = PAD ? dk_true : DK, dv = PAD ? dv_true : DV;

    __shared__ float sm_acc[kSdWaves][GQ][DV];
    __shared__ float sm_ml[kSdWaves][GQ][2];

    const int split = blockIdx.x, kvh = blockIdx.y, n = blockIdx.z;
    const int t = tok_list ? tok_list[n] : n;
    const int g = nh / nkvh;
    const int pos = positions[t];
    const int* bt = block_tables + (size_t)token_req[t] * bt_stride;
    const SpanRuns runs = span_runs(pos, window, keep_first);
    const int per = (runs.total + nsplit - 1) / nsplit;
    const int lo = split * per;
    int hi = lo + per;
    if (hi > runs.total) hi = runs.total;

    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int sub = lane % LPK, grp = lane / LPK;
    // scores in units of log 2; with a cap c the query carries scale / c and the score becomes (c log2 e) tanh(.)
    const float qscale = softcap > 0.f ? scale / softcap : scale * kLog2e;
    const float cap2 = softcap * kLog2e;

    for (int h0 = 0; h0 < g; h0 += GQ) {
        float qv[GQ][VEC], acc[GQ][NVS * VEC], m[GQ], l[GQ], sl[GQ];
#pragma unroll
        for (int j = 0; j < GQ; ++j) {
            m[j] = -INFINITY; l[j] = 0.f;
            const int hh = (h0 + j < g) ? h0 + j : g - 1;
            if (PAD && sub * VEC >= dk) {
#pragma unroll
                for (int i = 0; i < VEC; ++i) qv[j][i] = 0.f;
            } else {
                SpanVec<T>::load(q + (size_t)t * q_stride + (size_t)(kvh * g + hh) * dk + sub * VEC, qv[j]);
            }
            sl[j] = slopes ? slopes[kvh * g + hh] * kLog2e : 0.f;
#pragma unroll
            for (int i = 0; i < VEC; ++i) qv[j][i] *= qscale;
#pragma unroll
            for (int i = 0; i < NVS * VEC; ++i) acc[j][i] = 0.f;
        }
        // The page ids of an iteration's keys are looked up one iteration ahead: an iteration then waits for one trip to
        // memory (its rows), not for two in a row (page id, then row).
        constexpr int STEP = kSdUnroll * KPW * kSdWaves;
        int keyn[kSdUnroll], pgn[kSdUnroll];
        auto look = [&](int ib) {
#pragma unroll
            for (int u = 0; u < kSdUnroll; ++u) {
                const int idx = ib + u * KPW * kSdWaves;
                keyn[u] = span_key(runs, idx < hi ? idx : hi - 1);         // a stand-in key that is a real one
                pgn[u] = bt[keyn[u] / page_size];
            }
        };
        const int ib0 = lo + wave * KPW + grp;
        if (lo < hi) look(ib0);
        for (int ib = ib0; ib - grp - wave * KPW < hi; ib += STEP) {
            float kf[kSdUnroll][VEC], vf[kSdUnroll][NVS * VEC];
            bool ok[kSdUnroll];
            float back[kSdUnroll];                              // distance to the key
#pragma unroll
            for (int u = 0; u < kSdUnroll; ++u) {
                ok[u] = ib + u * KPW * kSdWaves < hi;
                back[u] = (float)(pos - keyn[u]);
                const size_t rowi = ((size_t)pgn[u] * nkvh + kvh) * page_size + (keyn[u] % page_size);
                if (PAD && sub * VEC >= dk) {
#pragma unroll
                    for (int i = 0; i < VEC; ++i) kf[u][i] = 0.f;
                } else {
                    SpanVec<T>::load(kcache + rowi * dk + sub * VEC, kf[u]);
                }
#pragma unroll
                for (int s = 0; s < NVS; ++s) {
                    if (PAD ? (sub + s * LPK) * VEC < dv : sub + s * LPK < LPV) SpanVec<T>::load(vcache + rowi * dv + (sub + s * LPK) * VEC, vf[u] + s * VEC);
                    else
#pragma unroll
                        for (int i = 0; i < VEC; ++i) vf[u][s * VEC + i] = 0.f;
                }
            }
            if (ib + STEP - grp - wave * KPW < hi) look(ib + STEP);
#pragma unroll
            for (int j = 0; j < GQ; ++j) {
                float s[kSdUnroll];
                float mx = m[j];
#pragma unroll
                for (int u = 0; u < kSdUnroll; ++u) {
                    float d = 0.f;
#pragma unroll
                    for (int i = 0; i < VEC; ++i) d += qv[j][i] * kf[u][i];
                    d = group_sum<LPK>(d);                  // over the lanes that share the key (DPP steps inside a row of 16 lanes)
                    if (softcap > 0.f) {
                        // 16-bit keys: tanh(z) = 1 - 2 / (1 + e^(2z)), a last place of the cap off; finite for every z
                        if (sizeof(T) == 2) d = cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(2.f * kLog2e * d));
                        else d = cap2 * tanhf(d);
                    }
                    d -= sl[j] * back[u];
                    s[u] = ok[u] ? d : -INFINITY;
                    mx = fmaxf(mx, s[u]);
                }
                if (mx == -INFINITY) continue;          // this lane group has seen no key yet
                const float corr = __builtin_amdgcn_exp2f(m[j] - mx);
                float lsum = l[j] * corr;
#pragma unroll
                for (int i = 0; i < NVS * VEC; ++i) acc[j][i] *= corr;
#pragma unroll
                for (int u = 0; u < kSdUnroll; ++u) {
                    const float p = __builtin_amdgcn_exp2f(s[u] - mx);      // 0 for a stand-in key
                    lsum += p;
#pragma unroll
                    for (int i = 0; i < NVS * VEC; ++i) acc[j][i] += p * vf[u][i];
                }
                l[j] = lsum;
                m[j] = mx;
            }
        }
        // merge the lane groups of the wave (lanes with the same `sub`)
#pragma unroll
        for (int j = 0; j < GQ; ++j) {
#pragma unroll
            for (int o = LPK; o < 64; o <<= 1) {
                const float mb = __shfl_xor(m[j], o, kWave);
                const float lb = __shfl_xor(l[j], o, kWave);
                const float mn = fmaxf(m[j], mb);
                const float ca = (mn == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(m[j] - mn);
                const float cb = (mn == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(mb - mn);
                l[j] = l[j] * ca + lb * cb;
#pragma unroll
                for (int i = 0; i < NVS * VEC; ++i) acc[j][i] = acc[j][i] * ca + __shfl_xor(acc[j][i], o, kWave) * cb;
                m[j] = mn;
            }
        }
        __syncthreads();                                // LDS free from the previous chunk of heads
        if (grp == 0) {
#pragma unroll
            for (int j = 0; j < GQ; ++j) {
#pragma unroll
                for (int s = 0; s < NVS; ++s)
                    if (sub + s * LPK < LPV)
#pragma unroll
                        for (int i = 0; i < VEC; ++i) sm_acc[wave][j][(sub + s * LPK) * VEC + i] = acc[j][s * VEC + i];
                if (sub == 0) { sm_ml[wave][j][0] = m[j]; sm_ml[wave][j][1] = l[j]; }
            }
        }
        __syncthreads();
        for (int idx = threadIdx.x; idx < GQ * DV; idx += kSdThreads) {
            const int j = idx / DV, d = idx - j * DV;
            if (h0 + j >= g || (PAD && d >= dv)) continue;
            float mm = -INFINITY;
            for (int w = 0; w < kSdWaves; ++w) mm = fmaxf(mm, sm_ml[w][j][0]);
            float a = 0.f, ll = 0.f;
            if (mm != -INFINITY) {
                for (int w = 0; w < kSdWaves; ++w) {
                    const float c = __builtin_amdgcn_exp2f(sm_ml[w][j][0] - mm);
                    a += sm_acc[w][j][d] * c;
                    ll += sm_ml[w][j][1] * c;
                }
            }
            const int h = kvh * g + h0 + j;
            if (final_out) {                            // a single split: this is the result, no second pass
                if (sink) {
                    const float sv = sinks ? sinks[h] * kLog2e : 0.f;
                    const float mf = fmaxf(mm, sv), c = __builtin_amdgcn_exp2f(mm - mf);
                    a *= c;
                    ll = ll * c + __builtin_amdgcn_exp2f(sv - mf);
                }
                float o = a / ll;
                if (gate) o *= sigmoid_f(to_f32(gate[(size_t)t * gate_stride + (size_t)h * dv + d]));
                final_out[(size_t)t * out_stride + (size_t)h * dv + d] = from_f32<T>(o);
                continue;
            }
            const size_t pidx = ((size_t)n * nh + h) * nsplit + split;
            part_acc[pidx * dv + d] = a;
            if (d == 0) { part_ml[pidx * 2] = mm; part_ml[pidx * 2 + 1] = ll; }      // the maximum in units of log 2
        }
    }
}

// Pass 2, grid (tokens * heads), one thread per value entry: merges the splits, lets the sink join, applies the gate.
template <typename T>
__global__ void attn_span_reduce_kernel(const float* __restrict__ part_acc, const float* __restrict__ part_ml,
                                        const int* __restrict__ tok_list, T* __restrict__ out, int out_stride,
                                        const T* __restrict__ gate, int gate_stride, int nh, int dv, int nsplit, int sink,
                                        const float* __restrict__ sinks) {
    const int n = blockIdx.x / nh, h = blockIdx.x % nh;
    const int t = tok_list ? tok_list[n] : n;
    const size_t base = ((size_t)n * nh + h) * nsplit;
    const float sv = (sink && sinks) ? sinks[h] * kLog2e : 0.f;      // in units of log 2, as the partial maxima
    float mm = sink ? sv : -INFINITY;
    for (int s = 0; s < nsplit; ++s) mm = fmaxf(mm, part_ml[(base + s) * 2]);
    float den = sink ? __builtin_amdgcn_exp2f(sv - mm) : 0.f;
    for (int s = 0; s < nsplit; ++s) {
        const float ms = part_ml[(base + s) * 2];
        if (ms != -INFINITY) den += part_ml[(base + s) * 2 + 1] * __builtin_amdgcn_exp2f(ms - mm);
    }
    for (int d = threadIdx.x; d < dv; d += blockDim.x) {
        float a = 0.f;
        for (int s = 0; s < nsplit; ++s) {
            const float ms = part_ml[(base + s) * 2];
            if (ms != -INFINITY) a += part_acc[(base + s) * dv + d] * __builtin_amdgcn_exp2f(ms - mm);
        }
        float o = a / den;
        if (gate) o *= sigmoid_f(to_f32(gate[(size_t)t * gate_stride + (size_t)h * dv + d]));
        out[(size_t)t * out_stride + (size_t)h * dv + d] = from_f32<T>(o);
    }
}

static bool span_dim_ok(int d) { return d == 32 || d == 64 || d == 128; }
// Sizes that the padded kernels take: whole 16-byte pieces, up to 128.
static bool span_dim_padded(int d, int dtype) { return d > 0 && d <= 128 && d % (dtype == IC_F32 ? 4 : 8) == 0; }

IC_EXPORT int ic_attn_span_decode_supported(int dtype, int dk, int dv) {
    return (dtype == IC_F32 || dtype == IC_BF16) && span_dim_padded(dk, dtype) && span_dim_padded(dv, dtype);
}

// How many ways to split the visible keys of n_rows single tokens (<= 32): enough blocks for the chip, at least 128 keys a split.
IC_EXPORT int ic_attn_span_decode_splits(int n_rows, int n_kv_heads, int max_keys, int compute_units) {
    if (n_rows <= 0 || n_kv_heads <= 0) return 1;
    long long blocks = (long long)n_rows * n_kv_heads;
    int want = (int)((2LL * compute_units + blocks - 1) / blocks);
    int most = (max_keys + 127) / 128;
    if (want > most) want = most;
    if (want > 32) want = 32;
    return want < 1 ? 1 : want;
}

struct SpanDecodeArgs {
    const void* q; int q_stride; void* out; int out_stride; const void* gate; int gate_stride;
    const void *kcache, *vcache; const int* block_tables; int bt_stride; const int *tok_list, *token_req, *positions;
    float *part_acc, *part_ml; int n_tok, nh, nkvh, dk, dv, page_size; float scale; int window, keep_first, sink;
    const float* sinks; float softcap; const float* slopes; int nsplit;
};

template <typename T, int DK, int DV, bool PAD>
static int span_decode_launch(const SpanDecodeArgs& a, hipStream_t stream) {
    dim3 grid(a.nsplit, a.nkvh, a.n_tok), block(kSdThreads);
    const int g = a.nh / a.nkvh;
#define IC_SPAN_GQ(GQ)                                                                                                          \
    hipLaunchKernelGGL((attn_span_decode_kernel<T, DK, DV, GQ, PAD>), grid, block, 0, stream, (const T*)a.q, a.q_stride,        \
                       (const T*)a.kcache, (const T*)a.vcache, a.block_tables, a.bt_stride, a.tok_list, a.token_req,            \
                       a.positions, a.part_acc, a.part_ml, a.nh, a.nkvh, a.page_size, a.scale, a.window, a.keep_first, a.nsplit, \
                       a.sink, a.sinks, a.softcap, a.nsplit == 1 ? (T*)a.out : (T*)nullptr, a.out_stride, (const T*)a.gate,     \
                       a.gate_stride, a.slopes, a.dk, a.dv)
    if (g == 1) IC_SPAN_GQ(1);                      // query heads served per walk over the keys: no more than there are
    else if (g == 2) IC_SPAN_GQ(2);
    else IC_SPAN_GQ(4);
#undef IC_SPAN_GQ
    int st = ic_launch_status();
    if (st != IC_OK || a.nsplit == 1) return st;
    hipLaunchKernelGGL(attn_span_reduce_kernel<T>, dim3((unsigned)(a.n_tok * a.nh)), dim3((a.dv + 63) / 64 * 64), 0, stream,
                       a.part_acc, a.part_ml, a.tok_list, (T*)a.out, a.out_stride, (const T*)a.gate, a.gate_stride, a.nh, a.dv,
                       a.nsplit, a.sink, a.sinks);
    return ic_launch_status();
}

template <typename T>
static int span_decode_dims(const SpanDecodeArgs& a, hipStream_t stream) {
#define IC_SPAN_DEC(K, V) \
    if (a.dk == K && a.dv == V) return span_decode_launch<T, K, V, false>(a, stream);
    IC_SPAN_DEC(32, 32) IC_SPAN_DEC(32, 64) IC_SPAN_DEC(32, 128)
    IC_SPAN_DEC(64, 32) IC_SPAN_DEC(64, 64) IC_SPAN_DEC(64, 128)
    IC_SPAN_DEC(128, 32) IC_SPAN_DEC(128, 64) IC_SPAN_DEC(128, 128)
#undef IC_SPAN_DEC
#define IC_SPAN_DEC(K, V) \
    if (a.dk <= K && a.dv <= V) return span_decode_launch<T, K, V, true>(a, stream);
    IC_SPAN_DEC(64, 64) IC_SPAN_DEC(64, 128) IC_SPAN_DEC(128, 64) IC_SPAN_DEC(128, 128)
#undef IC_SPAN_DEC
    return IC_ERR_UNSUPPORTED;
}

// tok_list (nullable): the rows that are single tokens, int32 [n_tok].  part_acc: float32 [n_tok, nh, nsplit, dv]; part_ml: [n_tok, nh, nsplit, 2].
IC_EXPORT int ic_attn_span_decode(const void* q, int q_stride, void* out, int out_stride, const void* gate, int gate_stride,
                                  int dtype, const void* kcache, const void* vcache, const int* block_tables, int bt_stride,
                                  const int* tok_list, const int* token_req, const int* positions, float* part_acc,
                                  float* part_ml, int n_tok, int nh, int nkvh, int dk, int dv, int page_size, float scale,
                                  int window, int keep_first, int sink, const float* sinks, float softcap, const float* slopes,
                                  int nsplit, hipStream_t stream) {
    if (n_tok <= 0) return IC_OK;
    if (nh <= 0 || nkvh <= 0 || nh % nkvh || page_size <= 0 || window < 0 || keep_first < 0 || nsplit < 1 || nsplit > 32)
        return IC_ERR_ARG;
    if (nkvh > 65535 || n_tok > 65535) return IC_ERR_ARG;
    if (nsplit > 1 && (part_acc == nullptr || part_ml == nullptr)) return IC_ERR_ARG;
    if (!ic_attn_span_decode_supported(dtype, dk, dv)) return IC_ERR_UNSUPPORTED;
    const SpanDecodeArgs a{q, q_stride, out, out_stride, gate, gate_stride, kcache, vcache, block_tables, bt_stride, tok_list,
                           token_req, positions, part_acc, part_ml, n_tok, nh, nkvh, dk, dv, page_size, scale, window, keep_first,
                           sink, sinks, softcap, slopes, nsplit};
    return dtype == IC_F32 ? span_decode_dims<float>(a, stream) : span_decode_dims<bf16>(a, stream);
}

IC_EXPORT int ic_attn_span_prefill_supported(int dtype, int dk, int dv) {
    return dtype == IC_BF16 && span_dim_padded(dk, dtype) && span_dim_padded(dv, dtype);
}

// tiles: int32 [n_tiles, 4] = (request row, first token row, rows <= 128, first position).  Pages of a power of two.  Strides in elements; q rows, out rows and
// gate rows must start on 16-, 8- and 8-byte boundaries.  scale > 0.
IC_EXPORT int ic_attn_span_prefill(const void* q, int q_stride, void* out, int out_stride, const void* gate, int gate_stride,
                                   int dtype, const void* kcache, const void* vcache, const int* block_tables, int bt_stride,
                                   const int* tiles, int n_tiles, int nh, int nkvh, int dk, int dv, int page_size, float scale,
                                   int window, int keep_first, int sink, const float* sinks, float softcap, const float* slopes,
                                   hipStream_t stream) {
    if (n_tiles <= 0) return IC_OK;
    if (nh <= 0 || nkvh <= 0 || nh % nkvh || page_size <= 0 || window < 0 || keep_first < 0 || !(scale > 0.f)) return IC_ERR_ARG;
    if (!ic_attn_span_prefill_supported(dtype, dk, dv) || (page_size & (page_size - 1))) return IC_ERR_UNSUPPORTED;
    int page_shift = 0;
    while ((1 << page_shift) < page_size) ++page_shift;
    if ((q_stride & 7) || (out_stride & 3) || (gate && (gate_stride & 3)) || ((uintptr_t)q & 15) || ((uintptr_t)out & 7) ||
        ((uintptr_t)gate & 7) || ((uintptr_t)kcache & 15) || ((uintptr_t)vcache & 15))
        return IC_ERR_ARG;
    if ((long long)n_tiles * nh > 0x7fffffffLL) return IC_ERR_ARG;
    dim3 grid((unsigned)(n_tiles * nh)), block(256);
    const float c = softcap > 0.f ? softcap * kLog2e : scale * kLog2e;
    const float cap_in = softcap > 0.f ? scale / softcap : 0.f;
    const SpanSizes z{dk, dv, 0, 0, 0, 0, 0, nullptr, int4{0, 0, 0, 0}};
#define IC_SPAN_PRE(K, V, MODE)                                                                                               \
    {                                                                                                                         \
        hipLaunchKernelGGL((attn_span_prefill_kernel<K, V, MODE>), grid, block, 0, stream, (const uint16_t*)q, q_stride,      \
                           (uint16_t*)out, out_stride, (const uint16_t*)gate, gate_stride, (const uint16_t*)kcache,           \
                           (const uint16_t*)vcache, block_tables, bt_stride, (const int4*)tiles, nh, nkvh, page_shift, c,      \
                           window, keep_first, sink, sinks, cap_in, slopes, z);                                               \
        return ic_launch_status();                                                                                            \
    }
#define IC_SPAN_EXACT(K, V) if (dk == K && dv == V) IC_SPAN_PRE(K, V, kSpanPaged)
    IC_SPAN_EXACT(32, 32) IC_SPAN_EXACT(32, 64) IC_SPAN_EXACT(32, 128)
    IC_SPAN_EXACT(64, 32) IC_SPAN_EXACT(64, 64) IC_SPAN_EXACT(64, 128)
    IC_SPAN_EXACT(128, 32) IC_SPAN_EXACT(128, 64) IC_SPAN_EXACT(128, 128)
#undef IC_SPAN_EXACT
#define IC_SPAN_WITHIN(K, V) if (dk <= K && dv <= V) IC_SPAN_PRE(K, V, kSpanPadded)
    IC_SPAN_WITHIN(64, 64) IC_SPAN_WITHIN(64, 128) IC_SPAN_WITHIN(96, 96) IC_SPAN_WITHIN(128, 64) IC_SPAN_WITHIN(128, 128)
#undef IC_SPAN_WITHIN
#undef IC_SPAN_PRE
    return IC_ERR_UNSUPPORTED;
}
