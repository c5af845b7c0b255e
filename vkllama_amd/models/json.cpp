#include "models/json.h"
#include "absl/strings/str_format.h"
#include <cmath>
#include <cstdlib>
#include <cstring>

namespace vkllama
{
struct JsonParser
{
  const char *p, *end;
  int depth = 0;

  void
  space ()
  {
    while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r'))
      ++p;
  }

  bool
  word (const char *w)
  {
    const size_t n = strlen (w);
    if ((size_t)(end - p) < n || strncmp (p, w, n) != 0)
      return false;
    p += n;
    return true;
  }

  static void
  append_utf8 (std::string &s, uint32_t c)
  {
    if (c < 0x80)
      s += (char)c;
    else if (c < 0x800)
      s += (char)(0xc0 | (c >> 6)), s += (char)(0x80 | (c & 63));
    else if (c < 0x10000)
      s += (char)(0xe0 | (c >> 12)), s += (char)(0x80 | ((c >> 6) & 63)), s += (char)(0x80 | (c & 63));
    else
      s += (char)(0xf0 | (c >> 18)), s += (char)(0x80 | ((c >> 12) & 63)),
          s += (char)(0x80 | ((c >> 6) & 63)), s += (char)(0x80 | (c & 63));
  }

  bool
  hex4 (uint32_t &v)
  {
    v = 0;
    if (end - p < 4)
      return false;
    for (int i = 0; i < 4; ++i, ++p)
      {
        const char c = *p;
        const int d = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
        if (d < 0)
          return false;
        v = v * 16 + (uint32_t)d;
      }
    return true;
  }

  bool
  text (std::string &s)
  {
    if (p >= end || *p != '"')
      return false;
    for (++p; p < end && *p != '"';)
      {
        if (*p != '\\')
          {
            s += *p++;
            continue;
          }
        if (++p >= end)
          return false;
        const char c = *p++;
        const char *from = "\"\\/bfnrt", *to = "\"\\/\b\f\n\r\t";
        if (const char *at = c ? strchr (from, c) : nullptr)
          s += to[at - from];
        else if (c == 'u')
          {
            uint32_t v, w;
            if (!hex4 (v))
              return false;
            if (v >= 0xd800 && v < 0xdc00)
              {
                if (end - p < 2 || p[0] != '\\' || p[1] != 'u')
                  return false;
                p += 2;
                if (!hex4 (w) || w < 0xdc00 || w > 0xdfff)
                  return false;
                v = 0x10000 + ((v - 0xd800) << 10) + (w - 0xdc00);
              }
            append_utf8 (s, v);
          }
        else
          return false;
      }
    if (p >= end)
      return false;
    ++p;
    return true;
  }

  bool
  value (Json &v)
  {
    if (++depth > 256)
      return false;
    const bool ok = value_ (v);
    --depth;
    space ();
    return ok;
  }

  bool
  value_ (Json &v)
  {
    space ();
    if (p >= end)
      return false;
    if (*p == '{')
      {
        v.kind_ = Json::Object;
        ++p;
        space ();
        if (p < end && *p == '}')
          return ++p, true;
        for (;;)
          {
            std::string name;
            space ();
            if (!text (name))
              return false;
            space ();
            if (p >= end || *p++ != ':' || !value (v.members_[name]))
              return false;
            if (p >= end)
              return false;
            if (*p == '}')
              return ++p, true;
            if (*p++ != ',')
              return false;
          }
      }
    if (*p == '[')
      {
        v.kind_ = Json::Array;
        ++p;
        space ();
        if (p < end && *p == ']')
          return ++p, true;
        for (;;)
          {
            v.items_.emplace_back ();
            if (!value (v.items_.back ()) || p >= end)
              return false;
            if (*p == ']')
              return ++p, true;
            if (*p++ != ',')
              return false;
          }
      }
    if (*p == '"')
      {
        v.kind_ = Json::String;
        return text (v.text_);
      }
    if (word ("null"))
      return true;
    if (word ("true"))
      return v.kind_ = Json::Bool, v.number_ = 1, true;
    if (word ("false"))
      return v.kind_ = Json::Bool, true;
    const char *q = p;
    while (q < end && *q && strchr ("+-.0123456789eE", *q))
      ++q;
    if (q == p)
      return false;
    const std::string num (p, q);
    char *stop = nullptr;
    v.kind_ = Json::Number;
    v.number_ = strtod (num.c_str (), &stop);
    p = q;
    return stop && *stop == 0;
  }
};

absl::StatusOr<Json>
Json::parse (const char *text, size_t n)
{
  JsonParser ps{ text, text + n };
  Json v;
  if (!ps.value (v) || ps.p != ps.end)
    return absl::InvalidArgumentError (absl::StrFormat ("not a JSON document (stopped at byte %zu)",
                                                        (size_t)(ps.p - text)));
  return v;
}

const Json &
Json::operator[] (const std::string &name) const
{
  static const Json none;
  const auto it = members_.find (name);
  return it == members_.end () ? none : it->second;
}

absl::StatusOr<double>
Json::need_number (const std::string &name, const std::string &where) const
{
  const Json &v = (*this)[name];
  if (v.kind_ != Number || !std::isfinite (v.number_))
    return absl::InvalidArgumentError ("configuration: " + where + "." + name + " must be a number");
  return v.number_;
}

absl::StatusOr<int>
Json::need_int (const std::string &name, int lo, const std::string &where) const
{
  const Json &v = (*this)[name];
  if (v.kind_ != Number || v.number_ != std::floor (v.number_) || v.number_ < lo || v.number_ > 2147483647.0)
    return absl::InvalidArgumentError ("configuration: " + where + "." + name + " must be a whole number, at least "
                                       + std::to_string (lo));
  return (int)v.number_;
}

absl::StatusOr<std::string>
Json::need_string (const std::string &name, const std::string &where) const
{
  const Json &v = (*this)[name];
  if (v.kind_ != String)
    return absl::InvalidArgumentError ("configuration: " + where + "." + name + " must be a string");
  return v.text_;
}
}
